// Row kernels of the layered decoders, whose residual stream is fp32: embedding with learned
// positions, grouped RMS norm, and the step between two sublayers (norm of the sublayer's output,
// residual sum, norm of the next sublayer's input) in one launch.  The counterpart for the fp16
// models is rmsnorm_kernel in elementwise.hip.
#include <type_traits>

#include "linear.hpp"
#include "router.hpp"
#include "rownorm.hpp"

using namespace lcu;

namespace {

// x[row] = scale table[token] + pos_table[start + row] (when given), its norm under w0 (when given); h[row] = x[row],
// its norm under w1 when given
template <class T, int NV, int TH>
__global__ __launch_bounds__(TH) void embed_pos_norm_kernel(float* __restrict__ x, T* __restrict__ h,
                                                                     const int* __restrict__ ids, const T* __restrict__ table, float scale,
                                                                     const T* __restrict__ pos_table, const float* __restrict__ w0,
                                                                     const float* __restrict__ w1, const int* __restrict__ start,
                                                                     int n_vocab, int n_pos, row_shape rs) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int r = blockIdx.x;
  const int id = min(max(ids[r], 0), n_vocab - 1);
  row_t<NV, TH> row, at, w, next;
  if (w0) load_row(w, w0, rs);
  if (w1) load_row(next, w1, rs);
  load_row(row, table + (size_t)id * rs.ld, rs);
#pragma unroll
  for (int j = 0; j < NV; ++j) row.v[j] *= scale;
  if (pos_table) {
    load_row(at, pos_table + (size_t)min(max(*start + r, 0), n_pos - 1) * rs.ld, rs);
#pragma unroll
    for (int j = 0; j < NV; ++j) row.v[j] += at.v[j];
  }
  if (w0) scale_row(row, rs, lds, w);
  store_row(x + (size_t)r * rs.ld, row, rs);
  if (!h) return;
  if (w1) scale_row(row, rs, lds, next);
  store_row(h + (size_t)r * rs.ld, row, rs);
}

// what sublayers left for row r: its rows of src.out, and the shared expert's row times its gate
template <int NV, int TH>
__device__ __forceinline__ void load_sum(row_t<NV, TH>& m, row_t<NV, TH>& t, const sublayer_rows& src, int r, const row_shape& rs) {
  const auto from = [&](int k) {
    const size_t at = (size_t)r * src.top + k;
    return src.out + (src.inverse ? (size_t)src.inverse[at] : at) * rs.ld;
  };
  load_row(m, from(0), rs);
  for (int k = 1; k < src.top; ++k) {
    load_row(t, from(k), rs);
#pragma unroll
    for (int j = 0; j < NV; ++j) m.v[j] += t.v[j];
  }
  if (src.shared) {
    const float f = src.shared_gate[r];
    load_row(t, src.shared + (size_t)r * rs.ld, rs);
#pragma unroll
    for (int j = 0; j < NV; ++j) m.v[j] += f * t.v[j];
  }
}

// m = the sublayer's result; x += norm(m) under w_after; h = x, its norm under w_next when given.
template <class T, int NV, int TH>
__global__ __launch_bounds__(TH) void residual_norm_kernel(float* __restrict__ x, T* __restrict__ h,
                                                                    sublayer_rows src, const float* __restrict__ w_after,
                                                                    const float* __restrict__ w_next, row_shape rs) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int r = blockIdx.x;
  row_t<NV, TH> m, t, old;
  load_sum(m, t, src, r, rs);
  float* xr = x + (size_t)r * rs.ld;
  load_row(old, xr, rs);
  load_row(t, w_after, rs);
  scale_row(m, rs, lds, t);
#pragma unroll
  for (int j = 0; j < NV; ++j) m.v[j] += old.v[j];
  store_row(xr, m, rs);
  if (!h) return;
  if (w_next) {
    load_row(t, w_next, rs);
    scale_row(m, rs, lds, t);
  }
  store_row(h + (size_t)r * rs.ld, m, rs);
}

// The step between two sublayers for one row, and the router behind it when there is one: every wavefront
// takes rows of the router's matrix (its first two asked for before the norms are worked out), the first one
// then chooses.
template <int NV>
__global__ __launch_bounds__(STEP_THREADS) void residual_step_kernel(float* __restrict__ x, bf16_t* __restrict__ h, sublayer_rows src,
                                                                     const float* __restrict__ w_after,
                                                                     const float* __restrict__ w_next, row_shape rs, router_step rt) {
  constexpr int TH = STEP_THREADS, AHEAD = 8;  // 16-byte pieces of a router row a lane asks for ahead: 4096 columns
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float z[ROUTER_MAX_ROWS];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  row_t<NV, TH> m, t, old, after, next;
  load_row(after, w_after, rs);
  load_row(old, x, rs);
  if (w_next) load_row(next, w_next, rs);
  load_sum(m, t, src, 0, rs);
  bf16x8_t ahead[2][AHEAD];
  if (rt.w) {
#pragma unroll
    for (int turn = 0; turn < 2; ++turn) {
      const bf16_t* we = rt.w + (size_t)min(wave + turn * TH / WAVE, rt.rows - 1) * rs.ld;
#pragma unroll
      for (int a = 0; a < AHEAD; ++a) ahead[turn][a] = *reinterpret_cast<const bf16x8_t*>(we + min((a * WAVE + lane) * 8, rs.ld - 8));
    }
  }
  scale_row(m, rs, lds, after);
#pragma unroll
  for (int j = 0; j < NV; ++j) m.v[j] += old.v[j];
  store_row(x, m, rs);
  if (!h) return;
  if (w_next) scale_row(m, rs, lds, next);
  store_row(h, m, rs);
  if (!rt.w) return;
  bf16_t* hs = reinterpret_cast<bf16_t*>(lds);  // scale_row is done with it
  store_row(hs, m, rs);
  __syncthreads();
  const auto dot = [&](float s, bf16x8_t wv, int c) {
    const bf16x8_t hv = *reinterpret_cast<const bf16x8_t*>(hs + c);
#pragma unroll
    for (int b = 0; b < 8; ++b) s = fmaf((float)hv[b], (float)wv[b], s);
    return s;
  };
  const auto row = [&](int e, auto&& held) {
    if (e >= rt.rows) return;
    float s = 0.0f;
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      const int c = (a * WAVE + lane) * 8;
      if (c < rs.ld) s = dot(s, held(a, c), c);
    }
    for (int c = (AHEAD * WAVE + lane) * 8; c < rs.ld; c += WAVE * 8) {
      s = dot(s, *reinterpret_cast<const bf16x8_t*>(rt.w + (size_t)e * rs.ld + c), c);
    }
    s = wave_sum(s);
    if (lane == 0) z[e] = s;
  };
  row(wave, [&](int a, int) { return ahead[0][a]; });
  row(wave + TH / WAVE, [&](int a, int) { return ahead[1][a]; });
  for (int e = wave + 2 * TH / WAVE; e < rt.rows; e += TH / WAVE) {
    row(e, [&](int, int c) { return *reinterpret_cast<const bf16x8_t*>(rt.w + (size_t)e * rs.ld + c); });
  }
  __syncthreads();
  if (wave != 0) return;
  if (rt.shared_gate && lane == 0) *rt.shared_gate = sigmoid_f32(z[rt.experts]);
  choose_experts(z, rt.experts, rt.top, rt.expert, rt.weight);
}

// h[i] = norm(x[rows[i]]) under w (rows NULL: row i)
template <class T, int NV, int TH>
__global__ __launch_bounds__(TH) void group_norm_kernel(T* __restrict__ h, const float* __restrict__ x,
                                                                 const int* __restrict__ rows, const float* __restrict__ w,
                                                                 row_shape rs) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int r = rows ? rows[blockIdx.x] : blockIdx.x;
  row_t<NV, TH> row, wr;
  load_row(row, x + (size_t)r * rs.ld, rs);
  load_row(wr, w, rs);
  scale_row(row, rs, lds, wr);
  store_row(h + (size_t)blockIdx.x * rs.ld, row, rs);
}

// calls f with a null pointer of the element type, the pieces of a row and the threads that share it
template <class F>
void with_row_kind(int dtype, int ld, bool single, F&& f) {
  const auto typed = [&](auto nv, auto th) {
    if (dtype == LCU_F32) {
      f((float*)nullptr, nv, th);
    } else {
      f((bf16_t*)nullptr, nv, th);
    }
  };
  if (single) {
    with_step_pieces(ld, [&](auto nv) { typed(nv, std::integral_constant<int, STEP_THREADS>{}); });
  } else {
    with_row_pieces(ld, [&](auto nv) { typed(nv, std::integral_constant<int, ROW_THREADS>{}); });
  }
}

// index = the first maximum of n fp32 values
__global__ __launch_bounds__(1024) void argmax_f32_kernel(int* __restrict__ index, const float* __restrict__ x, int n) {
  __shared__ float sred[16];
  __shared__ int sidx[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  float best = -INFINITY;
  int idx = 0x7fffffff;
  const auto take = [&](float v, int i) {
    if (v > best || (v == best && i < idx)) {
      best = v;
      idx = i;
    }
  };
  const int n4 = (reinterpret_cast<uintptr_t>(x) & 15) == 0 ? n / 4 : 0;
  for (int c0 = 0; c0 < n4; c0 += 8 * 1024) {
    float4_t v[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = load4(x + 4 * (size_t)min(c0 + j * 1024 + tid, n4 - 1));
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int c = min(c0 + j * 1024 + tid, n4 - 1);
#pragma unroll
      for (int e = 0; e < 4; ++e) take(v[j][e], c * 4 + e);
    }
  }
  for (int i = n4 * 4 + tid; i < n; i += 1024) take(x[i], i);
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) {
    const float ob = __shfl_xor(best, off, WAVE);
    const int oi = __shfl_xor(idx, off, WAVE);
    take(ob, oi);
  }
  if (lane == 0) {
    sred[wave] = best;
    sidx[wave] = idx;
  }
  __syncthreads();
  if (tid == 0) {
    for (int w = 1; w < 16; ++w) take(sred[w], sidx[w]);
    *index = idx == 0x7fffffff ? 0 : idx;
  }
}

// One row of n fp32 logits: probs = fp16(softmax(logits / temp)).
__global__ __launch_bounds__(1024) void softmax_f32_kernel(half_t* __restrict__ probs, const float* __restrict__ logits, int n,
                                                           float temp) {
  __shared__ float sred[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  float m = -INFINITY;
  for (int i = tid; i < n; i += 1024) m = fmaxf(m, logits[i]);
  m = wave_max(m);
  if (lane == 0) sred[wave] = m;
  __syncthreads();
  m = sred[0];
  for (int w = 1; w < 16; ++w) m = fmaxf(m, sred[w]);
  __syncthreads();
  float s = 0.0f;
  for (int i = tid; i < n; i += 1024) s += exp_ieee((logits[i] - m) / temp);
  s = wave_sum(s);
  if (lane == 0) sred[wave] = s;
  __syncthreads();
  float total = 0.0f;
#pragma unroll
  for (int w = 0; w < 16; ++w) total += sred[w];
  for (int i = tid; i < n; i += 1024) probs[i] = round_f16(exp_ieee((logits[i] - m) / temp) / total);
}

template <class T>
__global__ void fill_normal_kernel(T* __restrict__ out, size_t rows, int cols, int ld, uint64_t seed, uint64_t stream_id,
                                   float mean, float std) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= rows * (size_t)cols) return;
  // the sum of eight 16-bit fields of two chained splitmix64 hashes, as lcu_fill_normal_f16
  uint64_t z = seed + 0x9E3779B97F4A7C15ull * (stream_id * 0x100000001B3ull + i + 1);
  int S = 0;
#pragma unroll
  for (int k = 0; k < 2; ++k) {
    z = (z ^ (z >> 30)) * 0xBF58476D1CE4E5B9ull;
    z = (z ^ (z >> 27)) * 0x94D049BB133111EBull;
    z ^= z >> 31;
    S += (int)(z & 0xffff) + (int)((z >> 16) & 0xffff) + (int)((z >> 32) & 0xffff) + (int)(z >> 48);
  }
  const float unit = (float)(S - 262140) * 1.8688e-5f;  // unit variance: 1 / sqrt(8 (65536^2 - 1) / 12)
  out[(i / cols) * ld + i % cols] = (T)(mean + std * unit);
}

int check_rows(const char* who, int dtype, int rows, const row_shape& rs) {
  LCU_REQUIRE(dtype == LCU_BF16 || dtype == LCU_F32, "%s: element type %d", who, dtype);
  LCU_REQUIRE(rows >= 0 && rs.width > 0 && rs.ld >= rs.width && rs.ld % 64 == 0 && rs.groups > 0 && rs.width % rs.groups == 0,
              "%s: bad shape rows %d width %d ld %d groups %d", who, rows, rs.width, rs.ld, rs.groups);
  LCU_REQUIRE(rs.width <= ROW_MAX_WIDTH && rs.groups <= ROW_MAX_GROUPS, "%s: width %d (at most %d), groups %d (at most %d)", who,
              rs.width, ROW_MAX_WIDTH, rs.groups, ROW_MAX_GROUPS);
  return LCU_OK;
}

}  // namespace

extern "C" {

int lcu_embed_pos_norm(void* x_dev, void* h_dev, const void* ids_dev, int n_ids, const void* table_dev, int n_vocab,
                       const void* pos_table_dev, int n_pos, const void* start_dev, const void* w_embed_dev,
                       const void* w_next_dev, int dtype, int width, int ld, int groups, float eps, void* stream) {
  LCU_REQUIRE(x_dev && ids_dev && table_dev && pos_table_dev && start_dev && w_embed_dev && (h_dev || !w_next_dev),
              "lcu_embed_pos_norm: null pointer");
  const row_shape rs{width, ld, groups, eps};
  const int rc = check_rows("lcu_embed_pos_norm", dtype, n_ids, rs);
  if (rc) return rc;
  LCU_REQUIRE(n_vocab > 0 && n_pos > 0, "lcu_embed_pos_norm: bad table sizes %d %d", n_vocab, n_pos);
  if (n_ids == 0) return LCU_OK;
  hipStream_t st = as_stream(stream);
  with_row_kind(dtype, ld, n_ids == 1, [&](auto* kind, auto nv, auto th) {
    using T = std::remove_pointer_t<decltype(kind)>;
    embed_pos_norm_kernel<T, decltype(nv)::value, decltype(th)::value><<<n_ids, decltype(th)::value, row_lds_bytes(rs), st>>>(
        (float*)x_dev, (T*)h_dev, (const int*)ids_dev, (const T*)table_dev, 1.0f, (const T*)pos_table_dev, (const float*)w_embed_dev,
        (const float*)w_next_dev, (const int*)start_dev, n_vocab, n_pos, rs);
  });
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_embed_scaled(void* x_dev, void* h_dev, const void* ids_dev, int n_ids, const void* table_dev, int n_vocab, float scale,
                     const void* w_next_dev, int dtype, int width, int ld, int groups, float eps, void* stream) {
  LCU_REQUIRE(x_dev && ids_dev && table_dev && (h_dev || !w_next_dev), "lcu_embed_scaled: null pointer");
  const row_shape rs{width, ld, groups, eps};
  const int rc = check_rows("lcu_embed_scaled", dtype, n_ids, rs);
  if (rc) return rc;
  LCU_REQUIRE(n_vocab > 0, "lcu_embed_scaled: bad table size %d", n_vocab);
  if (n_ids == 0) return LCU_OK;
  hipStream_t st = as_stream(stream);
  with_row_kind(dtype, ld, n_ids == 1, [&](auto* kind, auto nv, auto th) {
    using T = std::remove_pointer_t<decltype(kind)>;
    embed_pos_norm_kernel<T, decltype(nv)::value, decltype(th)::value><<<n_ids, decltype(th)::value, row_lds_bytes(rs), st>>>(
        (float*)x_dev, (T*)h_dev, (const int*)ids_dev, (const T*)table_dev, scale, nullptr, nullptr, (const float*)w_next_dev, nullptr,
        n_vocab, 0, rs);
  });
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_residual_norm(void* x_dev, void* h_dev, const void* out_f32_dev, const void* inverse_dev, int top,
                      const void* shared_f32_dev, const void* shared_gate_dev, const void* w_after_dev,
                      const void* w_next_dev, int dtype, int rows, int width, int ld, int groups, float eps, void* stream) {
  LCU_REQUIRE(x_dev && out_f32_dev && w_after_dev && (h_dev || !w_next_dev) && (!shared_f32_dev || shared_gate_dev),
              "lcu_residual_norm: null pointer");
  const row_shape rs{width, ld, groups, eps};
  const int rc = check_rows("lcu_residual_norm", dtype, rows, rs);
  if (rc) return rc;
  if (rows == 0) return LCU_OK;
  LCU_REQUIRE(top >= 1, "lcu_residual_norm: %d rows per token", top);
  const sublayer_rows src{(const float*)out_f32_dev, (const int*)inverse_dev, top, (const float*)shared_f32_dev,
                          (const float*)shared_gate_dev};
  hipStream_t st = as_stream(stream);
  with_row_kind(dtype, ld, rows == 1, [&](auto* kind, auto nv, auto th) {
    using T = std::remove_pointer_t<decltype(kind)>;
    residual_norm_kernel<T, decltype(nv)::value, decltype(th)::value><<<rows, decltype(th)::value, row_lds_bytes(rs), st>>>(
        (float*)x_dev, (T*)h_dev, src, (const float*)w_after_dev, (const float*)w_next_dev, rs);
  });
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_decode_residual_router(void* x_dev, void* h_dev, const void* out_f32_dev, int top, const void* shared_f32_dev,
                               const void* shared_gate_dev, const void* w_after_dev, const void* w_next_dev, int width, int ld,
                               int groups, float eps, const void* router_w_dev, int n_experts, int choose, void* expert_dev,
                               void* weight_dev, void* router_gate_dev, void* stream) {
  LCU_REQUIRE(x_dev && out_f32_dev && w_after_dev && (h_dev || !w_next_dev) && (!shared_f32_dev || shared_gate_dev) &&
                  (!router_w_dev || (w_next_dev && expert_dev && weight_dev)),
              "lcu_decode_residual_router: null pointer");
  const row_shape rs{width, ld, groups, eps};
  const int rc = check_rows("lcu_decode_residual_router", LCU_BF16, 1, rs);
  if (rc) return rc;
  router_step rt{};
  if (router_w_dev) {
    rt = router_step{(const bf16_t*)router_w_dev, n_experts + (router_gate_dev ? 1 : 0), n_experts, choose, (int*)expert_dev,
                     (float*)weight_dev, (float*)router_gate_dev};
    LCU_REQUIRE(n_experts > 0 && rt.rows <= ROUTER_MAX_ROWS && choose > 0 && choose <= n_experts,
                "lcu_decode_residual_router: experts %d (at most %d), top %d", n_experts, ROUTER_MAX_ROWS - 1, choose);
  }
  LCU_REQUIRE(top >= 1, "lcu_decode_residual_router: %d rows", top);
  const sublayer_rows src{(const float*)out_f32_dev, nullptr, top, (const float*)shared_f32_dev, (const float*)shared_gate_dev};
  size_t lds = row_lds_bytes(rs);
  if (router_w_dev && lds < (size_t)ld * 2) lds = (size_t)ld * 2;
  with_step_pieces(ld, [&](auto nv) {
    residual_step_kernel<decltype(nv)::value><<<1, STEP_THREADS, lds, as_stream(stream)>>>(
        (float*)x_dev, (bf16_t*)h_dev, src, (const float*)w_after_dev, (const float*)w_next_dev, rs, rt);
  });
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_group_norm(void* h_dev, const void* x_f32_dev, const void* row_index_dev, const void* w_dev, int dtype, int rows,
                   int width, int ld, int groups, float eps, void* stream) {
  LCU_REQUIRE(h_dev && x_f32_dev && w_dev, "lcu_group_norm: null pointer");
  const row_shape rs{width, ld, groups, eps};
  const int rc = check_rows("lcu_group_norm", dtype, rows, rs);
  if (rc) return rc;
  if (rows == 0) return LCU_OK;
  hipStream_t st = as_stream(stream);
  with_row_kind(dtype, ld, rows == 1, [&](auto* kind, auto nv, auto th) {
    using T = std::remove_pointer_t<decltype(kind)>;
    group_norm_kernel<T, decltype(nv)::value, decltype(th)::value><<<rows, decltype(th)::value, row_lds_bytes(rs), st>>>(
        (T*)h_dev, (const float*)x_f32_dev, (const int*)row_index_dev, (const float*)w_dev, rs);
  });
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_argmax_f32(void* out_index_dev, const void* values_dev, int n, void* stream) {
  LCU_REQUIRE(out_index_dev && values_dev && n > 0, "lcu_argmax_f32: bad arguments");
  argmax_f32_kernel<<<1, 1024, 0, as_stream(stream)>>>((int*)out_index_dev, (const float*)values_dev, n);
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_softmax_f32(void* probs_f16_dev, const void* logits_dev, int n, float temp, void* stream) {
  LCU_REQUIRE(probs_f16_dev && logits_dev && n > 0 && temp > 0.0f, "lcu_softmax_f32: bad arguments");
  softmax_f32_kernel<<<1, 1024, 0, as_stream(stream)>>>((half_t*)probs_f16_dev, (const float*)logits_dev, n, temp);
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_fill_normal_matrix(void* out_dev, size_t rows, int cols, int ld, int dtype, uint64_t seed, uint64_t stream_id, float mean,
                           float std, void* stream) {
  LCU_REQUIRE(out_dev && cols > 0 && ld >= cols && (dtype == LCU_BF16 || dtype == LCU_F32), "lcu_fill_normal_matrix: bad arguments");
  if (rows == 0) return LCU_OK;
  const size_t blocks = (rows * (size_t)cols + 255) / 256;
  LCU_REQUIRE(blocks < ((size_t)1 << 31), "lcu_fill_normal_matrix: too many elements");
  if (dtype == LCU_F32) {
    fill_normal_kernel<float><<<(unsigned)blocks, 256, 0, as_stream(stream)>>>((float*)out_dev, rows, cols, ld, seed, stream_id, mean, std);
  } else {
    fill_normal_kernel<bf16_t><<<(unsigned)blocks, 256, 0, as_stream(stream)>>>((bf16_t*)out_dev, rows, cols, ld, seed, stream_id, mean, std);
  }
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

}  // extern "C"
