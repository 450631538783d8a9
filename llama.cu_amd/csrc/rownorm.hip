// Row kernels of the layered decoders, whose residual stream is fp32: embedding with learned
// positions, grouped RMS norm, and the step between two sublayers (norm of the sublayer's output,
// residual sum, norm of the next sublayer's input) in one launch.  The counterpart for the fp16
// models is rmsnorm_kernel in elementwise.hip.
#include <type_traits>

#include "linear.hpp"
#include "rownorm.hpp"

using namespace lcu;

namespace {

// x[row] = norm(table[token] + pos_table[start + row]) under w0; h[row] = norm(x[row]) under w1 when given
template <class T, int NV>
__global__ __launch_bounds__(ROW_THREADS) void embed_pos_norm_kernel(float* __restrict__ x, T* __restrict__ h,
                                                                     const int* __restrict__ ids, const T* __restrict__ table,
                                                                     const T* __restrict__ pos_table, const float* __restrict__ w0,
                                                                     const float* __restrict__ w1, const int* __restrict__ start,
                                                                     int n_vocab, int n_pos, row_shape rs) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int r = blockIdx.x;
  const int id = min(max(ids[r], 0), n_vocab - 1), p = min(max(*start + r, 0), n_pos - 1);
  row_t<NV> row, at, w;
  load_row(row, table + (size_t)id * rs.ld, rs);
  load_row(at, pos_table + (size_t)p * rs.ld, rs);
  load_row(w, w0, rs);
#pragma unroll
  for (int j = 0; j < NV; ++j) row.v[j] += at.v[j];
  scale_row(row, rs, lds, w);
  store_row(x + (size_t)r * rs.ld, row, rs);
  if (w1) {
    load_row(w, w1, rs);
    scale_row(row, rs, lds, w);
    store_row(h + (size_t)r * rs.ld, row, rs);
  }
}

// m[row] = out[row], or the sum of a token's expert rows (inverse[row * top + k] is where the k-th of them
// lies) plus its shared expert's row times shared_gate[row]; x += norm(m) under w_after; h = norm(x) under w_next.
template <class T, int NV>
__global__ __launch_bounds__(ROW_THREADS) void residual_norm_kernel(float* __restrict__ x, T* __restrict__ h,
                                                                    sublayer_rows src, const float* __restrict__ w_after,
                                                                    const float* __restrict__ w_next, row_shape rs) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int r = blockIdx.x;
  row_t<NV> m, t, old;
  if (src.inverse) {
    load_row(m, src.out + (size_t)src.inverse[(size_t)r * src.top] * rs.ld, rs);
    for (int k = 1; k < src.top; ++k) {
      load_row(t, src.out + (size_t)src.inverse[(size_t)r * src.top + k] * rs.ld, rs);
#pragma unroll
      for (int j = 0; j < NV; ++j) m.v[j] += t.v[j];
    }
    if (src.shared) {
      const float f = src.shared_gate[r];
      load_row(t, src.shared + (size_t)r * rs.ld, rs);
#pragma unroll
      for (int j = 0; j < NV; ++j) m.v[j] += f * t.v[j];
    }
  } else {
    load_row(m, src.out + (size_t)r * rs.ld, rs);
  }
  float* xr = x + (size_t)r * rs.ld;
  load_row(old, xr, rs);
  load_row(t, w_after, rs);
  scale_row(m, rs, lds, t);
#pragma unroll
  for (int j = 0; j < NV; ++j) m.v[j] += old.v[j];
  store_row(xr, m, rs);
  if (w_next) {
    load_row(t, w_next, rs);
    scale_row(m, rs, lds, t);
    store_row(h + (size_t)r * rs.ld, m, rs);
  }
}

// h[i] = norm(x[rows[i]]) under w (rows NULL: row i)
template <class T, int NV>
__global__ __launch_bounds__(ROW_THREADS) void group_norm_kernel(T* __restrict__ h, const float* __restrict__ x,
                                                                 const int* __restrict__ rows, const float* __restrict__ w,
                                                                 row_shape rs) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int r = rows ? rows[blockIdx.x] : blockIdx.x;
  row_t<NV> row, wr;
  load_row(row, x + (size_t)r * rs.ld, rs);
  load_row(wr, w, rs);
  scale_row(row, rs, lds, wr);
  store_row(h + (size_t)blockIdx.x * rs.ld, row, rs);
}

// calls f with a null pointer of the element type and the pieces of a row
template <class F>
void with_row_kind(int dtype, int ld, F&& f) {
  with_row_pieces(ld, [&](auto nv) {
    if (dtype == LCU_F32) {
      f((float*)nullptr, nv);
    } else {
      f((bf16_t*)nullptr, nv);
    }
  });
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
  with_row_kind(dtype, ld, [&](auto* kind, auto nv) {
    using T = std::remove_pointer_t<decltype(kind)>;
    embed_pos_norm_kernel<T, decltype(nv)::value><<<n_ids, ROW_THREADS, row_lds_bytes(rs), st>>>(
        (float*)x_dev, (T*)h_dev, (const int*)ids_dev, (const T*)table_dev, (const T*)pos_table_dev, (const float*)w_embed_dev,
        (const float*)w_next_dev, (const int*)start_dev, n_vocab, n_pos, rs);
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
  const sublayer_rows src{(const float*)out_f32_dev, (const int*)inverse_dev, top, (const float*)shared_f32_dev,
                          (const float*)shared_gate_dev};
  hipStream_t st = as_stream(stream);
  with_row_kind(dtype, ld, [&](auto* kind, auto nv) {
    using T = std::remove_pointer_t<decltype(kind)>;
    residual_norm_kernel<T, decltype(nv)::value><<<rows, ROW_THREADS, row_lds_bytes(rs), st>>>(
        (float*)x_dev, (T*)h_dev, src, (const float*)w_after_dev, (const float*)w_next_dev, rs);
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
  with_row_kind(dtype, ld, [&](auto* kind, auto nv) {
    using T = std::remove_pointer_t<decltype(kind)>;
    group_norm_kernel<T, decltype(nv)::value><<<rows, ROW_THREADS, row_lds_bytes(rs), st>>>(
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
