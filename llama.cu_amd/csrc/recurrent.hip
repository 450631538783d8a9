// Gated linear recurrence (Griffin's recurrent block): causal per-channel convolution, block-diagonal
// gates, and the state S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t with log a_t = decay r_t.
//
// Channels are laid out block by block, each block padded with zeros to a multiple of 32 (a padded
// channel's state stays 0); ld is the row stride, a multiple of 64.  Gates, decays and state are fp32.
//
// Several tokens: the recurrence is linear in S, so tokens are cut into chunks of 64.  The gate
// kernel leaves a_t and the drive b_t of every token and, per chunk, the chunk's map S -> A S + B; one
// thread per channel runs over the chunks' maps (carry), and then every chunk runs through its own
// tokens from its incoming state (apply).
#include <type_traits>

#include "linear.hpp"
#include "rownorm.hpp"

using namespace lcu;

namespace {

constexpr int CHUNK = 64;   // tokens per chunk and per gate tile
constexpr int GATE_N = 32;  // channels per gate tile

// u[t][c] = bias[c] + sum_k w[k][c] z[t - (taps - 1) + k], then silu where asked; inputs before this call come from
// state [taps - 1][ld], oldest first.  A thread takes four channels of CONV_T tokens.
constexpr int CONV_T = 8;
template <class T, bool SILU>
__global__ __launch_bounds__(256) void conv_causal_kernel(T* __restrict__ u, const T* __restrict__ z, int ldz,
                                                          const float* __restrict__ w, const float* __restrict__ bias,
                                                          const T* __restrict__ state, int taps, int n, int channels, int ld) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 4, t0 = blockIdx.y * CONV_T;
  if (c >= channels) return;
  float4_t acc[CONV_T];
  const float4_t b = bias ? load4(bias + c) : (float4_t)(0.0f);
#pragma unroll
  for (int e = 0; e < CONV_T; ++e) acc[e] = b;
  for (int k = 0; k < taps; ++k) {
    const float4_t wk = load4(w + (size_t)k * ld + c);
#pragma unroll
    for (int e = 0; e < CONV_T; ++e) {
      const int s = min(t0 + e, n - 1) - (taps - 1) + k;
      const float4_t v = load4(s >= 0 ? z + (size_t)s * ldz + c : state + (size_t)(s + taps - 1) * ld + c);
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[e][i] = fmaf(wk[i], v[i], acc[e][i]);
    }
  }
#pragma unroll
  for (int e = 0; e < CONV_T; ++e) {
    if constexpr (SILU) {
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[e][i] *= sigmoid_f32(acc[e][i]);
    }
    if (t0 + e < n) store4(u + (size_t)(t0 + e) * ld + c, acc[e]);
  }
}

// the last taps - 1 inputs become the state; ascending order, so a short call shifts in place
template <class T>
__global__ __launch_bounds__(256) void conv_state_kernel(T* __restrict__ state, const T* __restrict__ z, int ldz, int n, int taps,
                                                         int channels, int ld) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= channels) return;
  for (int k = 0; k + 1 < taps; ++k) {
    const int s = k + n - (taps - 1);
    state[(size_t)k * ld + c] = s >= 0 ? z[(size_t)s * ldz + c] : state[(size_t)(k + n) * ld + c];
  }
}

// sqrt(1 - a^2) for a = exp(log_a), log_a <= 0, without cancellation: 1 - e^x by its series near 0
__device__ __forceinline__ float drive_factor(float log_a, float a) {
  const float x = 2.0f * log_a;
  const float series = -x * (1.0f + x * (1.0f / 2) * (1.0f + x * (1.0f / 3) * (1.0f + x * (1.0f / 4) * (1.0f + x * (1.0f / 5) * (1.0f + x * (1.0f / 6))))));
  return __builtin_amdgcn_sqrtf(x > -0.25f ? series : 1.0f - a * a);
}
// fp32 gates of the bfloat16 element type: the machine's exponential, reciprocal and square root (1 ulp each)
__device__ __forceinline__ float sigmoid_fast(float z) { return __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }

struct gate_args {
  const void* wr;       // [blocks][bw][bw], rows and blocks padded
  const void* wi;
  const float* br;
  const float* bi;
  const float* decay;   // log a = decay * r
  float* a;
  float* b;
  float* chunk_a;
  float* chunk_b;
  int n, bw, ld;
};

// The map S -> A S + B of consecutive tokens
struct state_map {
  float A{1.0f}, B{0.0f};
  __device__ __forceinline__ void then(float a, float b) {
    B = fmaf(a, B, b);
    A = a * A;
  }
};

// fp32.  One workgroup: 64 tokens x 32 channels of both gates.  Wavefront w multiplies 32 tokens (w & 1) by the
// channels of gate w >> 1; both gates of a channel then meet in LDS, and every thread turns eight
// consecutive tokens of one channel into a, b and their composite map.
__global__ __launch_bounds__(256) void gates_f32_kernel(const float* __restrict__ u, gate_args p) {
  __shared__ float gate[2][CHUNK][GATE_N + 1];
  __shared__ float seg[2][8][GATE_N];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int t0 = blockIdx.y * CHUNK, c0 = blockIdx.x * GATE_N;  // c0: first channel of the tile, inside one block
  const int blk = c0 / p.bw, j0 = c0 - blk * p.bw;
  const int which = wave >> 1, rows0 = (wave & 1) * 32;
  const float* W = (const float*)(which ? p.wi : p.wr) + ((size_t)blk * p.bw + j0) * p.bw;
  const float* ub = u + (size_t)blk * p.bw;
  {
    // lane (channel lane & 31, half lane >> 5) sums 16 tokens of its wavefront's 32
    float acc[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[i] = 0.0f;
    for (int k = 0; k < p.bw; ++k) {
      const float w = W[(size_t)(lane & 31) * p.bw + k];
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        acc[i] = fmaf(ub[(size_t)min(t0 + rows0 + (lane >> 5) * 16 + i, p.n - 1) * p.ld + k], w, acc[i]);
      }
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) gate[which][rows0 + (lane >> 5) * 16 + i][lane & 31] = acc[i];
  }
  __syncthreads();
  const int ch = tid & 31, s8 = tid >> 5, c = c0 + ch;
  const float br = p.br[c], bi = p.bi[c], decay = p.decay[c];
  state_map map;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const int lt = s8 * 8 + e, t = t0 + lt;
    if (t < p.n) {
      const float log_a = decay * sigmoid_f32(gate[0][lt][ch] + br);
      const float a = expf(log_a);
      const float b = sqrtf(-expm1f(2.0f * log_a)) * sigmoid_f32(gate[1][lt][ch] + bi) * u[(size_t)t * p.ld + c];
      p.a[(size_t)t * p.ld + c] = a;
      p.b[(size_t)t * p.ld + c] = b;
      map.then(a, b);
    }
  }
  seg[0][s8][ch] = map.A;
  seg[1][s8][ch] = map.B;
  __syncthreads();
  if (tid < GATE_N) {
    state_map whole;
#pragma unroll
    for (int s = 0; s < 8; ++s) whole.then(seg[0][s][tid], seg[1][s][tid]);
    p.chunk_a[(size_t)blockIdx.y * p.ld + c0 + tid] = whole.A;
    p.chunk_b[(size_t)blockIdx.y * p.ld + c0 + tid] = whole.B;
  }
}

// bfloat16.  A wavefront takes a chunk of 64 tokens x 32 channels of both gates in two halves of 32 tokens, so
// that a lane holds r and i of the same tokens of one channel: element v of half m belongs to token
// t0 + 32 m + (v >> 2) * 8 + 4 (lane >> 5) + (v & 3).
__device__ __forceinline__ void finish_gates(const gate_args& p, const bf16_t* __restrict__ u, const float16_t& r, const float16_t& g,
                                             int t0, int c, state_map& whole) {
  const int half = (threadIdx.x & 63) >> 5;
  const float br = p.br[c], bi = p.bi[c], decay = p.decay[c];
  float uv[16];
#pragma unroll
  for (int v = 0; v < 16; ++v) {
    uv[v] = (float)u[(size_t)min(t0 + (v >> 2) * 8 + half * 4 + (v & 3), p.n - 1) * p.ld + c];
  }
#pragma unroll
  for (int o = 0; o < 4; ++o) {
    state_map map;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int v = o * 4 + e, t = t0 + o * 8 + half * 4 + e;
      const float log_a = decay * sigmoid_fast(r[v] + br);
      const float a = __expf(log_a);
      const float b = drive_factor(log_a, a) * sigmoid_fast(g[v] + bi) * uv[v];
      if (t < p.n) {
        p.a[(size_t)t * p.ld + c] = a;
        p.b[(size_t)t * p.ld + c] = b;
        map.then(a, b);
      }
    }
    // the lane 32 further holds the neighbouring four tokens of the eight
    const float oA = __shfl_xor(map.A, 32, WAVE), oB = __shfl_xor(map.B, 32, WAVE);
    whole.then(half ? oA : map.A, half ? oB : map.B);
    whole.then(half ? map.A : oA, half ? map.B : oB);
  }
}

__device__ __forceinline__ void store_chunk_map(const gate_args& p, const state_map& whole, int c) {
  if ((threadIdx.x & 32) == 0) {
    p.chunk_a[(size_t)blockIdx.y * p.ld + c] = whole.A;
    p.chunk_b[(size_t)blockIdx.y * p.ld + c] = whole.B;
  }
}

// any block width: operands straight from memory
__global__ __launch_bounds__(256, 4) void gates_bf16_kernel(const bf16_t* __restrict__ u, gate_args p, int channels) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int t0 = blockIdx.y * CHUNK, c0 = (blockIdx.x * 4 + wave) * GATE_N;
  if (c0 >= channels) return;
  const int blk = c0 / p.bw, j0 = c0 - blk * p.bw, col = lane & 31, half = lane >> 5, c = c0 + col;
  const bf16_t* ua = u + (size_t)blk * p.bw + half * 8;
  const size_t w_at = ((size_t)blk * p.bw + j0 + col) * p.bw + half * 8;
  const bf16_t* wr = (const bf16_t*)p.wr + w_at;
  const bf16_t* wi = (const bf16_t*)p.wi + w_at;
  const auto piece = [](const bf16_t* q, int k) { return *reinterpret_cast<const bf16x8_t*>(q + k); };
  state_map whole;
  for (int m = 0; m < 2; ++m) {
    const bf16_t* um = ua + (size_t)min(t0 + 32 * m + col, p.n - 1) * p.ld;
    float16_t r = (float16_t)(0.0f), g = (float16_t)(0.0f);
#pragma unroll 2
    for (int k = 0; k < p.bw; k += 32) {  // block widths are multiples of 32
      const bf16x8_t a0 = piece(um, k), b0 = piece(wr, k), c0v = piece(wi, k);
      const bf16x8_t a1 = piece(um, k + 16), b1 = piece(wr, k + 16), c1v = piece(wi, k + 16);
      r = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a0, b0, r, 0, 0, 0);
      g = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a0, c0v, g, 0, 0, 0);
      r = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a1, b1, r, 0, 0, 0);
      g = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a1, c1v, g, 0, 0, 0);
    }
    finish_gates(p, u, r, g, t0 + 32 * m, c, whole);
  }
  store_chunk_map(p, whole, c);
}

// block widths that are multiples of 128: four wavefronts share a chunk's rows of u and 128 channels' gate rows
// in LDS, 64 columns of K at a time, the next ones in registers meanwhile
constexpr int TILE_C = 128, TILE_K = 64, LDG = TILE_K + 8;
__global__ __launch_bounds__(256, 2) void gates_tile_kernel(const bf16_t* __restrict__ u, gate_args p) {
  __shared__ __attribute__((aligned(16))) bf16_t us[CHUNK * LDG];
  __shared__ __attribute__((aligned(16))) bf16_t ws[2][TILE_C * LDG];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int t0 = blockIdx.y * CHUNK, c0 = blockIdx.x * TILE_C, blk = c0 / p.bw;
  const int row = tid >> 3, col8 = (tid & 7) * 8;  // eight threads per row of 64 columns, 32 rows per pass
  const bf16_t* ug = u + (size_t)blk * p.bw + col8;
  const bf16_t* wg[2] = {(const bf16_t*)p.wr + (size_t)c0 * p.bw + col8, (const bf16_t*)p.wi + (size_t)c0 * p.bw + col8};
  uint4_t ru[2], rw[2][4];
  const auto load = [&](int k) {
#pragma unroll
    for (int i = 0; i < 2; ++i) ru[i] = *reinterpret_cast<const uint4_t*>(ug + (size_t)min(t0 + row + 32 * i, p.n - 1) * p.ld + k);
#pragma unroll
    for (int w = 0; w < 2; ++w) {
#pragma unroll
      for (int i = 0; i < 4; ++i) rw[w][i] = *reinterpret_cast<const uint4_t*>(wg[w] + (size_t)(row + 32 * i) * p.bw + k);
    }
  };
  float16_t r[2], g[2];
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    r[m] = (float16_t)(0.0f);
    g[m] = (float16_t)(0.0f);
  }
  load(0);
  for (int k = 0; k < p.bw; k += TILE_K) {
    __syncthreads();  // the previous tile has been read
#pragma unroll
    for (int i = 0; i < 2; ++i) *reinterpret_cast<uint4_t*>(us + (row + 32 * i) * LDG + col8) = ru[i];
#pragma unroll
    for (int w = 0; w < 2; ++w) {
#pragma unroll
      for (int i = 0; i < 4; ++i) *reinterpret_cast<uint4_t*>(ws[w] + (row + 32 * i) * LDG + col8) = rw[w][i];
    }
    __syncthreads();
    if (k + TILE_K < p.bw) load(k + TILE_K);
    const int frag = (lane & 31) * LDG + (lane >> 5) * 8;
#pragma unroll
    for (int s = 0; s < TILE_K; s += 16) {
      const bf16x8_t a0 = *reinterpret_cast<const bf16x8_t*>(us + frag + s);
      const bf16x8_t a1 = *reinterpret_cast<const bf16x8_t*>(us + 32 * LDG + frag + s);
      const bf16x8_t b0 = *reinterpret_cast<const bf16x8_t*>(ws[0] + wave * 32 * LDG + frag + s);
      const bf16x8_t b1 = *reinterpret_cast<const bf16x8_t*>(ws[1] + wave * 32 * LDG + frag + s);
      r[0] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a0, b0, r[0], 0, 0, 0);
      r[1] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a1, b0, r[1], 0, 0, 0);
      g[0] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a0, b1, g[0], 0, 0, 0);
      g[1] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a1, b1, g[1], 0, 0, 0);
    }
  }
  const int c = c0 + wave * 32 + (lane & 31);
  state_map whole;
  finish_gates(p, u, r[0], g[0], t0, c, whole);
  finish_gates(p, u, r[1], g[1], t0 + 32, c, whole);
  store_chunk_map(p, whole, c);
}

// chunk_a[k] <- the state that enters chunk k; state <- the state after the last chunk
__global__ __launch_bounds__(64) void carry_kernel(float* __restrict__ chunk_a, const float* __restrict__ chunk_b,
                                                   float* __restrict__ state, int chunks, int channels, int ld) {
  const int c = blockIdx.x * 64 + threadIdx.x;
  if (c >= channels) return;
  float S = state[c];
  for (int k0 = 0; k0 < chunks; k0 += 8) {
    float A[8], B[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int k = min(k0 + e, chunks - 1);
      A[e] = chunk_a[(size_t)k * ld + c];
      B[e] = chunk_b[(size_t)k * ld + c];
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      if (k0 + e < chunks) {
        chunk_a[(size_t)(k0 + e) * ld + c] = S;
        S = fmaf(A[e], S, B[e]);
      }
    }
  }
  state[c] = S;
}

// out[t][c] = S_t * y[t][c] over one chunk
template <class T>
__global__ __launch_bounds__(256) void apply_kernel(T* __restrict__ out, const float* __restrict__ a, const float* __restrict__ b,
                                                    const float* __restrict__ enter, const T* __restrict__ y, int ldy, int n,
                                                    int channels, int ld) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= channels) return;
  const int t0 = blockIdx.y * CHUNK, t1 = min(t0 + CHUNK, n);
  float S = enter[(size_t)blockIdx.y * ld + c];
  for (int t = t0; t < t1; t += 8) {
    float av[8], bv[8], yv[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int s = min(t + e, t1 - 1);
      av[e] = a[(size_t)s * ld + c];
      bv[e] = b[(size_t)s * ld + c];
      yv[e] = to_f32(y[(size_t)s * ldy + c]);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      if (t + e < t1) {
        S = fmaf(av[e], S, bv[e]);
        out[(size_t)(t + e) * ld + c] = (T)(S * yv[e]);
      }
    }
  }
}

// One new token: 16 lanes share a channel, whose two gate rows they multiply with the block's u; the first of
// them takes the channel's step.
__global__ __launch_bounds__(256) void recurrent_step_kernel(bf16_t* __restrict__ out, const bf16_t* __restrict__ u,
                                                             const bf16_t* __restrict__ y, float* __restrict__ state, gate_args p,
                                                             int channels) {
  const int sub = threadIdx.x & 15, c = blockIdx.x * 16 + (threadIdx.x >> 4);
  if (c >= channels) return;  // whole groups of 16 lanes
  const bf16_t* wr = (const bf16_t*)p.wr + (size_t)c * p.bw;
  const bf16_t* wi = (const bf16_t*)p.wi + (size_t)c * p.bw;
  const bf16_t* ub = u + c / p.bw * p.bw;
  float r = 0.0f, i = 0.0f;
#pragma unroll 4
  for (int k = sub * 8; k < p.bw; k += 128) {
    const bf16x8_t uv = *reinterpret_cast<const bf16x8_t*>(ub + k);
    const bf16x8_t rv = *reinterpret_cast<const bf16x8_t*>(wr + k), iv = *reinterpret_cast<const bf16x8_t*>(wi + k);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      r = fmaf((float)rv[e], (float)uv[e], r);
      i = fmaf((float)iv[e], (float)uv[e], i);
    }
  }
  r = row16_sum(r);
  i = row16_sum(i);
  if (sub != 0) return;
  r = sigmoid_f32(r + p.br[c]);
  i = sigmoid_f32(i + p.bi[c]);
  const float log_a = p.decay[c] * r;
  const float S = fmaf(expf(log_a), state[c], sqrtf(-expm1f(2.0f * log_a)) * i * (float)u[c]);
  state[c] = S;
  out[c] = (bf16_t)(S * (float)y[c]);
}

int check_channels(const char* who, int dtype, int n, int channels, int ld) {
  LCU_REQUIRE(dtype == LCU_BF16 || dtype == LCU_F32, "%s: element type %d", who, dtype);
  LCU_REQUIRE(n >= 0 && n <= 65535 && channels > 0 && ld >= channels && ld % 32 == 0, "%s: bad shape n %d channels %d ld %d", who, n,
              channels, ld);
  return LCU_OK;
}

}  // namespace

extern "C" {

int lcu_conv_causal(void* u_dev, const void* z_dev, int ldz, const void* w_dev, const void* bias_dev, void* state_dev, int taps,
                    int silu, int dtype, int n, int channels, int ld, void* stream) {
  LCU_REQUIRE(u_dev && z_dev && w_dev && (state_dev || taps == 1), "lcu_conv_causal: null pointer");
  const int rc = check_channels("lcu_conv_causal", dtype, n, channels, ld);
  if (rc) return rc;
  LCU_REQUIRE(taps >= 1 && ldz >= channels && ldz % 4 == 0 && channels % 4 == 0, "lcu_conv_causal: taps %d, input stride %d", taps, ldz);
  if (n == 0) return LCU_OK;
  hipStream_t st = as_stream(stream);
  const dim3 grid((channels / 4 + 255) / 256, (n + CONV_T - 1) / CONV_T), columns((channels + 255) / 256);
  const auto run = [&](auto* kind, auto act) {
    using T = std::remove_pointer_t<decltype(kind)>;
    conv_causal_kernel<T, decltype(act)::value><<<grid, 256, 0, st>>>((T*)u_dev, (const T*)z_dev, ldz, (const float*)w_dev,
                                                                      (const float*)bias_dev, (const T*)state_dev, taps, n, channels, ld);
    if (taps > 1) conv_state_kernel<T><<<columns, 256, 0, st>>>((T*)state_dev, (const T*)z_dev, ldz, n, taps, channels, ld);
  };
  const auto typed = [&](auto* kind) { silu ? run(kind, std::true_type{}) : run(kind, std::false_type{}); };
  if (dtype == LCU_F32) {
    typed((float*)nullptr);
  } else {
    typed((bf16_t*)nullptr);
  }
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_gated_recurrence(void* out_dev, const void* u_dev, const void* y_dev, int ldy, const void* wr_dev, const void* wi_dev,
                         const void* br_dev, const void* bi_dev, const void* decay_dev, void* state_dev, void* scratch_dev,
                         int dtype, int n, int channels, int block_width, int ld, void* stream) {
  LCU_REQUIRE(out_dev && u_dev && y_dev && wr_dev && wi_dev && br_dev && bi_dev && decay_dev && state_dev && scratch_dev,
              "lcu_gated_recurrence: null pointer");
  const int rc = check_channels("lcu_gated_recurrence", dtype, n, channels, ld);
  if (rc) return rc;
  LCU_REQUIRE(block_width > 0 && block_width % GATE_N == 0 && channels % block_width == 0 && ldy >= channels,
              "lcu_gated_recurrence: block width %d (a multiple of %d dividing %d channels), stride of y %d", block_width, GATE_N,
              channels, ldy);
  if (n == 0) return LCU_OK;
  hipStream_t st = as_stream(stream);
  const int chunks = (n + CHUNK - 1) / CHUNK;
  float* a = (float*)scratch_dev;
  float* b = a + (size_t)n * ld;
  float* ca = b + (size_t)n * ld;
  float* cb = ca + (size_t)chunks * ld;
  const gate_args p{wr_dev, wi_dev, (const float*)br_dev, (const float*)bi_dev, (const float*)decay_dev, a, b, ca, cb, n,
                    block_width, ld};
  const dim3 rows((channels + 255) / 256, chunks);
  if (dtype == LCU_F32) {
    gates_f32_kernel<<<dim3(channels / GATE_N, chunks), 256, 0, st>>>((const float*)u_dev, p);
  } else {
    if (block_width % TILE_C == 0) {
      gates_tile_kernel<<<dim3(channels / TILE_C, chunks), 256, 0, st>>>((const bf16_t*)u_dev, p);
    } else {
      gates_bf16_kernel<<<dim3((channels / GATE_N + 3) / 4, chunks), 256, 0, st>>>((const bf16_t*)u_dev, p, channels);
    }
  }
  carry_kernel<<<(channels + 63) / 64, 64, 0, st>>>(ca, cb, (float*)state_dev, chunks, channels, ld);
  if (dtype == LCU_F32) {
    apply_kernel<float><<<rows, 256, 0, st>>>((float*)out_dev, a, b, ca, (const float*)y_dev, ldy, n, channels, ld);
  } else {
    apply_kernel<bf16_t><<<rows, 256, 0, st>>>((bf16_t*)out_dev, a, b, ca, (const bf16_t*)y_dev, ldy, n, channels, ld);
  }
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

size_t lcu_gated_recurrence_scratch(int n, int ld) {
  return ((size_t)2 * n + (size_t)2 * ((n + CHUNK - 1) / CHUNK)) * ld * sizeof(float);
}

int lcu_decode_recurrent_step(void* out_dev, const void* u_dev, const void* y_dev, const void* wr_dev, const void* wi_dev,
                              const void* br_dev, const void* bi_dev, const void* decay_dev, void* state_dev, int channels,
                              int block_width, void* stream) {
  LCU_REQUIRE(out_dev && u_dev && y_dev && wr_dev && wi_dev && br_dev && bi_dev && decay_dev && state_dev,
              "lcu_decode_recurrent_step: null pointer");
  LCU_REQUIRE(channels > 0 && block_width > 0 && block_width % 32 == 0 && channels % block_width == 0,
              "lcu_decode_recurrent_step: block width %d of %d channels", block_width, channels);
  gate_args p{};
  p.wr = wr_dev;
  p.wi = wi_dev;
  p.br = (const float*)br_dev;
  p.bi = (const float*)bi_dev;
  p.decay = (const float*)decay_dev;
  p.bw = block_width;
  recurrent_step_kernel<<<channels / 16, 256, 0, as_stream(stream)>>>((bf16_t*)out_dev, (const bf16_t*)u_dev, (const bf16_t*)y_dev,
                                                                      (float*)state_dev, p, channels);
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

}  // extern "C"
