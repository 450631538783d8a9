// Gated delta rule (Yang, Kautz, Hatamizadeh: "Gated Delta Networks: Improving Mamba2 with Delta Rule").  Per head, with
// state S [D][E] and unit vectors q, k:
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// beta = sigmoid(b), log g = -exp(A_log) softplus(a + dt_bias).
//
// Channels of a token: q [kv_heads * D] | k [kv_heads * D] | v [heads * E], after their convolution; D is the head size
// padded to 32, 64, 128 or 256 and E the value size padded to a multiple of 32, padding zero.  Everything here is fp32
// but these channels and the result, which have the element type; products run on the fp32 matrix cores, and on the
// bfloat16 ones where both operands are channels as stored (their products are exact in fp32).
//
// Several tokens: chunks of 64.  With G_t the sum of log g up to t inside the chunk and S the state that enters it,
//   u_t = beta_t (v_t - e^G_t S^T k_t - sum_(s<t) e^(G_t - G_s) (k_s . k_t) u_s)
//   o_t = e^G_t S^T q_t + sum_(s<=t) e^(G_t - G_s) (k_s . q_t) u_s
//   S'  = e^G_64 S + sum_s e^(G_64 - G_s) k_s u_s^T
// The first is linear in S: u = X - Y S, where X and Y solve one triangular system with right sides beta v and beta e^G k.
// The chunk kernel solves it for every chunk at once; the scan kernel then runs over the chunks, sixteen columns of S
// per workgroup.  No exponent is ever positive.
#include <type_traits>

#include "linear.hpp"
#include "rownorm.hpp"

using namespace lcu;

namespace {

constexpr int CHUNK = 64;
constexpr float UNIT_EPS = 1e-6f;

struct delta_args {
  int heads, kv_heads, E, dim, vdim;  // dim, vdim: sizes without padding
  int n, ld;                          // tokens; row stride of the channels
  const float* ba;                    // fp32 rows [b heads | a heads]
  int ld_ba;
  const float* a_log;
  const float* dt_bias;
  const float* norm;                  // [vdim], plain
  float eps;
  // per (head, chunk): solutions X [64][E] and Y [64][D], decayed q.k [64][64], row factors [64][2] (of o, of k), e^G_64
  float* X;
  float* Y;
  float* P;
  float* rows;
  float* total;
};

__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float log_decay(const delta_args& p, float a, int h) {
  return -expf(p.a_log[h]) * softplus_f32(a + p.dt_bias[h]);
}

__device__ __forceinline__ float4_t mfma_f32(float a, float b, float4_t c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// 16 x 16 tile of x . y^T over D columns; x and y point at this lane's row
template <int D>
__device__ __forceinline__ float4_t row_products(const bf16_t* x, const bf16_t* y, float4_t acc) {
  const int quad = (threadIdx.x & 63) >> 4;
#pragma unroll
  for (int c = 0; c < D; c += 32) {
    const bf16x8_t a = *reinterpret_cast<const bf16x8_t*>(x + c + quad * 8), b = *reinterpret_cast<const bf16x8_t*>(y + c + quad * 8);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc, 0, 0, 0);
  }
  return acc;
}
template <int D>
__device__ __forceinline__ float4_t row_products(const float* x, const float* y, float4_t acc) {
  const int quad = (threadIdx.x & 63) >> 4;
#pragma unroll 4
  for (int c = 0; c < D; c += 16) {
    const float4_t a = load4(x + c + quad * 4), b = load4(y + c + quad * 4);
#pragma unroll
    for (int j = 0; j < 4; ++j) acc = mfma_f32(a[j], b[j], acc);
  }
  return acc;
}

// One workgroup: one chunk of one head.
template <class T, int D>
__global__ __launch_bounds__(256) void delta_chunk_kernel(const T* __restrict__ qkv, delta_args p) {
  constexpr int LDA = CHUNK + 4;
  __shared__ __attribute__((aligned(16))) float A[CHUNK * LDA];  // beta_t e^(G_t - G_s) k_t . k_s, s < t
  __shared__ float Gs[CHUNK], beta[CHUNK], inv_q[CHUNK], inv_k[CHUNK];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, quad = lane >> 4;
  const int h = blockIdx.x, chunk = blockIdx.y, g = h / (p.heads / p.kv_heads), t0 = chunk * CHUNK;
  const size_t at = (size_t)h * gridDim.y + chunk;
  const T* Q = qkv + (size_t)g * D;
  const T* K = qkv + (size_t)(p.kv_heads + g) * D;
  const T* V = qkv + (size_t)2 * p.kv_heads * D + (size_t)h * p.E;
  const auto row = [&](int t) { return (size_t)min(t0 + t, p.n - 1) * p.ld; };
  if (wave == 0) {
    const bool real = t0 + lane < p.n;
    const float* ba = p.ba + (size_t)min(t0 + lane, p.n - 1) * p.ld_ba;
    float G = real ? log_decay(p, ba[p.heads + h], h) : 0.0f;
    beta[lane] = real ? sigmoid_f32(ba[h]) : 0.0f;
#pragma unroll
    for (int off = 1; off < WAVE; off <<= 1) {
      const float before = __shfl_up(G, off, WAVE);
      if (lane >= off) G += before;
    }
    Gs[lane] = G;
  }
  {
    // four lanes per token
    const size_t r = row(tid >> 2);
    float q2 = 0.0f, k2 = 0.0f;
#pragma unroll 4
    for (int c = (tid & 3) * 4; c < D; c += 16) {
      const float4_t q = load4(Q + r + c), k = load4(K + r + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        q2 = fmaf(q[e], q[e], q2);
        k2 = fmaf(k[e], k[e], k2);
      }
    }
    q2 += dpp_f32<0xB1>(q2);
    q2 += dpp_f32<0x4E>(q2);
    k2 += dpp_f32<0xB1>(k2);
    k2 += dpp_f32<0x4E>(k2);
    if ((tid & 3) == 0) {
      inv_q[tid >> 2] = 1.0f / sqrtf(q2 + UNIT_EPS) / sqrtf((float)p.dim);
      inv_k[tid >> 2] = 1.0f / sqrtf(k2 + UNIT_EPS);
    }
  }
  __syncthreads();
  // wavefront w: rows 16 w .. 16 w + 15 of both products
  float* P = p.P + at * CHUNK * CHUNK;
#pragma unroll 1
  for (int ct = 0; ct < 4; ++ct) {
    float4_t kk = (float4_t)(0.0f), qk = (float4_t)(0.0f);
    if (ct <= wave) {
      const T* y = K + row(ct * 16 + col);
      kk = row_products<D>(K + row(wave * 16 + col), y, kk);
      qk = row_products<D>(Q + row(wave * 16 + col), y, qk);
    }
    const int s = ct * 16 + col;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = wave * 16 + quad * 4 + e;
      const float f = s <= t ? expf(Gs[t] - Gs[s]) * inv_k[s] : 0.0f;
      A[t * LDA + s] = s < t ? beta[t] * inv_k[t] * f * kk[e] : 0.0f;
      P[t * CHUNK + s] = inv_q[t] * f * qk[e];
    }
  }
  if (tid < CHUNK) {
    const float G = Gs[tid], end = Gs[CHUNK - 1];
    p.rows[(at * CHUNK + tid) * 2] = expf(G) * inv_q[tid];
    p.rows[(at * CHUNK + tid) * 2 + 1] = expf(end - G) * inv_k[tid];
    if (tid == 0) p.total[at] = expf(end);
  }
  __syncthreads();
  // forward substitution, one column of the right sides per thread
  for (int c = tid; c < p.E + D; c += 256) {
    const bool of_v = c < p.E;
    const T* src = of_v ? V + c : K + (c - p.E);
    float x[CHUNK];
#pragma unroll
    for (int t = 0; t < CHUNK; ++t) x[t] = to_f32(src[row(t)]);
#pragma unroll
    for (int t = 0; t < CHUNK; ++t) {
      float acc = x[t] * (of_v ? beta[t] : beta[t] * expf(Gs[t]) * inv_k[t]);
#pragma unroll
      for (int s4 = 0; s4 < t; s4 += 4) {
        const float4_t a = load4(A + t * LDA + s4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          if (s4 + e < t) acc = fmaf(-a[e], x[s4 + e], acc);
        }
      }
      x[t] = acc;
    }
    float* dst = of_v ? p.X + at * CHUNK * p.E + c : p.Y + at * CHUNK * D + (c - p.E);
    const int ldd = of_v ? p.E : D;
#pragma unroll
    for (int t = 0; t < CHUNK; ++t) dst[t * ldd] = x[t];
  }
}

// One workgroup: sixteen columns of one head's state through all chunks.  o: fp32 [n][heads * E].
template <class T, int D>
__global__ __launch_bounds__(256) void delta_scan_kernel(float* __restrict__ o, float* __restrict__ state, const T* __restrict__ qkv,
                                                         int chunks, delta_args p) {
  constexpr int LD = 20, TILES = (D / 16 + 3) / 4;  // state tiles of a wavefront
  __shared__ float S[D * LD];
  __shared__ float U[CHUNK * LD], Uk[CHUNK * LD];   // u, and u times the row's factor of k
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, quad = lane >> 4;
  const int h = blockIdx.x, c0 = blockIdx.y * 16, g = h / (p.heads / p.kv_heads);
  float* St = state + (size_t)h * D * p.E + c0;
  for (int i = tid; i < D * 16; i += 256) S[(i >> 4) * LD + (i & 15)] = St[(size_t)(i >> 4) * p.E + (i & 15)];
  const T* Q = qkv + (size_t)g * D;
  const T* K = qkv + (size_t)(p.kv_heads + g) * D;
  for (int chunk = 0; chunk < chunks; ++chunk) {
    const size_t at = (size_t)h * chunks + chunk;
    const int t0 = chunk * CHUNK, r0 = wave * 16 + quad * 4;
    const float* Y = p.Y + (at * CHUNK + wave * 16 + col) * D;
    const float* X = p.X + (at * CHUNK + r0) * p.E + c0 + col;
    const float* rows = p.rows + at * CHUNK * 2;
    __syncthreads();  // S is whole
    float4_t ys = (float4_t)(0.0f), qs = (float4_t)(0.0f);
    const T* q = Q + (size_t)min(t0 + wave * 16 + col, p.n - 1) * p.ld;
#pragma unroll 4
    for (int d = 0; d < D; d += 16) {
      const float4_t a = load4(Y + d + quad * 4), b = load4(q + d + quad * 4);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float s = S[(d + quad * 4 + j) * LD + col];
        ys = mfma_f32(a[j], s, ys);
        qs = mfma_f32(b[j], s, qs);
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float u = X[(size_t)e * p.E] - ys[e];
      U[(r0 + e) * LD + col] = u;
      Uk[(r0 + e) * LD + col] = u * rows[(r0 + e) * 2 + 1];
      qs[e] *= rows[(r0 + e) * 2];
    }
    __syncthreads();  // everyone has read S and written its part of u
    const float* P = p.P + (at * CHUNK + wave * 16 + col) * CHUNK;
    for (int s = 0; s <= wave * 16; s += 16) {
      const float4_t a = load4(P + s + quad * 4);
#pragma unroll
      for (int j = 0; j < 4; ++j) qs = mfma_f32(a[j], U[(s + quad * 4 + j) * LD + col], qs);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (t0 + r0 + e < p.n) o[(size_t)(t0 + r0 + e) * p.heads * p.E + (size_t)h * p.E + c0 + col] = qs[e];
    }
    const float total = p.total[at];
#pragma unroll
    for (int i = 0; i < TILES; ++i) {
      const int d0 = (wave + i * 4) * 16;
      if (d0 >= D) break;
      float4_t s;
#pragma unroll
      for (int e = 0; e < 4; ++e) s[e] = S[(d0 + quad * 4 + e) * LD + col] * total;
#pragma unroll
      for (int t = 0; t < CHUNK; t += 16) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int r = t + quad * 4 + j;
          s = mfma_f32(to_f32(K[(size_t)min(t0 + r, p.n - 1) * p.ld + d0 + col]), Uk[r * LD + col], s);
        }
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) S[(d0 + quad * 4 + e) * LD + col] = s[e];
    }
  }
  __syncthreads();
  for (int i = tid; i < D * 16; i += 256) St[(size_t)(i >> 4) * p.E + (i & 15)] = S[(i >> 4) * LD + (i & 15)];
}

// out[t][h * E + j] = o / rms(o of the head) * norm[j] * silu(gate): a wavefront per token and head
template <class T>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(T* __restrict__ out, int ldo, const float* __restrict__ o,
                                                             const T* __restrict__ gate, int ldg, delta_args p) {
  const int lane = threadIdx.x & 63, i = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (i >= p.n * p.heads) return;
  const int t = i / p.heads, h = i - t * p.heads;
  const float* src = o + (size_t)i * p.E;
  float s = 0.0f;
  for (int c = lane; c < p.E; c += WAVE) s = fmaf(src[c], src[c], s);  // padding is zero
  const float inv = 1.0f / sqrtf(wave_sum(s) / (float)p.vdim + p.eps);
  for (int c = lane; c < p.E; c += WAVE) {
    const float z = to_f32(gate[(size_t)t * ldg + (size_t)h * p.E + c]);
    out[(size_t)t * ldo + (size_t)h * p.E + c] = (T)(c < p.vdim ? src[c] * inv * p.norm[c] * (z * sigmoid_f32(z)) : 0.0f);
  }
}

// One new token: a workgroup per head holds the head's state in registers, ROWS rows of four columns per thread.
template <int D, int ROWS>
__global__ __launch_bounds__(1024) void delta_step_kernel(bf16_t* __restrict__ out, float* __restrict__ state,
                                                          const bf16_t* __restrict__ qkv, const bf16_t* __restrict__ gate, delta_args p) {
  extern __shared__ __attribute__((aligned(16))) float step_lds[];  // [row groups][2][E]
  __shared__ float qs[D], ks[D], red[16][4];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x, g = h / (p.heads / p.kv_heads);
  const int quads = p.E / 4, groups = 1024 / quads, grp = tid / quads, c = (tid - grp * quads) * 4;
  const bool holds = grp < groups;
  float* St = state + (size_t)h * D * p.E + c;
  float4_t s[ROWS];
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    const int d = grp + r * groups;
    s[r] = holds && d < D ? load4(St + (size_t)d * p.E) : (float4_t)(0.0f);
  }
  float q = 0.0f, k = 0.0f;
  if (tid < D) {
    q = (float)qkv[(size_t)g * D + tid];
    k = (float)qkv[(size_t)(p.kv_heads + g) * D + tid];
    qs[tid] = q;
    ks[tid] = k;
  }
  const float q2 = wave_sum(q * q), k2 = wave_sum(k * k), qk = wave_sum(q * k);
  if (lane == 0) {
    red[wave][0] = q2;
    red[wave][1] = k2;
    red[wave][2] = qk;
  }
  const float beta = sigmoid_f32(p.ba[h]), decay = expf(log_decay(p, p.ba[p.heads + h], h));
  __syncthreads();
  float sq = 0.0f, sk = 0.0f, sqk = 0.0f;
#pragma unroll
  for (int w = 0; w < (D + 63) / 64; ++w) {
    sq += red[w][0];
    sk += red[w][1];
    sqk += red[w][2];
  }
  const float inv_q = 1.0f / sqrtf(sq + UNIT_EPS) / sqrtf((float)p.dim), inv_k = 1.0f / sqrtf(sk + UNIT_EPS);
  float4_t pk = (float4_t)(0.0f), pq = (float4_t)(0.0f);
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    const int d = grp + r * groups;
    if (d < D) {
      const float kd = ks[d], qd = qs[d];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        pk[e] = fmaf(s[r][e], kd, pk[e]);
        pq[e] = fmaf(s[r][e], qd, pq[e]);
      }
    }
  }
  if (holds) {
    store4(step_lds + (size_t)grp * 2 * p.E + c, pk);
    store4(step_lds + (size_t)grp * 2 * p.E + p.E + c, pq);
  }
  __syncthreads();
  // halves of the parts meet: [2 E] sums, `split` threads per sum
  float* sums = step_lds + (size_t)groups * 2 * p.E;  // [2][E]: u, o
  for (int i = tid; i < 2 * p.E; i += 1024) {
    float v = 0.0f;
    for (int x = 0; x < groups; ++x) v += step_lds[(size_t)x * 2 * p.E + i];
    sums[i] = v;
  }
  __syncthreads();
  float o = 0.0f;
  if (tid < p.E) {
    const float v = (float)qkv[(size_t)2 * p.kv_heads * D + (size_t)h * p.E + tid];
    const float u = beta * (v - decay * sums[tid] * inv_k);
    o = decay * sums[p.E + tid] * inv_q + sqk * inv_q * inv_k * u;
    sums[tid] = u * inv_k;
  }
  const float o2 = wave_sum(o * o);
  if (lane == 0) red[wave][3] = o2;
  __syncthreads();
  if (holds) {
    const float4_t u = load4(sums + c);
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
      const int d = grp + r * groups;
      if (d < D) {
        const float kd = ks[d];
#pragma unroll
        for (int e = 0; e < 4; ++e) s[r][e] = fmaf(kd, u[e], decay * s[r][e]);
        store4(St + (size_t)d * p.E, s[r]);
      }
    }
  }
  if (tid < p.E) {
    float total = 0.0f;
    for (int w = 0; w < (p.E + 63) / 64; ++w) total += red[w][3];
    const float z = (float)gate[(size_t)h * p.E + tid];
    out[(size_t)h * p.E + tid] =
        (bf16_t)(tid < p.vdim ? o * (1.0f / sqrtf(total / (float)p.vdim + p.eps)) * p.norm[tid] * (z * sigmoid_f32(z)) : 0.0f);
  }
}

int check_delta(const char* who, const lcu_delta_params* d, int dtype) {
  LCU_REQUIRE(d && d->a_log_dev && d->dt_bias_dev && d->norm_dev, "%s: null pointer", who);
  LCU_REQUIRE(dtype == LCU_BF16 || dtype == LCU_F32, "%s: element type %d", who, dtype);
  LCU_REQUIRE(d->heads > 0 && d->kv_heads > 0 && d->heads % d->kv_heads == 0 && d->heads <= 65535 &&
                  (d->dk == 32 || d->dk == 64 || d->dk == 128 || d->dk == 256) && d->dv > 0 && d->dv % 32 == 0 && d->dv <= 256 &&
                  d->dim > 0 && d->dim <= d->dk && d->vdim > 0 && d->vdim <= d->dv,
              "%s: heads %d / %d, head size %d in %d (32, 64, 128, 256), value size %d in %d (a multiple of 32, at most 256)", who, d->heads,
              d->kv_heads, d->dim, d->dk, d->vdim, d->dv);
  return LCU_OK;
}

delta_args make_delta(const lcu_delta_params* d, const void* ba, int ld_ba, int n, int ld) {
  delta_args p{};
  p.heads = d->heads;
  p.kv_heads = d->kv_heads;
  p.E = d->dv;
  p.dim = d->dim;
  p.vdim = d->vdim;
  p.n = n;
  p.ld = ld;
  p.ba = (const float*)ba;
  p.ld_ba = ld_ba;
  p.a_log = (const float*)d->a_log_dev;
  p.dt_bias = (const float*)d->dt_bias_dev;
  p.norm = (const float*)d->norm_dev;
  p.eps = d->eps;
  return p;
}

template <class F>
void with_head_size(int dk, F&& f) {
  switch (dk) {
    case 32: f(std::integral_constant<int, 32>{}); break;
    case 64: f(std::integral_constant<int, 64>{}); break;
    case 128: f(std::integral_constant<int, 128>{}); break;
    default: f(std::integral_constant<int, 256>{}); break;
  }
}

int delta_channels(const lcu_delta_params* d) { return 2 * d->kv_heads * d->dk + d->heads * d->dv; }

}  // namespace

extern "C" {

size_t lcu_delta_rule_scratch(const lcu_delta_params* d, int n) {
  if (d == nullptr || n <= 0) return 0;
  const size_t chunks = ((size_t)n + CHUNK - 1) / CHUNK;
  return ((size_t)d->heads * chunks * (CHUNK * ((size_t)d->dk + d->dv + CHUNK + 2) + 1) + (size_t)n * d->heads * d->dv) * sizeof(float);
}

int lcu_delta_rule(void* out_dev, int ldo, const void* qkv_dev, int ld, const void* gate_dev, int ldg, const void* ba_f32_dev, int ld_ba,
                   const lcu_delta_params* d, void* state_dev, void* scratch_dev, int dtype, int n, void* stream) {
  LCU_REQUIRE(out_dev && qkv_dev && gate_dev && ba_f32_dev && state_dev && scratch_dev, "lcu_delta_rule: null pointer");
  const int rc = check_delta("lcu_delta_rule", d, dtype);
  if (rc) return rc;
  LCU_REQUIRE(n >= 0 && n <= 65535 && ld >= delta_channels(d) && ld % 8 == 0 && ldo >= d->heads * d->dv && ldg >= d->heads * d->dv &&
                  ld_ba >= 2 * d->heads,
              "lcu_delta_rule: bad shape n %d strides %d %d %d %d", n, ld, ldo, ldg, ld_ba);
  if (n == 0) return LCU_OK;
  hipStream_t st = as_stream(stream);
  delta_args p = make_delta(d, ba_f32_dev, ld_ba, n, ld);
  const int chunks = (n + CHUNK - 1) / CHUNK;
  const size_t units = (size_t)d->heads * chunks;
  p.X = (float*)scratch_dev;
  p.Y = p.X + units * CHUNK * d->dv;
  p.P = p.Y + units * CHUNK * d->dk;
  p.rows = p.P + units * CHUNK * CHUNK;
  float* o = p.rows + units * CHUNK * 2;
  p.total = o + (size_t)n * d->heads * d->dv;
  const unsigned norms = (unsigned)(((size_t)n * d->heads + 3) / 4);
  const auto run = [&](auto* kind, auto size) {
    using T = std::remove_pointer_t<decltype(kind)>;
    constexpr int D = decltype(size)::value;
    delta_chunk_kernel<T, D><<<dim3(d->heads, chunks), 256, 0, st>>>((const T*)qkv_dev, p);
    delta_scan_kernel<T, D><<<dim3(d->heads, d->dv / 16), 256, 0, st>>>(o, (float*)state_dev, (const T*)qkv_dev, chunks, p);
    head_norm_gate_kernel<T><<<norms, 256, 0, st>>>((T*)out_dev, ldo, o, (const T*)gate_dev, ldg, p);
  };
  with_head_size(d->dk, [&](auto size) {
    if (dtype == LCU_F32) {
      run((float*)nullptr, size);
    } else {
      run((bf16_t*)nullptr, size);
    }
  });
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_decode_delta_step(void* out_dev, const void* qkv_dev, const void* gate_dev, const void* ba_f32_dev, const lcu_delta_params* d,
                          void* state_dev, void* stream) {
  LCU_REQUIRE(out_dev && qkv_dev && gate_dev && ba_f32_dev && state_dev, "lcu_decode_delta_step: null pointer");
  const int rc = check_delta("lcu_decode_delta_step", d, LCU_BF16);
  if (rc) return rc;
  const delta_args p = make_delta(d, ba_f32_dev, 2 * d->heads, 1, delta_channels(d));
  const int groups = 1024 / (d->dv / 4), per = (d->dk + groups - 1) / groups;
  const size_t lds = ((size_t)groups + 1) * 2 * d->dv * sizeof(float);
  hipStream_t st = as_stream(stream);
  const auto go = [&](auto size, auto rows) {
    delta_step_kernel<decltype(size)::value, decltype(rows)::value><<<d->heads, 1024, lds, st>>>(
        (bf16_t*)out_dev, (float*)state_dev, (const bf16_t*)qkv_dev, (const bf16_t*)gate_dev, p);
  };
  using std::integral_constant;
  with_head_size(d->dk, [&](auto size) {
    if (per <= 2) {
      go(size, integral_constant<int, 2>{});
    } else if (per <= 4) {
      go(size, integral_constant<int, 4>{});
    } else if (per <= 8) {
      go(size, integral_constant<int, 8>{});
    } else if (per <= 16) {
      go(size, integral_constant<int, 16>{});
    } else {
      go(size, integral_constant<int, 32>{});
    }
  });
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

}  // extern "C"
