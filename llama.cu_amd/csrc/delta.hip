// Gated delta rule (Yang, Kautz, Hatamizadeh: "Gated Delta Networks: Improving Mamba2 with Delta Rule").  Per head, with
// state S [D][E] and unit vectors q, k:
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// beta = sigmoid(b), log g = -exp(A_log) softplus(a + dt_bias).
//
// Channels of a token: q [kv_heads * D] | k [kv_heads * D] | v [heads * E], after their convolution; D is the head size
// padded to 32, 64, 128 or 256 and E the value size padded to a multiple of 32, padding zero.  Everything here is fp32
// but these channels and the result, which have the element type; products run on the fp32 matrix cores, or on the
// bfloat16 ones where both operands are channels as stored (their products are exact in fp32).
//
// Several tokens: chunks of 64.  With G_t the sum of log g up to t inside the chunk and S the state that enters it,
//   u_t + beta_t sum_(s<t) e^(G_t - G_s) (k_s . k_t) u_s = r_t = beta_t (v_t - e^G_t S^T k_t)
//   o_t = e^G_t S^T q_t + sum_(s<=t) e^(G_t - G_s) (k_s . q_t) u_s
//   S'  = e^G_64 S + sum_s e^(G_64 - G_s) k_s u_s^T
// or u = T r and o = e^G S^T q + P T r, with T the inverse of the unit triangular matrix of the first line and P the
// factors of the second.  The chunk kernel leaves T and P T of every chunk at once; the scan kernel runs over the chunks,
// sixteen columns of S per workgroup.  No exponent is ever positive.
//
// Where the channels are bfloat16, the products with S and u have one operand that bfloat16 holds exactly; the fp32 one goes
// in as three bfloat16 terms, which together hold all of its bits.
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
  // per (head, chunk): T and P T [64][64], on and below the diagonal blocks; per row the factors beta, beta e^G / |k|,
  // e^G / |q|, e^(G_64 - G) / |k| [4][64]; e^G_64.  Per (q/k head, chunk): the keys transposed [D][64], in their own type.
  float* T;
  float* PT;
  float* rows;
  float* total;
  void* Kt;
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

// One workgroup: one chunk of one head.  `role`, one per wavefront: a block of sixteen rows, then a block of columns.
template <class T, int D>
__global__ __launch_bounds__(256) void delta_chunk_kernel(const T* __restrict__ qkv, delta_args p) {
  constexpr int LDA = CHUNK + 4;
  // A: beta_t e^(G_t - G_s) k_t . k_s, s < t, whose diagonal blocks the inverses of theirs replace; P
  __shared__ __attribute__((aligned(16))) float A[CHUNK * LDA], P[CHUNK * LDA];
  __shared__ float Gs[CHUNK], beta[CHUNK], inv_q[CHUNK], inv_k[CHUNK];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, quad = lane >> 4;
  const int role = (wave + blockIdx.x + blockIdx.y) & 3;  // the roles differ in length
  const int h = blockIdx.x, chunk = blockIdx.y, group = p.heads / p.kv_heads, g = h / group, t0 = chunk * CHUNK;
  const size_t at = (size_t)h * gridDim.y + chunk;
  const T* Q = qkv + (size_t)g * D;
  const T* K = qkv + (size_t)(p.kv_heads + g) * D;
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
  if (h == g * group) {
    T* Kt = (T*)p.Kt + ((size_t)g * gridDim.y + chunk) * D * CHUNK;
    const size_t r = row(lane);
#pragma unroll 2
    for (int d = wave * 4; d < D; d += 16) {
      const float4_t k = load4(K + r + d);
#pragma unroll
      for (int e = 0; e < 4; ++e) Kt[(size_t)(d + e) * CHUNK + lane] = (T)k[e];
    }
  }
  __syncthreads();
#pragma unroll 1
  for (int ct = 0; ct <= role; ++ct) {
    const T* y = K + row(ct * 16 + col);
    const float4_t kk = row_products<D>(K + row(role * 16 + col), y, (float4_t)(0.0f));
    const float4_t qk = row_products<D>(Q + row(role * 16 + col), y, (float4_t)(0.0f));
    const int s = ct * 16 + col;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = role * 16 + quad * 4 + e;
      const float f = s <= t ? expf(Gs[t] - Gs[s]) * inv_k[s] : 0.0f;
      A[t * LDA + s] = s < t ? beta[t] * inv_k[t] * f * kk[e] : 0.0f;
      P[t * LDA + s] = inv_q[t] * f * qk[e];
    }
  }
  if (tid < CHUNK) {
    const float G = Gs[tid], end = Gs[CHUNK - 1];
    float* rows = p.rows + at * 4 * CHUNK + tid;
    rows[0] = beta[tid];
    rows[CHUNK] = beta[tid] * expf(G) * inv_k[tid];
    rows[2 * CHUNK] = expf(G) * inv_q[tid];
    rows[3 * CHUNK] = expf(end - G) * inv_k[tid];
    if (tid == 0) p.total[at] = expf(end);
  }
  {
    // the inverse of the role's own diagonal block, written by this wavefront alone; lane = column
    float* B = A + role * 16 * (LDA + 1);
    float x[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      float acc = t == col ? 1.0f : 0.0f;
#pragma unroll
      for (int s4 = 0; s4 < t; s4 += 4) {
        const float4_t a = load4(B + t * LDA + s4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          if (s4 + e < t) acc = fmaf(-a[e], x[s4 + e], acc);
        }
      }
      x[t] = acc;
    }
    if (quad == 0) {
#pragma unroll
      for (int t = 0; t < 16; ++t) B[t * LDA + col] = x[t];
    }
  }
  __syncthreads();
  // Block column `role` of T, top to bottom: T_ij = -T_ii sum_m A_im T_mj.  A tile as it leaves the matrix core (four
  // neighbouring rows per lane) is the second operand of the next product, its rows taken in the order of the lanes.
  const auto times = [&](const float* M, int i, int m, float4_t b, float4_t acc) {
    const float4_t a = load4(M + (i * 16 + col) * LDA + m * 16 + quad * 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) acc = mfma_f32(a[e], b[e], acc);
    return acc;
  };
  float4_t t[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    t[i] = (float4_t)(0.0f);
    if (i == role) {
#pragma unroll
      for (int e = 0; e < 4; ++e) t[i][e] = A[(i * 16 + quad * 4 + e) * LDA + i * 16 + col];
    } else if (i > role) {
      float4_t sum = (float4_t)(0.0f);
#pragma unroll
      for (int m = 0; m < i; ++m) {
        if (m >= role) sum = times(A, i, m, t[m], sum);
      }
      t[i] = times(A, i, i, -sum, t[i]);
    }
  }
  float* To = p.T + at * CHUNK * CHUNK + role * 16 + col;
  float* PTo = p.PT + at * CHUNK * CHUNK + role * 16 + col;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    if (i < role) continue;
    float4_t sum = (float4_t)(0.0f);
#pragma unroll
    for (int m = 0; m <= i; ++m) {
      if (m >= role) sum = times(P, i, m, t[m], sum);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      To[(i * 16 + quad * 4 + e) * CHUNK] = t[i][e];
      PTo[(i * 16 + quad * 4 + e) * CHUNK] = sum[e];
    }
  }
}

// fp32 values as matrix operands: three bfloat16 terms beside bfloat16 channels, one value beside fp32 ones.  An array is
// [terms][16 columns][LD], along the products' inner dimension.
template <class T>
struct terms_of;
template <>
struct terms_of<float> {
  static constexpr int COUNT = 1, STEP = 16, PER = 4, PAD = 4;  // inner extent of a step, elements of a lane
  typedef float4_t piece;
};
template <>
struct terms_of<bf16_t> {
  static constexpr int COUNT = 3, STEP = 32, PER = 8, PAD = 8;
  typedef bf16x8_t piece;
};
typedef bf16_t bf16x4_t __attribute__((ext_vector_type(4)));

template <int LD>
__device__ __forceinline__ void put_terms(float* dst, int c, int at, float4_t v) {
  store4(dst + c * LD + at, v);
}
template <int LD>
__device__ __forceinline__ void put_terms(bf16_t* dst, int c, int at, float4_t v) {
#pragma unroll
  for (int term = 0; term < 3; ++term) {
    bf16x4_t x;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      x[e] = (bf16_t)v[e];
      v[e] -= (float)x[e];
    }
    *reinterpret_cast<bf16x4_t*>(dst + (term * 16 + c) * LD + at) = x;
  }
}
template <int LD>
__device__ __forceinline__ float4_t step_product(float4_t a, const float* terms, int col, int at, float4_t acc) {
  const float4_t b = load4(terms + col * LD + at);
#pragma unroll
  for (int e = 0; e < 4; ++e) acc = mfma_f32(a[e], b[e], acc);
  return acc;
}
template <int LD>
__device__ __forceinline__ float4_t step_product(bf16x8_t a, const bf16_t* terms, int col, int at, float4_t acc) {
#pragma unroll
  for (int term = 2; term >= 0; --term) {
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, *reinterpret_cast<const bf16x8_t*>(terms + (term * 16 + col) * LD + at), acc, 0, 0, 0);
  }
  return acc;
}

// One workgroup: sixteen columns of one head's state through all chunks.  Wavefronts 0 .. 3 take sixteen rows of a chunk
// each and work out u, wavefronts 4 .. 7 take the same rows and work out o; each keeps up to TILES blocks of sixteen rows of the
// state in registers and brings them up to date, and LDS holds all of the state as operands.  What the next chunk needs
// from memory is asked for as soon as this chunk's has been used.  o: fp32 [n][heads * E].
template <class T, int D>
__global__ __launch_bounds__(512) void delta_scan_kernel(float* __restrict__ o, float* __restrict__ state, const T* __restrict__ qkv,
                                                         int chunks, delta_args p) {
  typedef terms_of<T> terms;
  typedef typename terms::piece piece;
  constexpr int STEPS = D / terms::STEP, CSTEPS = CHUNK / terms::STEP, TILES = (D / 16 + 7) / 8;
  constexpr int LDR = CHUNK + 4, LDU = CHUNK + terms::PAD, LDD = D + terms::PAD;
  __shared__ __attribute__((aligned(16))) T S[terms::COUNT * 16 * LDD];
  __shared__ __attribute__((aligned(16))) T U[terms::COUNT * 16 * LDU];  // u times the row's factor of k
  __shared__ __attribute__((aligned(16))) float R[16 * LDR];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 15, quad = lane >> 4;
  const int block = wave & 3, r0 = block * 16 + quad * 4;
  const bool of_u = wave < 4;
  const int h = blockIdx.x, c0 = blockIdx.y * 16, g = h / (p.heads / p.kv_heads);
  const T* QK = qkv + (size_t)(of_u ? p.kv_heads + g : g) * D;
  const T* V = qkv + (size_t)2 * p.kv_heads * D + (size_t)h * p.E + c0;
  float* St = state + (size_t)h * D * p.E + c0 + col;
  // offsets of this lane, beside uniform pointers; rows behind the last token are the last one again
  const unsigned ld = p.ld, last = (unsigned)(p.n - 1) * ld, row = (unsigned)(block * 16 + col) * ld, v_row = (unsigned)r0 * ld;
  const unsigned m_at = (block * 16 + col) * CHUNK + quad * 4, o_ld = p.heads * p.E, o_at = r0 * o_ld + col;
  unsigned kt_at[TILES];
#pragma unroll
  for (int i = 0; i < TILES; ++i) kt_at[i] = (min((wave + i * 8) * 16, D - 16) + col) * CHUNK + quad * terms::PER;

  piece x[STEPS];  // rows of k or q
  const auto fetch_rows = [&](int chunk) {
    const unsigned r = min((unsigned)chunk * CHUNK * ld + row, last) + quad * terms::PER;
#pragma unroll
    for (int i = 0; i < STEPS; ++i) x[i] = *reinterpret_cast<const piece*>(QK + r + i * terms::STEP);
  };
  T v[4];
  float4_t beta, of_k;
  const auto fetch_values = [&](int chunk) {
    const float* rows = p.rows + ((size_t)h * chunks + chunk) * 4 * CHUNK;
    beta = load4(rows + (unsigned)r0);
    of_k = load4(rows + CHUNK + (unsigned)r0);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = V[min((unsigned)chunk * CHUNK * ld + v_row + e * ld, last) + col];
  };
  float4_t m[4], factor;  // rows of T or P T; e^(G_64 - G) / |k| or e^G / |q|
  const auto fetch_matrix = [&](int chunk) {
    const size_t at = (size_t)h * chunks + chunk;
    const float* src = (of_u ? p.T : p.PT) + at * CHUNK * CHUNK;
    factor = load4(p.rows + at * 4 * CHUNK + (of_u ? 3 : 2) * CHUNK + (unsigned)r0);
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      if (b <= block) m[b] = load4(src + b * 16 + m_at);
    }
  };
  piece kt[TILES * CSTEPS];  // transposed keys
  float total;
  const auto fetch_keys = [&](int chunk) {
    const T* src = (const T*)p.Kt + ((size_t)g * chunks + chunk) * D * CHUNK;
#pragma unroll
    for (int i = 0; i < TILES; ++i) {
#pragma unroll
      for (int c = 0; c < CSTEPS; ++c) kt[i * CSTEPS + c] = *reinterpret_cast<const piece*>(src + kt_at[i] + c * terms::STEP);
    }
    total = p.total[(size_t)h * chunks + chunk];
  };
  fetch_rows(0);
  if (of_u) fetch_values(0);
  fetch_matrix(0);
  fetch_keys(0);
  float4_t s[TILES];
#pragma unroll
  for (int i = 0; i < TILES; ++i) {
    const int d0 = (wave + i * 8) * 16 + quad * 4;
    if (d0 >= D) break;
#pragma unroll
    for (int e = 0; e < 4; ++e) s[i][e] = St[(size_t)(d0 + e) * p.E];
    put_terms<LDD>(S, col, d0, s[i]);
  }
#pragma unroll 1
  for (int chunk = 0; chunk < chunks; ++chunk) {
    const int next = min(chunk + 1, chunks - 1);
    __syncthreads();  // S is whole
    float4_t xs = (float4_t)(0.0f);
#pragma unroll
    for (int i = 0; i < STEPS; ++i) xs = step_product<LDD>(x[i], S, col, i * terms::STEP + quad * terms::PER, xs);
    fetch_rows(next);
    if (of_u) {
      float4_t r;
#pragma unroll
      for (int e = 0; e < 4; ++e) r[e] = beta[e] * to_f32(v[e]) - of_k[e] * xs[e];
      store4(R + col * LDR + r0, r);
      fetch_values(next);
    }
    __syncthreads();  // R is whole, S has been read
    float4_t y = (float4_t)(0.0f);
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      if (b <= block) {
        const float4_t r = load4(R + col * LDR + b * 16 + quad * 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) y = mfma_f32(m[b][e], r[e], y);
      }
    }
    if (of_u) {
#pragma unroll
      for (int e = 0; e < 4; ++e) y[e] *= factor[e];
      put_terms<LDU>(U, col, r0, y);
    } else {
      float* out = o + (size_t)chunk * CHUNK * o_ld + h * p.E + c0;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        if (chunk * CHUNK + r0 + e < p.n) out[o_at + e * o_ld] = fmaf(factor[e], xs[e], y[e]);
      }
    }
    fetch_matrix(next);
    __syncthreads();  // U is whole, R has been read
#pragma unroll
    for (int i = 0; i < TILES; ++i) {
      const int d0 = (wave + i * 8) * 16 + quad * 4;
      if (d0 >= D) break;
#pragma unroll
      for (int e = 0; e < 4; ++e) s[i][e] *= total;
#pragma unroll
      for (int c = 0; c < CSTEPS; ++c) {
        s[i] = step_product<LDU>(kt[i * CSTEPS + c], U, col, c * terms::STEP + quad * terms::PER, s[i]);
      }
      put_terms<LDD>(S, col, d0, s[i]);
    }
    fetch_keys(next);
  }
#pragma unroll
  for (int i = 0; i < TILES; ++i) {
    const int d0 = (wave + i * 8) * 16 + quad * 4;
    if (d0 >= D) break;
#pragma unroll
    for (int e = 0; e < 4; ++e) St[(size_t)(d0 + e) * p.E] = s[i][e];
  }
}

// out[t][h * E + j] = o / rms(o of the head) * norm[j] * silu(gate): `lanes` lanes (8 .. 64) per token and head, four
// values each
template <class T>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(T* __restrict__ out, int ldo, const float* __restrict__ o,
                                                             const T* __restrict__ gate, int ldg, int lanes, delta_args p) {
  const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) / lanes;
  const int c = (threadIdx.x & (lanes - 1)) * 4;
  const bool has = i < (size_t)p.n * p.heads && c < p.E;
  const size_t t = i / p.heads, h = i - t * p.heads;
  const float4_t x = has ? load4(o + i * p.E + c) : (float4_t)(0.0f), z = has ? load4(gate + t * ldg + h * p.E + c) : (float4_t)(0.0f);
  float s = fmaf(x[0], x[0], fmaf(x[1], x[1], fmaf(x[2], x[2], x[3] * x[3])));  // padding is zero
  for (int off = lanes >> 1; off > 0; off >>= 1) s += __shfl_xor(s, off, WAVE);
  const float inv = 1.0f / sqrtf(s / (float)p.vdim + p.eps);
  if (!has) return;
  float4_t y;
#pragma unroll
  for (int e = 0; e < 4; ++e) y[e] = c + e < p.vdim ? x[e] * inv * p.norm[c + e] * (z[e] * sigmoid_f32(z[e])) : 0.0f;
  store4(out + t * ldo + h * p.E + c, y);
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
  return (chunks * ((size_t)d->heads * (2 * CHUNK * CHUNK + 4 * CHUNK + 1) + (size_t)d->kv_heads * d->dk * CHUNK + 4) +
          (size_t)n * d->heads * d->dv) * sizeof(float);
}

int lcu_delta_rule(void* out_dev, int ldo, const void* qkv_dev, int ld, const void* gate_dev, int ldg, const void* ba_f32_dev, int ld_ba,
                   const lcu_delta_params* d, void* state_dev, void* scratch_dev, int dtype, int n, void* stream) {
  LCU_REQUIRE(out_dev && qkv_dev && gate_dev && ba_f32_dev && state_dev && scratch_dev, "lcu_delta_rule: null pointer");
  const int rc = check_delta("lcu_delta_rule", d, dtype);
  if (rc) return rc;
  LCU_REQUIRE(n >= 0 && n <= 65535 && ld >= delta_channels(d) && ld % 8 == 0 && ldo >= d->heads * d->dv && ldg >= d->heads * d->dv &&
                  ld_ba >= 2 * d->heads,
              "lcu_delta_rule: bad shape n %d strides %d %d %d %d", n, ld, ldo, ldg, ld_ba);
  LCU_REQUIRE(((size_t)n + 2 * CHUNK) * ld < ((size_t)1 << 32), "lcu_delta_rule: %d rows of %d", n, ld);
  if (n == 0) return LCU_OK;
  hipStream_t st = as_stream(stream);
  delta_args p = make_delta(d, ba_f32_dev, ld_ba, n, ld);
  const int chunks = (n + CHUNK - 1) / CHUNK;
  const size_t units = (size_t)d->heads * chunks;
  p.T = (float*)scratch_dev;
  p.PT = p.T + units * CHUNK * CHUNK;
  p.rows = p.PT + units * CHUNK * CHUNK;
  float* o = p.rows + units * 4 * CHUNK;
  float* Kt = o + (size_t)n * d->heads * d->dv;
  p.Kt = Kt;
  p.total = Kt + (size_t)d->kv_heads * chunks * d->dk * CHUNK;
  const int lanes = d->dv <= 32 ? 8 : d->dv <= 64 ? 16 : d->dv <= 128 ? 32 : 64;
  const unsigned norms = (unsigned)(((size_t)n * d->heads * lanes + 255) / 256);
  const auto run = [&](auto* kind, auto size) {
    using T = std::remove_pointer_t<decltype(kind)>;
    constexpr int D = decltype(size)::value;
    delta_chunk_kernel<T, D><<<dim3(d->heads, chunks), 256, 0, st>>>((const T*)qkv_dev, p);
    delta_scan_kernel<T, D><<<dim3(d->heads, d->dv / 16), 512, 0, st>>>(o, (float*)state_dev, (const T*)qkv_dev, chunks, p);
    head_norm_gate_kernel<T><<<norms, 256, 0, st>>>((T*)out_dev, ldo, o, (const T*)gate_dev, ldg, lanes, p);
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
