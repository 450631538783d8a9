// Latent attention (DeepSeek-AI, "DeepSeek-V2: A Strong, Economical, and Efficient Mixture-of-Experts Language Model"):
// keys and values of all heads are products of one normed latent c per token, and a rotated key part, if there is
// one, is shared by the heads.  The caches hold c [positions][ldc] and the rotated part [positions][dr].
//
// Two ways to attend, the same sums in another order.  Long prompts: keys and values are multiplied out of the latents
// (an ordinary product) and go to the kernels of windowed.hip.  One or a few tokens: the head's key matrix is applied to
// the query instead, q_h . (U_h c) = (U_h^T q_h) . c, so that scores and weighted sums are over the latents themselves,
// which are read once for sixteen rows (heads of a token, or of neighbouring tokens) together; the weighted latent
// then passes through the head's value matrix.
//
// Padding: unrotated and rotated head parts to multiples of 32 (dn, dr), ldc to a multiple of 64, values to dv; zeros.
#include <algorithm>
#include <type_traits>

#include "linear.hpp"
#include "rownorm.hpp"

using namespace lcu;

namespace {

// ---- row kernel -----------------------------------------------------------------------------------------
struct latent_row_args {
  void* rows;            // projected rows: queries (or their latent), c, rotated key part
  int ld, n;
  int latent_at, rank, ldc;
  const float* latent_norm;
  void* latents;         // cache [max_pos][ldc]
  int key_at, rot, dr;   // rotated dimensions (0: none) of the dr of the shared key part
  void* keys;            // cache [max_pos][dr]
  int query_at, heads, head_ld;  // rotated part of head h at query_at + h * head_ld; heads 0: none here
  const float* freq;     // [rot / 2]
  float gain;            // on cos and sin
  int low_rank, low_ld;  // latent of the queries at column 0, 0: none
  const float* low_norm;
  void* low;             // [n][low_ld]
  const int* start;
  int max_pos;
  float eps;
};

// dst = rms norm of src[0 .. count) times w, padding zero; one wavefront
template <class T>
__device__ __forceinline__ void norm_part(T* __restrict__ dst, const T* __restrict__ src, const float* __restrict__ w, int count, int ld,
                                          float eps) {
  const int lane = threadIdx.x & 63;
  float s = 0.0f;
  for (int c = lane * 4; c < ld; c += WAVE * 4) {
    const float4_t v = load4(src + c);
#pragma unroll
    for (int e = 0; e < 4; ++e) s = fmaf(v[e], v[e], s);  // padding is zero
  }
  const float inv = 1.0f / sqrtf(wave_sum(s) / (float)count + eps);
  for (int c = lane * 4; c < ld; c += WAVE * 4) store4(dst + c, load4(src + c) * inv * load4(w + c));
}

// pairs (2i, 2i + 1) of src[0 .. rot) turned by angle position * freq[i]; i in steps of `step`
template <class T>
__device__ __forceinline__ void rotate_part(T* dst, const T* src, const latent_row_args& p, float position, int i) {
  const float a = position * p.freq[i];
  float sn, cs;
  sincosf(a, &sn, &cs);
  sn *= p.gain;
  cs *= p.gain;
  const float u = to_f32(src[2 * i]), v = to_f32(src[2 * i + 1]);
  dst[2 * i] = (T)fmaf(u, cs, -(v * sn));
  dst[2 * i + 1] = (T)fmaf(v, cs, u * sn);
}

// one token: wavefront 0 the latent, wavefront 1 the queries' latent, the others (and these afterwards) the rotations
template <class T>
__device__ __forceinline__ void latent_row(const latent_row_args& p, int t) {
  const int tid = threadIdx.x, wave = tid >> 6;
  const int pos = min(max(*p.start + t, 0), p.max_pos - 1);
  T* row = (T*)p.rows + (size_t)t * p.ld;
  if (wave == 0) norm_part((T*)p.latents + (size_t)pos * p.ldc, row + p.latent_at, p.latent_norm, p.rank, p.ldc, p.eps);
  if (wave == 1 && p.low_rank > 0) norm_part((T*)p.low + (size_t)t * p.low_ld, row, p.low_norm, p.low_rank, p.low_ld, p.eps);
  if (p.dr == 0) return;
  const int half = p.rot / 2;
  T* key = (T*)p.keys + (size_t)pos * p.dr;
  for (int i = tid; i < p.dr / 2; i += 256) {
    if (i < half) {
      rotate_part(key, row + p.key_at, p, (float)pos, i);
    } else {
      key[2 * i] = row[p.key_at + 2 * i];
      key[2 * i + 1] = row[p.key_at + 2 * i + 1];
    }
  }
  for (int i = tid; i < p.heads * half; i += 256) {
    T* q = row + p.query_at + (size_t)(i / half) * p.head_ld;
    rotate_part(q, q, p, (float)pos, i % half);
  }
}

template <class T>
__global__ __launch_bounds__(256) void latent_rows_kernel(latent_row_args p) {
  latent_row<T>(p, blockIdx.x);
}

// ---- head by head products, few tokens ------------------------------------------------------------------
// out[t][h * N + j] = sum_k in[t * ldi + h * in_h + k] w[(h * N + j) * K + k].  Workgroup: 64 columns of one head, 16
// tokens.  The workgroups behind the products of the first sixteen tokens take the row kernel's tokens.
__global__ __launch_bounds__(256) void head_products_kernel(bf16_t* __restrict__ out, int ldo, const bf16_t* __restrict__ in, int ldi,
                                                            int in_h, const bf16_t* __restrict__ w, int N, int K, int n, int products,
                                                            latent_row_args rows) {
  if ((int)blockIdx.x >= products) {
    latent_row<bf16_t>(rows, blockIdx.x - products);
    return;
  }
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, col = lane & 15, quad = lane >> 4;
  const int per_head = N / 64, tiles = per_head * ((n + 15) / 16), h = blockIdx.x / tiles, rest = blockIdx.x - h * tiles;
  const int t0 = rest / per_head * 16, j = (rest % per_head) * 64 + wave * 16 + col;
  const bf16_t* a = in + (size_t)min(t0 + col, n - 1) * ldi + (size_t)h * in_h + quad * 8;
  const bf16_t* b = w + ((size_t)h * N + j) * K + quad * 8;
  float4_t acc = (float4_t)(0.0f);
#pragma unroll 8
  for (int k = 0; k < K; k += 32) {
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(a + k), *reinterpret_cast<const bf16x8_t*>(b + k), acc,
                                                  0, 0, 0);
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int t = t0 + quad * 4 + e;
    if (t < n) out[(size_t)t * ldo + (size_t)h * N + j] = (bf16_t)acc[e];
  }
}

// ---- scores and weighted sums over the latents ----------------------------------------------------------
// Row r of the n * heads query rows belongs to token r / heads, head r % heads.  Workgroup (sixteen rows, slice of the
// keys), keys in tiles of 64, sixteen per wavefront: a wavefront takes its keys' latents from memory straight into
// matrix operands, multiplies them with the rows, and leaves them transposed in LDS for the weighted sums, of which it
// then takes a fourth of the columns over all 64 keys.  Probabilities go in as two bfloat16 terms (value and remainder).
// A slice's sums go to part[slice][row][ldc], its maximum and sum to ml[slice][row][2]; a slice without keys leaves a sum
// of zero and nothing else.
struct latent_args {
  int heads, n, ldc, dr, window, slices;
  float scale;
  const bf16_t* q;       // [n][heads * ldc]
  const bf16_t* q_rot;   // head h of token t at t * ldq + h * head_ld
  int ldq, head_ld;
  const bf16_t* c;
  const bf16_t* keys;
  const int* start;
  int max_pos;
  float* part;
  float* ml;
};
constexpr int LROWS = 16, LKEYS = 64, LDV = LKEYS + 8;

template <int NT>
__global__ __launch_bounds__(256) void latent_attention_kernel(latent_args p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char latent_lds[];
  __shared__ float red[2][4][LROWS];
  const int ldk = p.ldc + p.dr + 8;
  bf16_t* Qs = reinterpret_cast<bf16_t*>(latent_lds);  // [16][ldk]: latent part, rotated part
  bf16_t* Vt = Qs + LROWS * ldk;                       // [ldc][LDV]
  bf16_t* Ps = Vt + p.ldc * LDV;                       // [value, remainder][16][LDV]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, quad = lane >> 4;
  const int rows = p.n * p.heads, r0 = blockIdx.x * LROWS, slice = blockIdx.y;
  const int first = min(max(*p.start, 0), p.max_pos - p.n);
  const int hi = first + min(r0 + LROWS - 1, rows - 1) / p.heads, lo = max(0, first + r0 / p.heads - p.window + 1);
  const int tiles = (hi - lo) / LKEYS + 1, per = (tiles + p.slices - 1) / p.slices;
  const int tile0 = slice * per, tile1 = min(tile0 + per, tiles);
  float* ml = p.ml + ((size_t)slice * rows + r0) * 2;
  if (tile0 >= tile1) {
    if (tid < LROWS && r0 + tid < rows) {
      ml[tid * 2] = -1e30f;
      ml[tid * 2 + 1] = 0.0f;
    }
    return;
  }
  const int c8 = p.ldc / 8, k8 = (p.ldc + p.dr) / 8;
  for (int i = tid; i < LROWS * k8; i += 256) {
    const int r = i / k8, e = i - r * k8, row = min(r0 + r, rows - 1), t = row / p.heads, h = row - t * p.heads;
    const bf16_t* src = e < c8 ? p.q + (size_t)row * p.ldc + e * 8 : p.q_rot + (size_t)t * p.ldq + (size_t)h * p.head_ld + (e - c8) * 8;
    *reinterpret_cast<uint4_t*>(Qs + r * ldk + e * 8) = *reinterpret_cast<const uint4_t*>(src);
  }
  int at[4];  // positions of this lane's rows
  float m[4], l[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    at[e] = first + min(r0 + quad * 4 + e, rows - 1) / p.heads;
    m[e] = -1e30f;
    l[e] = 0.0f;
  }
  float4_t o[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) o[i] = (float4_t)(0.0f);
  __syncthreads();
  for (int tile = tile0; tile < tile1; ++tile) {
    const int j = lo + tile * LKEYS + wave * 16 + col;  // this lane's key
    const bf16_t* c = p.c + (size_t)min(j, hi) * p.ldc + quad * 8;
    bf16x8_t kv[2 * NT];
#pragma unroll
    for (int f = 0; f < 2 * NT; ++f) kv[f] = f * 32 < p.ldc ? *reinterpret_cast<const bf16x8_t*>(c + f * 32) : (bf16x8_t)(0.0f);
    float4_t s = (float4_t)(0.0f);
    const bf16_t* qr = Qs + col * ldk + quad * 8;
    for (int k = 0; k < p.dr; k += 32) {
      s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(qr + p.ldc + k),
                                                  *reinterpret_cast<const bf16x8_t*>(p.keys + (size_t)min(j, hi) * p.dr + quad * 8 + k), s, 0,
                                                  0, 0);
    }
#pragma unroll
    for (int f = 0; f < 2 * NT; ++f) {
      if (f * 32 < p.ldc) {
        s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(qr + f * 32), kv[f], s, 0, 0, 0);
      }
    }
    bool see[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      see[e] = j <= at[e] && at[e] - j < p.window;
      s[e] *= p.scale;
      float top = see[e] ? s[e] : -1e30f;
      top = fmaxf(top, dpp_f32<0xB1>(top));
      top = fmaxf(top, dpp_f32<0x4E>(top));
      top = fmaxf(top, dpp_f32<0x141>(top));
      top = fmaxf(top, dpp_f32<0x140>(top));
      if (col == 0) red[0][wave][quad * 4 + e] = top;
    }
    __syncthreads();  // the previous tile's Vt and Ps have been read, the maxima are there
#pragma unroll
    for (int f = 0; f < 2 * NT; ++f) {
      if (f * 32 < p.ldc) {
#pragma unroll
        for (int b = 0; b < 8; ++b) Vt[(f * 32 + quad * 8 + b) * LDV + wave * 16 + col] = kv[f][b];
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = quad * 4 + e;
      const float now = fmaxf(m[e], fmaxf(fmaxf(red[0][0][r], red[0][1][r]), fmaxf(red[0][2][r], red[0][3][r])));
      const float shrink = __expf(m[e] - now), pr = see[e] ? __expf(s[e] - now) : 0.0f;
      m[e] = now;
      l[e] *= shrink;
#pragma unroll
      for (int i = 0; i < NT; ++i) o[i][e] *= shrink;
      const bf16_t value = (bf16_t)pr;
      Ps[r * LDV + wave * 16 + col] = value;
      Ps[(LROWS + r) * LDV + wave * 16 + col] = (bf16_t)(pr - (float)value);
      const float sum = row16_sum(pr);
      if (col == 0) red[1][wave][r] = sum;
    }
    __syncthreads();
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = quad * 4 + e;
      l[e] += (red[1][0][r] + red[1][1][r]) + (red[1][2][r] + red[1][3][r]);
    }
#pragma unroll
    for (int k = 0; k < LKEYS; k += 32) {
      const bf16x8_t value = *reinterpret_cast<const bf16x8_t*>(Ps + col * LDV + k + quad * 8);
      const bf16x8_t rem = *reinterpret_cast<const bf16x8_t*>(Ps + (LROWS + col) * LDV + k + quad * 8);
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const int c0 = (i * 4 + wave) * 16;
        if (c0 < p.ldc) {
          const bf16x8_t b = *reinterpret_cast<const bf16x8_t*>(Vt + (c0 + col) * LDV + k + quad * 8);
          o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(rem, b, o[i], 0, 0, 0);
          o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(value, b, o[i], 0, 0, 0);
        }
      }
    }
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int r = quad * 4 + e;
    if (r0 + r >= rows) continue;
    float* dst = p.part + ((size_t)slice * rows + r0 + r) * p.ldc;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int c0 = (i * 4 + wave) * 16;
      if (c0 < p.ldc) dst[c0 + col] = o[i][e];
    }
    if (wave == 0 && col == 0) {
      ml[r * 2] = m[e];
      ml[r * 2 + 1] = l[e];
    }
  }
}

// out[t][h * dv + j] = sigmoid(gate) * (value matrix of head h . weighted latent of (t, h)): the slices are added up (with
// the sink in the denominator), then multiplied.  Workgroup: 64 value columns of one head, sixteen tokens.
struct latent_value_args {
  int heads, n, ldc, dv, slices;
  const float* part;
  const float* ml;
  const float* sink;     // [heads] or nullptr
  const bf16_t* w;       // [heads * dv][ldc]
  const bf16_t* gate;    // [n][ldg] or nullptr
  int ldg;
  bf16_t* out;
  int ldo;
};
constexpr int MAX_SLICES = 32;

template <int NT>
__global__ __launch_bounds__(256) void latent_value_kernel(latent_value_args p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char value_lds[];
  bf16_t* C = reinterpret_cast<bf16_t*>(value_lds);  // [16][ldc + 8]
  __shared__ float weight[16][MAX_SLICES];
  __shared__ int live[16];  // slices up to the last one with keys
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, quad = lane >> 4;
  const int h = blockIdx.x, t0 = blockIdx.z * 16, tokens = min(16, p.n - t0), rows = p.n * p.heads, ld = p.ldc + 8;
  const int j = blockIdx.y * 64 + wave * 16 + col;
  const bool multiplies = blockIdx.y * 64 + wave * 16 < p.dv;
  bf16x8_t w[2 * NT];
  const bf16_t* b = p.w + ((size_t)h * p.dv + (multiplies ? j : 0)) * p.ldc + quad * 8;
#pragma unroll
  for (int f = 0; f < 2 * NT; ++f) w[f] = f * 32 < p.ldc ? *reinterpret_cast<const bf16x8_t*>(b + f * 32) : (bf16x8_t)(0.0f);
  for (int t = wave; t < tokens; t += 4) {
    const int row = (t0 + t) * p.heads + h;
    const bool has = lane < p.slices;
    const float* src = p.ml + ((size_t)(has ? lane : 0) * rows + row) * 2;
    const float m = has ? src[0] : -1e30f, l = has ? src[1] : 0.0f;
    float top = wave_max_dpp(m);
    if (p.sink) top = fmaxf(top, p.sink[h]);
    const float f = l > 0.0f ? __expf(m - top) : 0.0f;
    float total = wave_sum(f * l);
    if (p.sink) total += __expf(p.sink[h] - top);
    if (has) weight[t][lane] = f / total;
    const uint64_t with_keys = __ballot(l > 0.0f);
    if (lane == 0) live[t] = 64 - __clzll(with_keys | 1);
  }
  __syncthreads();
  const int c4 = p.ldc / 4;
  for (int i = tid; i < 16 * c4; i += 256) {
    const int t = i / c4, c = (i - t * c4) * 4;
    float4_t v = (float4_t)(0.0f);
    if (t < tokens) {
      const float* src = p.part + ((size_t)(t0 + t) * p.heads + h) * p.ldc + c;
      const int n = live[t];  // those behind have written nothing
#pragma unroll 8
      for (int s = 0; s < n; ++s) v += weight[t][s] * load4(src + (size_t)s * rows * p.ldc);
    }
    store4(C + t * ld + c, v);
  }
  __syncthreads();
  if (!multiplies) return;
  const bf16_t* a = C + col * ld + quad * 8;
  float4_t acc = (float4_t)(0.0f);
#pragma unroll
  for (int f = 0; f < 2 * NT; ++f) {
    if (f * 32 < p.ldc) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(a + f * 32), w[f], acc, 0, 0, 0);
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int t = quad * 4 + e;
    if (t < tokens) {
      float v = acc[e];
      if (p.gate) v *= sigmoid_f32((float)p.gate[(size_t)(t0 + t) * p.ldg + (size_t)h * p.dv + j]);
      p.out[(size_t)(t0 + t) * p.ldo + (size_t)h * p.dv + j] = (bf16_t)v;
    }
  }
}

int check_latent(const char* who, const lcu_latent_params* p) {
  LCU_REQUIRE(p, "%s: null pointer", who);
  LCU_REQUIRE(p->heads > 0 && p->heads <= 4096 && p->dn > 0 && p->dn % 32 == 0 && p->dr >= 0 && p->dr % 32 == 0 && p->rot >= 0 &&
                  p->rot % 2 == 0 && p->rot <= p->dr && p->dv > 0 && p->dv % 32 == 0 && p->ldc > 0 && p->ldc % 64 == 0 && p->rank > 0 &&
                  p->rank <= p->ldc && p->window > 0,
              "%s: heads %d, head parts %d + %d (%d rotated), values %d, latent %d in %d, window %d", who, p->heads, p->dn, p->dr, p->rot,
              p->dv, p->rank, p->ldc, p->window);
  return LCU_OK;
}

int row_args(const char* who, const lcu_latent_rows_args* a, const lcu_latent_params* p, latent_row_args& r) {
  LCU_REQUIRE(a->rows_dev && a->latent_norm_dev && a->latents_dev && a->start_dev && (p->dr == 0 || (a->keys_dev && a->freq_dev)) &&
                  (a->low_rank == 0 || (a->low_norm_dev && a->low_dev)),
              "%s: null pointer", who);
  LCU_REQUIRE(a->n >= 0 && a->max_positions > 0 && a->n <= a->max_positions && a->ld >= a->latent_at + p->ldc &&
                  (p->dr == 0 || a->ld >= a->key_at + p->dr) && a->ld % 8 == 0 && a->latent_at % 8 == 0 && a->key_at % 8 == 0 &&
                  a->low_rank >= 0 && a->low_rank <= a->low_ld && a->low_ld % 4 == 0 && a->low_ld <= a->ld &&
                  (!a->rotate_queries || a->query_at + p->heads * (p->dn + p->dr) <= a->ld + p->dn),
              "%s: bad shape n %d of %d, row %d: latent at %d, key at %d, queries at %d, queries' latent %d in %d", who, a->n,
              a->max_positions, a->ld, a->latent_at, a->key_at, a->query_at, a->low_rank, a->low_ld);
  r = latent_row_args{a->rows_dev, a->ld, a->n, a->latent_at, p->rank, p->ldc, (const float*)a->latent_norm_dev, a->latents_dev,
                      a->key_at, p->rot, p->dr, a->keys_dev, a->query_at, a->rotate_queries ? p->heads : 0, p->dn + p->dr,
                      (const float*)a->freq_dev, a->gain, a->low_rank, a->low_ld, (const float*)a->low_norm_dev, a->low_dev,
                      (const int*)a->start_dev, a->max_positions, a->eps};
  return LCU_OK;
}

size_t attention_lds(int ldc, int dr) { return ((size_t)LROWS * (ldc + dr + 8) + (size_t)ldc * LDV + 2 * LROWS * LDV) * 2; }

}  // namespace

extern "C" {

int lcu_latent_rows(const lcu_latent_rows_args* rows, const lcu_latent_params* p, int dtype, void* stream) {
  LCU_REQUIRE(rows, "lcu_latent_rows: null pointer");
  int rc = check_latent("lcu_latent_rows", p);
  if (rc) return rc;
  LCU_REQUIRE(dtype == LCU_BF16 || dtype == LCU_F32, "lcu_latent_rows: element type %d", dtype);
  latent_row_args r{};
  rc = row_args("lcu_latent_rows", rows, p, r);
  if (rc || rows->n == 0) return rc;
  if (dtype == LCU_F32) {
    latent_rows_kernel<float><<<rows->n, 256, 0, as_stream(stream)>>>(r);
  } else {
    latent_rows_kernel<bf16_t><<<rows->n, 256, 0, as_stream(stream)>>>(r);
  }
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_latent_queries(void* out_dev, const void* q_dev, int ldq, const void* uk_t_dev, const lcu_latent_params* p,
                       const lcu_latent_rows_args* rows, int n, void* stream) {
  LCU_REQUIRE(out_dev && q_dev && uk_t_dev, "lcu_latent_queries: null pointer");
  int rc = check_latent("lcu_latent_queries", p);
  if (rc) return rc;
  LCU_REQUIRE(n >= 0 && n <= 4096 && ldq >= p->heads * (p->dn + p->dr) && ldq % 8 == 0, "lcu_latent_queries: bad shape n %d stride %d", n, ldq);
  latent_row_args r{};
  if (rows) {
    LCU_REQUIRE(rows->n == n, "lcu_latent_queries: %d rows for %d tokens", rows->n, n);
    rc = row_args("lcu_latent_queries", rows, p, r);
    if (rc) return rc;
  }
  if (n == 0) return LCU_OK;
  const int products = p->heads * (p->ldc / 64) * ((n + 15) / 16);
  head_products_kernel<<<products + (rows ? n : 0), 256, 0, as_stream(stream)>>>((bf16_t*)out_dev, p->heads * p->ldc, (const bf16_t*)q_dev,
                                                                               ldq, p->dn + p->dr, (const bf16_t*)uk_t_dev, p->ldc, p->dn, n,
                                                                               products, r);
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_latent_attention_fits(const lcu_latent_params* p) {
  return p != nullptr && p->ldc <= 512 && attention_lds(p->ldc, p->dr) <= 150 * 1024 ? 1 : 0;
}

int lcu_latent_slices(const lcu_latent_params* p, int n, int max_positions) {
  if (p == nullptr || n <= 0) return 1;
  const long most = std::min<long>((long)p->window + n, max_positions);  // keys of any sixteen rows
  const long row_tiles = ((long)n * p->heads + LROWS - 1) / LROWS;
  const long room = std::max<long>(1, 512 / row_tiles);
  return (int)std::min<long>(std::min<long>((most + LKEYS - 1) / LKEYS, room), MAX_SLICES);
}

size_t lcu_latent_attention_scratch(const lcu_latent_params* p, int n, int max_positions) {
  return p == nullptr ? 0 : (size_t)lcu_latent_slices(p, n, max_positions) * n * p->heads * (p->ldc + 2) * sizeof(float);
}

int lcu_latent_attention(void* out_dev, int ldo, const void* q_latent_dev, const void* q_rot_dev, int ldq, const void* latents_dev,
                         const void* keys_dev, const void* start_dev, int max_positions, const void* uv_dev, const void* sink_dev,
                         const void* gate_dev, int ldg, const lcu_latent_params* p, void* scratch_dev, int n, void* stream) {
  LCU_REQUIRE(out_dev && q_latent_dev && latents_dev && start_dev && uv_dev && scratch_dev, "lcu_latent_attention: null pointer");
  const int rc = check_latent("lcu_latent_attention", p);
  if (rc) return rc;
  LCU_REQUIRE(p->dr == 0 || (q_rot_dev && keys_dev && ldq % 8 == 0), "lcu_latent_attention: no rotated part (stride %d)", ldq);
  LCU_REQUIRE(n > 0 && n <= 4096 && n <= max_positions && ldo >= p->heads * p->dv && (!gate_dev || ldg >= p->heads * p->dv),
              "lcu_latent_attention: bad shape n %d of %d, strides %d %d", n, max_positions, ldo, ldg);
  LCU_REQUIRE(lcu_latent_attention_fits(p), "lcu_latent_attention: latent %d with rotated part %d", p->ldc, p->dr);
  const int slices = lcu_latent_slices(p, n, max_positions), rows = n * p->heads;
  float* part = (float*)scratch_dev;
  float* ml = part + (size_t)slices * rows * p->ldc;
  const latent_args a{p->heads, n, p->ldc, p->dr, p->window, slices, p->scale, (const bf16_t*)q_latent_dev, (const bf16_t*)q_rot_dev, ldq,
                      p->dn + p->dr, (const bf16_t*)latents_dev, (const bf16_t*)keys_dev, (const int*)start_dev, max_positions, part, ml};
  hipStream_t st = as_stream(stream);
  const size_t lds = attention_lds(p->ldc, p->dr);
  const latent_value_args v{p->heads, n, p->ldc, p->dv, slices, part, ml, (const float*)sink_dev, (const bf16_t*)uv_dev,
                            (const bf16_t*)gate_dev, ldg, (bf16_t*)out_dev, ldo};
  const auto go = [&](auto nt) -> int {
    auto kernel = latent_attention_kernel<decltype(nt)::value>;
    static bool raised[16] = {};  // per device, once
    int dev = 0;
    LCU_HIP(hipGetDevice(&dev));
    if (!raised[dev & 15]) {
      LCU_HIP(hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024));
      raised[dev & 15] = true;
    }
    kernel<<<dim3((rows + LROWS - 1) / LROWS, slices), 256, lds, st>>>(a);
    latent_value_kernel<decltype(nt)::value>
        <<<dim3(p->heads, (p->dv + 63) / 64, (n + 15) / 16), 256, (size_t)16 * (p->ldc + 8) * 2, st>>>(v);
    LCU_LAUNCH_CHECK();
    return LCU_OK;
  };
  using std::integral_constant;
  return p->ldc <= 64    ? go(integral_constant<int, 1>{})
         : p->ldc <= 128 ? go(integral_constant<int, 2>{})
         : p->ldc <= 256 ? go(integral_constant<int, 4>{})
                         : go(integral_constant<int, 8>{});
}

}  // extern "C"
