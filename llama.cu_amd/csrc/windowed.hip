// Attention over a key/value cache with a sliding window, kept first tokens, grouped heads and a
// per-head distance bias:
//   score(i, j) = scale q_i.k_j - r1 ln(1 + r2 (i - j)),  visible when j <= i and (i - j < window or j < keep)
// followed by a softmax, whose denominator may hold one more term per head, exp(sink).  Scores, softmax and weighted
// sums are fp32.  The last columns of a key may come from an array that all heads share, and the result may be
// multiplied with the sigmoid of a gate (neither in the one-token kernel).
//
// Layouts: q rows of heads x dk inside rows of ldq elements; caches k [positions][kv_heads * dk] and
// v [positions][kv_heads * dv].  dk is the head size padded to a multiple of 32, dv the value size padded
// to 32, 64, 128 or 256; the padding holds zeros.  A head's visible keys are the first ones, [0, kept), and
// the window [lo, i]: every kernel walks exactly these.
#include <algorithm>
#include <type_traits>

#include "linear.hpp"
#include "rownorm.hpp"

using namespace lcu;

namespace {

struct window_args {
  int heads, kv_heads, dk, dv, ldq, ldo;
  int window, keep;
  float scale;
  const float* r1;     // NULL: no distance bias
  const float* r2;
  int k_ld, v_ld;      // elements from position to position
  int base;            // position of the first row of k, v and k_shared
  int dk_shared;       // the last dk_shared columns of a key are k_shared [position][dk_shared]
  const void* k_shared;
  const float* sink;   // [heads] or NULL
  const void* gate;    // [row][ldg], heads x dv, or NULL
  int ldg;
};

// first key of the window of position i, and how many kept keys lie below it
__device__ __forceinline__ int window_begin(const window_args& p, int i) { return max(0, i - p.window + 1); }

// ---- new rows of the caches -----------------------------------------------------------------------------
// Row t of qkv holds q | k | v.  k goes to cache row start + t; v too, after mixing with the row of
// v_first when MIX_WITH: (1 - lambda) v + lambda v_first; KEEP_AS_FIRST leaves the projected v in v_first.
enum v_mode { V_PLAIN = 0, V_KEEP_AS_FIRST = 1, V_MIX_WITH_FIRST = 2 };

// four columns per thread (column counts are multiples of 32)
template <class T>
__global__ __launch_bounds__(256) void kv_store_kernel(T* __restrict__ k_cache, T* __restrict__ v_cache, const T* __restrict__ qkv,
                                                       int ldq, int q_cols, int k_cols, int v_cols, T* __restrict__ v_first,
                                                       int mode, const float* __restrict__ lambda, const int* __restrict__ start,
                                                       int max_pos, int n) {
  const int per = (k_cols + v_cols) / 4, i = blockIdx.x * 256 + threadIdx.x;
  if (i >= n * per) return;
  const int t = i / per, c = (i - t * per) * 4;
  const size_t pos = min(max(*start + t, 0), max_pos - 1);
  float4_t v = load4(qkv + (size_t)t * ldq + q_cols + c);
  if (c < k_cols) {
    store4(k_cache + pos * k_cols + c, v);
    return;
  }
  const int vc = c - k_cols;
  T* first = v_first + (size_t)t * v_cols + vc;
  if (mode == V_KEEP_AS_FIRST) store4(first, v);
  if (mode == V_MIX_WITH_FIRST) {
    const float l = *lambda;
    const float4_t f = load4(first);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = (1.0f - l) * v[e] + l * f[e];
  }
  store4(v_cache + pos * v_cols + vc, v);
}

// ---- one workgroup per (query row, head), plain fp32 arithmetic: the fp32 element type -----------------
template <class T>
__global__ __launch_bounds__(256) void attention_row_kernel(T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ k,
                                                            const T* __restrict__ v, int start, window_args p) {
  extern __shared__ float sc[];  // scores of the visible keys
  __shared__ float red[4];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int t = blockIdx.x, h = blockIdx.y, g = h / (p.heads / p.kv_heads), i = start + t;
  const int lo = window_begin(p, i), kept = min(p.keep, lo), n_keys = kept + i - lo + 1, own = p.dk - p.dk_shared;
  const T* qr = q + (size_t)t * p.ldq + (size_t)h * p.dk;
  const float r1 = p.r1 ? p.r1[h] : 0.0f, r2 = p.r1 ? p.r2[h] : 0.0f;
  float m = p.sink ? p.sink[h] : -INFINITY;
  for (int x = wave; x < n_keys; x += 4) {
    const int j = x < kept ? x : lo + x - kept;
    const T* kr = k + (size_t)(j - p.base) * p.k_ld + (size_t)g * own;
    const T* ks = (const T*)p.k_shared + (size_t)(j - p.base) * p.dk_shared;
    float s = 0.0f;
    for (int c = lane; c < p.dk; c += WAVE) s = fmaf(to_f32(qr[c]), to_f32(c < own ? kr[c] : ks[c - own]), s);
    s = wave_sum(s) * p.scale - r1 * log1pf(r2 * (float)(i - j));
    if (lane == 0) sc[x] = s;
    m = fmaxf(m, s);
  }
  if (lane == 0) red[wave] = m;
  __syncthreads();
  m = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
  __syncthreads();
  float l = 0.0f;
  for (int x = tid; x < n_keys; x += 256) {
    const float e = expf(sc[x] - m);
    sc[x] = e;
    l += e;
  }
  l = wave_sum(l);
  if (lane == 0) red[wave] = l;
  __syncthreads();
  l = (red[0] + red[1]) + (red[2] + red[3]);
  if (p.sink) l += expf(p.sink[h] - m);
  for (int c = tid; c < p.dv; c += 256) {
    float o = 0.0f;
    for (int x = 0; x < n_keys; ++x) {
      const int j = x < kept ? x : lo + x - kept;
      o = fmaf(sc[x], to_f32(v[(size_t)(j - p.base) * p.v_ld + (size_t)g * p.dv + c]), o);
    }
    o /= l;
    if (p.gate) o *= sigmoid_f32(to_f32(((const T*)p.gate)[(size_t)t * p.ldg + (size_t)h * p.dv + c]));
    out[(size_t)t * p.ldo + (size_t)h * p.dv + c] = (T)o;
  }
}

// ---- prompts, bfloat16: matrix cores --------------------------------------------------------------------
// One workgroup: 64 query rows of one head, 16 per wavefront, against tiles of 64 keys with a running
// maximum and sum.  Key tiles that hold no visible key of any of the rows (between the kept tokens and the
// windows) are not visited; the next tile is asked for while one is worked on.  Scores are computed with the keys as
// rows, so that a lane holds sixteen of its own query row, which are the second operand of the product with the
// transposed values as they are: keys of a block of 32 lie in LDS in the order in which lanes hold them.  Probabilities go
// in as two bfloat16 terms (value and remainder), so that they keep 16 significant bits.  Workgroups of a head differ in id
// by the number of heads: where that is a multiple of eight they share an L2, and long rows come first.
constexpr int QT = 64, KT = 64;

// where key r of a tile lies in a row of transposed values
__device__ __forceinline__ int key_place(int r) { return (r & ~31) + ((r >> 2) & 3) * 8 + ((r >> 4) & 1) * 4 + (r & 3); }

template <int DV, bool BIAS>
__global__ __launch_bounds__(256) void attention_tile_kernel(bf16_t* __restrict__ out, const bf16_t* __restrict__ q,
                                                             const bf16_t* __restrict__ k, const bf16_t* __restrict__ v, int n,
                                                             int start, window_args p) {
  constexpr int NT = DV / 16, LDP = KT + 8, KP = 8, VP = (DV + 63) / 64;  // KP, VP: pieces of a tile per thread
  extern __shared__ __attribute__((aligned(16))) unsigned char attn_lds[];
  const int ldk = p.dk + 8;
  bf16_t* Ks = reinterpret_cast<bf16_t*>(attn_lds);   // [KT][ldk]
  bf16_t* Vt = Ks + KT * ldk;                         // [DV][LDP]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, quad = lane >> 4;
  const int h = blockIdx.x % p.heads, q0 = ((int)gridDim.x / p.heads - 1 - (int)blockIdx.x / p.heads) * QT;
  const int g = h / (p.heads / p.kv_heads), dk8 = p.dk / 8, own8 = (p.dk - p.dk_shared) / 8;
  const float r1 = BIAS ? p.r1[h] : 0.0f, r2 = BIAS ? p.r2[h] : 0.0f;
  const int first = start + q0, last = start + min(q0 + QT, n) - 1;  // positions of the tile's rows
  const int win_tile = window_begin(p, first) / KT, kept_tiles = (min(p.keep, first + QT) + KT - 1) / KT;
  uint4_t kr[KP], vr[VP][2];
  int k_at[KP];  // row and piece of the keys
#pragma unroll
  for (int x = 0; x < KP; ++x) {
    const int c = tid + x * 256;
    k_at[x] = c < KT * dk8 ? c / dk8 << 8 | c % dk8 : -1;
  }
  const auto fetch = [&](int kt) {
#pragma unroll
    for (int x = 0; x < KP; ++x) {
      if (k_at[x] < 0) continue;
      const int e = k_at[x] & 255;
      const size_t row = max(min(kt * KT + (k_at[x] >> 8), last) - p.base, 0);
      kr[x] = *reinterpret_cast<const uint4_t*>(e < own8 ? k + row * p.k_ld + ((size_t)g * own8 + e) * 8
                                                         : (const bf16_t*)p.k_shared + row * p.dk_shared + (e - own8) * 8);
    }
#pragma unroll
    for (int x = 0; x < VP; ++x) {
      const int c = tid + x * 256, r = (c & 31) * 2, e = (c >> 5) * 8;
      if (e >= DV) continue;
#pragma unroll
      for (int y = 0; y < 2; ++y) {
        const size_t row = max(min(kt * KT + r + y, last) - p.base, 0);
        vr[x][y] = *reinterpret_cast<const uint4_t*>(v + row * p.v_ld + (size_t)g * DV + e);
      }
    }
  };
  int kt = kept_tiles > 0 ? 0 : win_tile;
  fetch(kt);
  bf16x8_t qf[KP];
#pragma unroll
  for (int c = 0; c < KP; ++c) {
    if (c * 32 >= p.dk) continue;
    qf[c] = *reinterpret_cast<const bf16x8_t*>(q + (size_t)min(q0 + wave * 16 + col, n - 1) * p.ldq + (size_t)h * p.dk + c * 32 + quad * 8);
  }
  const int i = first + wave * 16 + col;             // position of this lane's row
  float m = p.sink ? p.sink[h] : -1e30f;             // the sink counts as a key of value zero
  float l = p.sink && quad == 0 ? 1.0f : 0.0f;       // of this lane's keys
  float4_t o[NT];                                    // values t * 16 + quad * 4 .. + 3 of the row
#pragma unroll
  for (int t = 0; t < NT; ++t) o[t] = (float4_t)(0.0f);

  while (kt * KT <= last) {
    const int k0 = kt * KT;
    __syncthreads();  // the previous tile has been read
#pragma unroll
    for (int x = 0; x < KP; ++x) {
      if (k_at[x] >= 0) *reinterpret_cast<uint4_t*>(Ks + (k_at[x] >> 8) * ldk + (k_at[x] & 255) * 8) = kr[x];
    }
#pragma unroll
    for (int x = 0; x < VP; ++x) {
      const int c = tid + x * 256, at = key_place((c & 31) * 2), e = (c >> 5) * 8;
      if (e >= DV) continue;
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        const uint32_t a = vr[x][0][w], b = vr[x][1][w];
        *reinterpret_cast<uint32_t*>(Vt + (e + 2 * w) * LDP + at) = (a & 0xFFFFu) | b << 16;
        *reinterpret_cast<uint32_t*>(Vt + (e + 2 * w + 1) * LDP + at) = a >> 16 | (b & 0xFFFF0000u);
      }
    }
    __syncthreads();
    ++kt;
    if (kt >= kept_tiles && kt < win_tile) kt = win_tile;
    if (kt * KT <= last) fetch(kt);
    float4_t s[4];  // element e of s[t]: key t * 16 + quad * 4 + e
#pragma unroll
    for (int t = 0; t < 4; ++t) s[t] = (float4_t)(0.0f);
#pragma unroll
    for (int c = 0; c < KP; ++c) {
      if (c * 32 >= p.dk) continue;
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            *reinterpret_cast<const bf16x8_t*>(Ks + (t * 16 + col) * ldk + c * 32 + quad * 8), qf[c], s[t], 0, 0, 0);
      }
    }
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      s[t] *= p.scale;
      if constexpr (BIAS) {
#pragma unroll
        for (int e = 0; e < 4; ++e) s[t][e] -= r1 * __logf(1.0f + r2 * (float)max(i - (k0 + t * 16 + quad * 4 + e), 0));
      }
    }
    const int lowest = first + wave * 16;  // of the wavefront's positions
    if (k0 + KT - 1 > lowest || (lowest + 15 - k0 >= p.window && k0 + KT > p.keep)) {
#pragma unroll
      for (int t = 0; t < 4; ++t) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int j = k0 + t * 16 + quad * 4 + e, d = i - j;
          if (!(d >= 0 && (d < p.window || j < p.keep))) s[t][e] = -INFINITY;
        }
      }
    }
    float top = m;
#pragma unroll
    for (int t = 0; t < 4; ++t) top = fmaxf(top, fmaxf(fmaxf(s[t][0], s[t][1]), fmaxf(s[t][2], s[t][3])));
    top = fmaxf(top, __shfl_xor(top, 16, WAVE));
    top = fmaxf(top, __shfl_xor(top, 32, WAVE));
    if (__ballot(top != m) != 0) {
      const float shrink = __expf(m - top);
      m = top;
      l *= shrink;
#pragma unroll
      for (int t = 0; t < NT; ++t) o[t] *= shrink;
    }
#pragma unroll
    for (int c = 0; c < KT / 32; ++c) {
      bf16x8_t hi, rem;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float pr = __expf(s[c * 2 + e / 4][e % 4] - m);
        l += pr;
        hi[e] = (bf16_t)pr;
        rem[e] = (bf16_t)(pr - (float)hi[e]);
      }
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const bf16x8_t a = *reinterpret_cast<const bf16x8_t*>(Vt + (t * 16 + col) * LDP + c * 32 + quad * 8);
        o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, rem, o[t], 0, 0, 0);
        o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, hi, o[t], 0, 0, 0);
      }
    }
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  const int r = q0 + wave * 16 + col;
  if (r < n) {
    const float inv = 1.0f / l;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const size_t c = (size_t)h * DV + t * 16 + quad * 4;
      float4_t x = o[t] * inv;
      if (p.gate) {
        const float4_t z = load4((const bf16_t*)p.gate + (size_t)r * p.ldg + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] *= sigmoid_f32(z[e]);
      }
      store4(out + (size_t)r * p.ldo + c, x);
    }
  }
}

size_t tile_lds(int dk, int dv) { return ((size_t)KT * (dk + 8) + (size_t)dv * (KT + 8)) * 2; }

template <int DV, bool BIAS>
int launch_tiles(void* out, const void* q, const void* k, const void* v, int n, int start, const window_args& p, hipStream_t st) {
  const size_t lds = tile_lds(p.dk, DV);
  LCU_REQUIRE(lds <= 160 * 1024, "lcu_attention_windowed: head size %d with value size %d", p.dk, DV);
  auto kernel = attention_tile_kernel<DV, BIAS>;
  static bool raised[16] = {};  // per device, once
  int dev = 0;
  LCU_HIP(hipGetDevice(&dev));
  if (!raised[dev & 15]) {
    LCU_HIP(hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));
    raised[dev & 15] = true;
  }
  kernel<<<(unsigned)((n + QT - 1) / QT) * p.heads, 256, lds, st>>>((bf16_t*)out, (const bf16_t*)q, (const bf16_t*)k, (const bf16_t*)v, n,
                                                              start, p);
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

// ---- one new token, bfloat16 ----------------------------------------------------------------------------
// Workgroup (kv head, slice of the visible keys): 16 lanes share a key, eight columns each (DKP / DVP passes of
// 128 columns), and score it for every query head of the group, so that a cache row is read once for all of
// them; keys and values of DEC_FLIGHT rows per lane group are requested together, before anything is
// computed.  Each of the 16 groups keeps a running maximum, sum and weighted values per head; the groups
// meet in LDS, the slice's result goes to part[kv head][slice][head][dv + 4] (values, maximum, sum), and the
// last workgroup of a kv head to arrive adds the slices up: a counter says which it is, and that workgroup sets
// it back to zero.  Nobody waits.
constexpr int DEC_FLIGHT = 4;
constexpr int DEC_MAX_SLICES = 64, DEC_TOGETHER = 16;  // slices; those whose results are asked for together
constexpr int DEC_MAX_GROUP = 16;  // query heads per kv head

template <int RMAX, int DKP, int DVP>
__global__ __launch_bounds__(256) void attention_decode_kernel(bf16_t* __restrict__ out, const bf16_t* __restrict__ q,
                                                               const bf16_t* __restrict__ k, const bf16_t* __restrict__ v,
                                                               const int* __restrict__ pos_dev, int max_pos,
                                                               float* __restrict__ part, uint32_t* __restrict__ arrived,
                                                               window_args p) {
  extern __shared__ __attribute__((aligned(16))) float dec_lds[];  // [16 groups][R][dv], then [16][R][2]
  __shared__ bool last;
  const int R = p.heads / p.kv_heads;
  const int tid = threadIdx.x, sub = tid & 15, grp = tid >> 4;
  const int g = blockIdx.x, slice = blockIdx.y, slices = gridDim.y;
  const int i = min(max(*pos_dev, 0), max_pos - 1);
  const int lo = window_begin(p, i), kept = min(p.keep, lo), n_keys = kept + i - lo + 1;
  const int per = (n_keys + slices - 1) / slices;
  const int x0 = slice * per, x1 = min(x0 + per, n_keys);
  const bool k_lane[2] = {sub * 8 < p.dk, 128 + sub * 8 < p.dk}, v_lane[2] = {sub * 8 < p.dv, 128 + sub * 8 < p.dv};
  bf16x8_t qv[RMAX][DKP];
#pragma unroll
  for (int r = 0; r < RMAX; ++r) {
#pragma unroll
    for (int d = 0; d < DKP; ++d) {
      qv[r][d] = r < R && k_lane[d] ? *reinterpret_cast<const bf16x8_t*>(q + ((size_t)g * R + r) * p.dk + d * 128 + sub * 8) : (bf16x8_t)(0.0f);
    }
  }
  float m[RMAX], l[RMAX], o[RMAX][DVP][8], r1[RMAX], r2[RMAX];
#pragma unroll
  for (int r = 0; r < RMAX; ++r) {
    m[r] = -1e30f;
    l[r] = 0.0f;
    r1[r] = p.r1[g * R + min(r, R - 1)];
    r2[r] = p.r2[g * R + min(r, R - 1)];
#pragma unroll
    for (int d = 0; d < DVP; ++d) {
#pragma unroll
      for (int e = 0; e < 8; ++e) o[r][d][e] = 0.0f;
    }
  }
  for (int xb = x0; xb < x1; xb += 16 * DEC_FLIGHT) {
    bf16x8_t kv[DEC_FLIGHT][DKP], vv[DEC_FLIGHT][DVP];
    int j[DEC_FLIGHT];
#pragma unroll
    for (int f = 0; f < DEC_FLIGHT; ++f) {
      const int x = min(xb + f * 16 + grp, x1 - 1);
      j[f] = x < kept ? x : lo + x - kept;
      const bf16_t* kr = k + ((size_t)j[f] * p.kv_heads + g) * p.dk + sub * 8;
#pragma unroll
      for (int d = 0; d < DKP; ++d) kv[f][d] = k_lane[d] ? *reinterpret_cast<const bf16x8_t*>(kr + d * 128) : (bf16x8_t)(0.0f);
    }
#pragma unroll
    for (int f = 0; f < DEC_FLIGHT; ++f) {
      const bf16_t* vr = v + ((size_t)j[f] * p.kv_heads + g) * p.dv + sub * 8;
#pragma unroll
      for (int d = 0; d < DVP; ++d) vv[f][d] = v_lane[d] ? *reinterpret_cast<const bf16x8_t*>(vr + d * 128) : (bf16x8_t)(0.0f);
    }
#pragma unroll
    for (int r = 0; r < RMAX; ++r) {
      if (r < R) {
        float s[DEC_FLIGHT], top = m[r];
#pragma unroll
        for (int f = 0; f < DEC_FLIGHT; ++f) {
          float d0 = 0.0f;
#pragma unroll
          for (int d = 0; d < DKP; ++d) {
#pragma unroll
            for (int e = 0; e < 8; ++e) d0 = fmaf((float)qv[r][d][e], (float)kv[f][d][e], d0);
          }
          s[f] = row16_sum(d0) * p.scale - r1[r] * __logf(1.0f + r2[r] * (float)(i - j[f]));
          if (xb + f * 16 + grp < x1) top = fmaxf(top, s[f]);
        }
        const float shrink = __expf(m[r] - top);
        m[r] = top;
        l[r] *= shrink;
#pragma unroll
        for (int d = 0; d < DVP; ++d) {
#pragma unroll
          for (int e = 0; e < 8; ++e) o[r][d][e] *= shrink;
        }
#pragma unroll
        for (int f = 0; f < DEC_FLIGHT; ++f) {
          const float w = xb + f * 16 + grp < x1 ? __expf(s[f] - top) : 0.0f;
          l[r] += w;
#pragma unroll
          for (int d = 0; d < DVP; ++d) {
#pragma unroll
            for (int e = 0; e < 8; ++e) o[r][d][e] = fmaf(w, (float)vv[f][d][e], o[r][d][e]);
          }
        }
      }
    }
  }
  float* ml = dec_lds + 16 * R * p.dv;
#pragma unroll
  for (int r = 0; r < RMAX; ++r) {
    if (r < R) {
#pragma unroll
      for (int d = 0; d < DVP; ++d) {
        if (v_lane[d]) {
          float* dst = dec_lds + ((size_t)grp * R + r) * p.dv + d * 128 + sub * 8;
          store4(dst, (float4_t){o[r][d][0], o[r][d][1], o[r][d][2], o[r][d][3]});
          store4(dst + 4, (float4_t){o[r][d][4], o[r][d][5], o[r][d][6], o[r][d][7]});
        }
      }
      if (sub == 0) {
        ml[(grp * R + r) * 2] = m[r];
        ml[(grp * R + r) * 2 + 1] = l[r];
      }
    }
  }
  __syncthreads();
  const int ldp = p.dv + 4;
  float* pg = part + (size_t)(g * slices + slice) * R * ldp;
  for (int c = tid; c < R * p.dv; c += 256) {
    const int r = c / p.dv, e = c - r * p.dv;
    float mx = -1e30f;
#pragma unroll
    for (int w = 0; w < 16; ++w) mx = fmaxf(mx, ml[(w * R + r) * 2]);
    float sum = 0.0f, val = 0.0f;
#pragma unroll
    for (int w = 0; w < 16; ++w) {
      const float f = __expf(ml[(w * R + r) * 2] - mx);
      sum = fmaf(f, ml[(w * R + r) * 2 + 1], sum);
      val = fmaf(f, dec_lds[((size_t)w * R + r) * p.dv + e], val);
    }
    __hip_atomic_store(pg + r * ldp + e, val, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    if (e == 0) {
      __hip_atomic_store(pg + r * ldp + p.dv, mx, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      __hip_atomic_store(pg + r * ldp + p.dv + 1, sum, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // every wavefront's stores are out before the count goes up
  __syncthreads();
  if (tid == 0) {
    last = __hip_atomic_fetch_add(arrived + g, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == (uint32_t)slices - 1;
    if (last) __hip_atomic_store(arrived + g, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
  __syncthreads();
  if (!last) return;
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");  // ordinary loads from here on see the other workgroups' stores
  const float* all = part + (size_t)g * slices * R * ldp;
  const int quads = p.dv / 4;
  for (int c = tid; c < R * quads; c += 256) {
    const int r = c / quads, e = (c - r * quads) * 4;
    float mx = -1e30f, sum = 0.0f;
    float4_t val = (float4_t)(0.0f);
    for (int s0 = 0; s0 < slices; s0 += DEC_TOGETHER) {
      float4_t pv[DEC_TOGETHER];
      float pm[DEC_TOGETHER], pl[DEC_TOGETHER];
#pragma unroll
      for (int b = 0; b < DEC_TOGETHER; ++b) {
        const float* src = all + ((size_t)min(s0 + b, slices - 1) * R + r) * ldp;
        pv[b] = load4(src + e);
        pm[b] = src[p.dv];
        pl[b] = src[p.dv + 1];
      }
#pragma unroll
      for (int b = 0; b < DEC_TOGETHER; ++b) {
        if (s0 + b < slices) {
          const float now = fmaxf(mx, pm[b]), was = __expf(mx - now), f = __expf(pm[b] - now);
          sum = sum * was + f * pl[b];
          val = val * was + f * pv[b];
          mx = now;
        }
      }
    }
    store4(out + ((size_t)g * R + r) * p.dv + e, val * (1.0f / sum));
  }
}

template <int DKP, int DVP>
int launch_decode(bf16_t* out, const bf16_t* q, const bf16_t* k, const bf16_t* v, const int* pos, int max_pos, float* part,
                  uint32_t* arrived, const window_args& p, int slices, hipStream_t st) {
  const int R = p.heads / p.kv_heads;
  const size_t lds = (size_t)16 * R * (p.dv + 2) * sizeof(float);
  const auto go = [&](auto rmax) -> int {
    auto kernel = attention_decode_kernel<decltype(rmax)::value, DKP, DVP>;
    if (lds > 64 * 1024) {
      static bool raised[16] = {};  // per device, once
      int dev = 0;
      LCU_HIP(hipGetDevice(&dev));
      if (!raised[dev & 15]) {
        LCU_HIP(hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024));
        raised[dev & 15] = true;
      }
    }
    kernel<<<dim3(p.kv_heads, slices), 256, lds, st>>>(out, q, k, v, pos, max_pos, part, arrived, p);
    LCU_LAUNCH_CHECK();
    return LCU_OK;
  };
  if (R <= 1) return go(std::integral_constant<int, 1>{});
  if (R <= 4) return go(std::integral_constant<int, 4>{});
  if (R <= 8) return go(std::integral_constant<int, 8>{});
  return go(std::integral_constant<int, DEC_MAX_GROUP>{});
}

int check_window(const char* who, const lcu_window_params* w, int dtype) {
  LCU_REQUIRE(w && (!w->r1_dev || w->r2_dev), "%s: null pointer", who);
  LCU_REQUIRE(dtype == LCU_BF16 || dtype == LCU_F32, "%s: element type %d", who, dtype);
  LCU_REQUIRE(w->heads > 0 && w->kv_heads > 0 && w->heads % w->kv_heads == 0 && w->dk > 0 && w->dk % 32 == 0 && w->dk <= 256 &&
                  (w->dv == 32 || w->dv == 64 || w->dv == 128 || w->dv == 256),
              "%s: heads %d / %d, head size %d (a multiple of 32, at most 256), value size %d (32, 64, 128, 256)", who, w->heads,
              w->kv_heads, w->dk, w->dv);
  LCU_REQUIRE(w->window > 0 && w->keep >= 0 && w->heads <= 65535, "%s: window %d keep %d", who, w->window, w->keep);
  LCU_REQUIRE(w->dk_shared >= 0 && w->dk_shared % 8 == 0 && w->dk_shared < w->dk && (w->dk_shared == 0 || w->k_shared_dev),
              "%s: %d shared columns of a key of %d", who, w->dk_shared, w->dk);
  LCU_REQUIRE((w->k_ld == 0 || (w->k_ld >= w->kv_heads * (w->dk - w->dk_shared) && w->k_ld % 8 == 0)) &&
                  (w->v_ld == 0 || (w->v_ld >= w->kv_heads * w->dv && w->v_ld % 8 == 0)),
              "%s: position strides %d %d", who, w->k_ld, w->v_ld);
  LCU_REQUIRE(!w->gate_dev || w->ldg >= w->heads * w->dv, "%s: gate rows of %d", who, w->ldg);
  return LCU_OK;
}

window_args make_window(const lcu_window_params* w, int ldq, int ldo) {
  return window_args{w->heads,
                     w->kv_heads,
                     w->dk,
                     w->dv,
                     ldq,
                     ldo,
                     w->window,
                     w->keep,
                     w->scale,
                     (const float*)w->r1_dev,
                     (const float*)w->r2_dev,
                     w->k_ld ? w->k_ld : w->kv_heads * (w->dk - w->dk_shared),
                     w->v_ld ? w->v_ld : w->kv_heads * w->dv,
                     w->first_position,
                     w->dk_shared,
                     w->k_shared_dev,
                     (const float*)w->sink_dev,
                     w->gate_dev,
                     w->ldg};
}

}  // namespace

extern "C" {

int lcu_kv_store(void* k_cache_dev, void* v_cache_dev, const void* qkv_dev, int ldq, int q_cols, int k_cols, int v_cols,
                 void* v_first_dev, int v_mode, const void* lambda_dev, const void* start_dev, int max_positions, int dtype, int n,
                 void* stream) {
  LCU_REQUIRE(k_cache_dev && v_cache_dev && qkv_dev && start_dev && (v_mode == V_PLAIN || v_first_dev) &&
                  (v_mode != V_MIX_WITH_FIRST || lambda_dev),
              "lcu_kv_store: null pointer");
  LCU_REQUIRE(v_mode >= 0 && v_mode <= 2 && n >= 0 && n <= max_positions && n <= 65535 && k_cols > 0 && v_cols > 0 &&
                  ldq >= q_cols + k_cols + v_cols && (dtype == LCU_BF16 || dtype == LCU_F32),
              "lcu_kv_store: bad shape n %d of %d, columns %d %d %d of %d", n, max_positions, q_cols, k_cols, v_cols, ldq);
  if (n == 0) return LCU_OK;
  LCU_REQUIRE(k_cols % 4 == 0 && v_cols % 4 == 0 && q_cols % 4 == 0 && ldq % 4 == 0, "lcu_kv_store: columns in groups of four");
  const unsigned grid = (unsigned)(((size_t)n * ((k_cols + v_cols) / 4) + 255) / 256);
  hipStream_t st = as_stream(stream);
  if (dtype == LCU_F32) {
    kv_store_kernel<float><<<grid, 256, 0, st>>>((float*)k_cache_dev, (float*)v_cache_dev, (const float*)qkv_dev, ldq, q_cols, k_cols,
                                                 v_cols, (float*)v_first_dev, v_mode, (const float*)lambda_dev,
                                                 (const int*)start_dev, max_positions, n);
  } else {
    kv_store_kernel<bf16_t><<<grid, 256, 0, st>>>((bf16_t*)k_cache_dev, (bf16_t*)v_cache_dev, (const bf16_t*)qkv_dev, ldq, q_cols,
                                                  k_cols, v_cols, (bf16_t*)v_first_dev, v_mode, (const float*)lambda_dev,
                                                  (const int*)start_dev, max_positions, n);
  }
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_attention_windowed(void* out_dev, int ldo, const void* q_dev, int ldq, const void* k_cache_dev, const void* v_cache_dev,
                           int start, const lcu_window_params* window, int dtype, int n, void* stream) {
  LCU_REQUIRE(out_dev && q_dev && k_cache_dev && v_cache_dev, "lcu_attention_windowed: null pointer");
  const int rc = check_window("lcu_attention_windowed", window, dtype);
  if (rc) return rc;
  LCU_REQUIRE(n >= 0 && start >= 0 && ldq >= window->heads * window->dk && ldo >= window->heads * window->dv && ldq % 8 == 0,
              "lcu_attention_windowed: bad shape n %d start %d strides %d %d", n, start, ldq, ldo);
  LCU_REQUIRE(window->first_position >= 0 &&
                  (window->first_position == 0 ||
                   (window->keep == 0 && (long)window->first_position <= std::max(0L, (long)start - window->window + 1))),
              "lcu_attention_windowed: keys from position %d on do not hold the window of position %d", window->first_position, start);
  LCU_REQUIRE(ldo % 4 == 0 && (!window->gate_dev || window->ldg % 4 == 0), "lcu_attention_windowed: row strides %d %d", ldo, window->ldg);
  if (n == 0) return LCU_OK;
  hipStream_t st = as_stream(stream);
  const window_args p = make_window(window, ldq, ldo);
  if (dtype == LCU_F32) {
    const long seen = (long)window->window + window->keep;
    const size_t lds = (size_t)(seen < start + n ? seen : start + n) * sizeof(float);
    LCU_REQUIRE(lds <= 128 * 1024, "lcu_attention_windowed: %zu visible keys (at most 32768 in fp32)", lds / 4);
    static bool raised[16] = {};
    int dev = 0;
    LCU_HIP(hipGetDevice(&dev));
    if (!raised[dev & 15]) {
      LCU_HIP(hipFuncSetAttribute((const void*)attention_row_kernel<float>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024));
      raised[dev & 15] = true;
    }
    attention_row_kernel<float><<<dim3(n, window->heads), 256, lds, st>>>((float*)out_dev, (const float*)q_dev, (const float*)k_cache_dev,
                                                                          (const float*)v_cache_dev, start, p);
    LCU_LAUNCH_CHECK();
    return LCU_OK;
  }
  const auto run = [&](auto size) {
    constexpr int DV = decltype(size)::value;
    return p.r1 ? launch_tiles<DV, true>(out_dev, q_dev, k_cache_dev, v_cache_dev, n, start, p, st)
                : launch_tiles<DV, false>(out_dev, q_dev, k_cache_dev, v_cache_dev, n, start, p, st);
  };
  switch (window->dv) {
    case 32: return run(std::integral_constant<int, 32>{});
    case 64: return run(std::integral_constant<int, 64>{});
    case 128: return run(std::integral_constant<int, 128>{});
    default: return run(std::integral_constant<int, 256>{});
  }
}

int lcu_attention_windowed_decode(void* out_dev, const void* q_dev, const void* k_cache_dev, const void* v_cache_dev,
                                  const void* pos_dev, int max_positions, const lcu_window_params* window, void* arrived_dev,
                                  void* stream) {
  LCU_REQUIRE(out_dev && q_dev && k_cache_dev && v_cache_dev && pos_dev && arrived_dev, "lcu_attention_windowed_decode: null pointer");
  const int rc = check_window("lcu_attention_windowed_decode", window, LCU_BF16);
  if (rc) return rc;
  const int R = window->heads / window->kv_heads;
  LCU_REQUIRE(window->r1_dev && window->dk_shared == 0 && !window->sink_dev && !window->gate_dev && window->first_position == 0 &&
                  window->k_ld == 0 && window->v_ld == 0,
              "lcu_attention_windowed_decode: only the distance bias and caches of its own layout");
  LCU_REQUIRE(R <= DEC_MAX_GROUP && max_positions > 0, "lcu_attention_windowed_decode: %d query heads per kv head (at most %d)", R,
              DEC_MAX_GROUP);
  hipStream_t st = as_stream(stream);
  const workspace_t ws = workspace_for(st);
  if (ws.ptr == nullptr) return set_error(LCU_E_NOINIT, "lcu_attention_windowed_decode: lcu_init has not run on this device");
  const long seen = (long)window->window + window->keep;
  const int most = (int)(seen < max_positions ? seen : max_positions);  // visible keys of any position
  // a slice for every 64 keys, sixteen of them while that gives half the compute units a workgroup
  const int even = std::max(DEC_TOGETHER, 128 / window->kv_heads);
  const int slices = std::min(std::min((most + 63) / 64, even), DEC_MAX_SLICES);
  const size_t need = (size_t)window->heads * slices * (window->dv + 4) * sizeof(float);
  LCU_REQUIRE(need <= ws.bytes, "lcu_attention_windowed_decode: %d slices do not fit the workspace", slices);
  LCU_REQUIRE((size_t)16 * R * (window->dv + 2) * sizeof(float) <= 150 * 1024,
              "lcu_attention_windowed_decode: %d query heads per kv head with value size %d", R, window->dv);
  const window_args p = make_window(window, window->heads * window->dk, window->heads * window->dv);
  const auto run = [&](auto dkp, auto dvp) {
    return launch_decode<decltype(dkp)::value, decltype(dvp)::value>(
        (bf16_t*)out_dev, (const bf16_t*)q_dev, (const bf16_t*)k_cache_dev, (const bf16_t*)v_cache_dev, (const int*)pos_dev,
        max_positions, (float*)ws.ptr, (uint32_t*)arrived_dev, p, slices, st);
  };
  const std::integral_constant<int, 1> one;
  const std::integral_constant<int, 2> two;
  if (window->dk <= 128) return window->dv <= 128 ? run(one, one) : run(one, two);
  return window->dv <= 128 ? run(two, one) : run(two, two);
}

}  // extern "C"
