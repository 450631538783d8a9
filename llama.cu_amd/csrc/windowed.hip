// Attention over a key/value cache with a sliding window, kept first tokens, grouped heads and a
// per-head distance bias:
//   score(i, j) = scale q_i.k_j - r1 ln(1 + r2 (i - j)),  visible when j <= i and (i - j < window or j < keep)
// followed by an ordinary softmax.  Scores, softmax and weighted sums are fp32.
//
// Layouts: q rows of heads x dk inside rows of ldq elements; caches k [positions][kv_heads * dk] and
// v [positions][kv_heads * dv].  dk is the head size padded to a multiple of 32, dv the value size padded
// to 32, 64, 128 or 256; the padding holds zeros.  A head's visible keys are the first ones, [0, kept), and
// the window [lo, i]: every kernel walks exactly these.
#include <algorithm>

#include "linear.hpp"
#include "rownorm.hpp"

using namespace lcu;

namespace {

struct window_args {
  int heads, kv_heads, dk, dv, ldq, ldo;
  int window, keep;
  float scale;
  const float* r1;
  const float* r2;
};

// first key of the window of position i, and how many kept keys lie below it
__device__ __forceinline__ int window_begin(const window_args& p, int i) { return max(0, i - p.window + 1); }

// ---- new rows of the caches -----------------------------------------------------------------------------
// Row t of qkv holds q | k | v.  k goes to cache row start + t; v too, after mixing with the row of
// v_first when MIX_WITH: (1 - lambda) v + lambda v_first; KEEP_AS_FIRST leaves the projected v in v_first.
enum v_mode { V_PLAIN = 0, V_KEEP_AS_FIRST = 1, V_MIX_WITH_FIRST = 2 };

template <class T>
__device__ __forceinline__ float mixed_value(float v, T* v_first, int mode, float lambda) {
  if (mode == V_KEEP_AS_FIRST) *v_first = (T)v;
  if (mode == V_MIX_WITH_FIRST) v = (1.0f - lambda) * v + lambda * to_f32(*v_first);
  return v;
}

template <class T>
__global__ __launch_bounds__(256) void kv_store_kernel(T* __restrict__ k_cache, T* __restrict__ v_cache, const T* __restrict__ qkv,
                                                       int ldq, int q_cols, int k_cols, int v_cols, T* __restrict__ v_first,
                                                       int mode, const float* __restrict__ lambda, const int* __restrict__ start,
                                                       int max_pos) {
  const int c = blockIdx.x * 256 + threadIdx.x, t = blockIdx.y;
  if (c >= k_cols + v_cols) return;
  const size_t pos = min(max(*start + t, 0), max_pos - 1);
  const T* row = qkv + (size_t)t * ldq + q_cols;
  if (c < k_cols) {
    k_cache[pos * k_cols + c] = row[c];
  } else {
    const int vc = c - k_cols;
    const float v = mixed_value(to_f32(row[c]), v_first + (size_t)t * v_cols + vc, mode, mode == V_MIX_WITH_FIRST ? *lambda : 0.0f);
    v_cache[pos * v_cols + vc] = (T)v;
  }
}

// ---- one workgroup per (query row, head), plain fp32 arithmetic: the fp32 element type -----------------
template <class T>
__global__ __launch_bounds__(256) void attention_row_kernel(T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ k,
                                                            const T* __restrict__ v, int start, window_args p) {
  extern __shared__ float sc[];  // scores of the visible keys
  __shared__ float red[4];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int t = blockIdx.x, h = blockIdx.y, g = h / (p.heads / p.kv_heads), i = start + t;
  const int lo = window_begin(p, i), kept = min(p.keep, lo), n_keys = kept + i - lo + 1;
  const T* qr = q + (size_t)t * p.ldq + (size_t)h * p.dk;
  const float r1 = p.r1[h], r2 = p.r2[h];
  float m = -INFINITY;
  for (int x = wave; x < n_keys; x += 4) {
    const int j = x < kept ? x : lo + x - kept;
    const T* kr = k + ((size_t)j * p.kv_heads + g) * p.dk;
    float s = 0.0f;
    for (int c = lane; c < p.dk; c += WAVE) s = fmaf(to_f32(qr[c]), to_f32(kr[c]), s);
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
  for (int c = tid; c < p.dv; c += 256) {
    float o = 0.0f;
    for (int x = 0; x < n_keys; ++x) {
      const int j = x < kept ? x : lo + x - kept;
      o = fmaf(sc[x], to_f32(v[((size_t)j * p.kv_heads + g) * p.dv + c]), o);
    }
    out[(size_t)t * p.ldo + (size_t)h * p.dv + c] = (T)(o / l);
  }
}

// ---- prompts, bfloat16: matrix cores --------------------------------------------------------------------
// One workgroup: 64 query rows of one head, 16 per wavefront, against tiles of 64 keys with a running
// maximum and sum.  Key tiles that hold no visible key of any of the rows (between the kept tokens and the
// windows) are not visited.  Probabilities go into the second product as two bfloat16 terms (value and
// remainder), so that they keep 16 significant bits.
constexpr int QT = 64, KT = 64;

template <int DV>
__global__ __launch_bounds__(256) void attention_tile_kernel(bf16_t* __restrict__ out, const bf16_t* __restrict__ q,
                                                             const bf16_t* __restrict__ k, const bf16_t* __restrict__ v, int n,
                                                             int start, window_args p) {
  constexpr int NT = DV / 16;
  constexpr int LDP = KT + 8;
  extern __shared__ __attribute__((aligned(16))) unsigned char attn_lds[];
  const int ldk = p.dk + 8;
  bf16_t* Qs = reinterpret_cast<bf16_t*>(attn_lds);   // [QT][ldk]
  bf16_t* Ks = Qs + QT * ldk;                         // [KT][ldk]
  bf16_t* Vt = Ks + KT * ldk;                         // [DV][LDP]: values, transposed
  bf16_t* Ps = Vt + DV * LDP;                         // [wave][value, remainder][16][LDP]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int q0 = (gridDim.x - 1 - blockIdx.x) * QT, h = blockIdx.y, g = h / (p.heads / p.kv_heads);
  const int dk8 = p.dk / 8;
  for (int c = tid; c < QT * dk8; c += 256) {
    const int r = c / dk8, e = (c % dk8) * 8;
    *reinterpret_cast<uint4_t*>(Qs + r * ldk + e) =
        *reinterpret_cast<const uint4_t*>(q + (size_t)min(q0 + r, n - 1) * p.ldq + (size_t)h * p.dk + e);
  }
  const float r1 = p.r1[h], r2 = p.r2[h];
  const int first = start + q0, last = start + min(q0 + QT, n) - 1;  // positions of the tile's rows
  const int win_tile = window_begin(p, first) / KT, kept_tiles = (min(p.keep, first + QT) + KT - 1) / KT;
  const int col = lane & 15, quad = lane >> 4;
  float m[4], l[4];
  float4_t o[NT];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    m[e] = -1e30f;
    l[e] = 0.0f;
  }
#pragma unroll
  for (int t = 0; t < NT; ++t) o[t] = (float4_t)(0.0f);
  bf16_t* Pw = Ps + wave * 2 * 16 * LDP;

  for (int kt = kept_tiles > 0 ? 0 : win_tile; kt * KT <= last; ++kt) {
    if (kt >= kept_tiles && kt < win_tile) kt = win_tile;
    const int k0 = kt * KT;
    __syncthreads();  // the previous tile has been read
    for (int c = tid; c < KT * dk8; c += 256) {
      const int r = c / dk8, e = (c % dk8) * 8;
      *reinterpret_cast<uint4_t*>(Ks + r * ldk + e) =
          *reinterpret_cast<const uint4_t*>(k + ((size_t)min(k0 + r, last) * p.kv_heads + g) * p.dk + e);
    }
    for (int c = tid; c < KT * (DV / 8); c += 256) {
      const int r = c % KT, e = (c / KT) * 8;
      const bf16x8_t x = *reinterpret_cast<const bf16x8_t*>(v + ((size_t)min(k0 + r, last) * p.kv_heads + g) * DV + e);
#pragma unroll
      for (int b = 0; b < 8; ++b) Vt[(e + b) * LDP + r] = x[b];
    }
    __syncthreads();
    float4_t s[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) s[t] = (float4_t)(0.0f);
    for (int c = 0; c < p.dk; c += 32) {
      const bf16x8_t a = *reinterpret_cast<const bf16x8_t*>(Qs + (wave * 16 + col) * ldk + c + quad * 8);
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        const bf16x8_t b = *reinterpret_cast<const bf16x8_t*>(Ks + (t * 16 + col) * ldk + c + quad * 8);
        s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, s[t], 0, 0, 0);
      }
    }
    // element e of s[t]: row quad * 4 + e of the wavefront's 16, key t * 16 + col
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = first + wave * 16 + quad * 4 + e;
      float top = -1e30f;
      bool see[4];
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        const int j = k0 + t * 16 + col, d = i - j;
        see[t] = d >= 0 && (d < p.window || j < p.keep);
        s[t][e] = s[t][e] * p.scale - r1 * __logf(1.0f + r2 * (float)max(d, 0));
        if (see[t]) top = fmaxf(top, s[t][e]);
      }
      top = fmaxf(top, dpp_f32<0xB1>(top));
      top = fmaxf(top, dpp_f32<0x4E>(top));
      top = fmaxf(top, dpp_f32<0x141>(top));
      top = fmaxf(top, dpp_f32<0x140>(top));
      const float m_new = fmaxf(m[e], top);
      const float shrink = __expf(m[e] - m_new);
      m[e] = m_new;
      float sum = 0.0f;
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        const float pr = see[t] ? __expf(s[t][e] - m_new) : 0.0f;
        sum += pr;
        const bf16_t hi = (bf16_t)pr;
        Pw[(quad * 4 + e) * LDP + t * 16 + col] = hi;
        Pw[(16 + quad * 4 + e) * LDP + t * 16 + col] = (bf16_t)(pr - (float)hi);
      }
      l[e] = l[e] * shrink + row16_sum(sum);
#pragma unroll
      for (int t = 0; t < NT; ++t) o[t][e] *= shrink;
    }
    __syncthreads();  // P is written and read by the same wavefront; the barrier orders its LDS accesses
#pragma unroll
    for (int c = 0; c < KT; c += 32) {
      const bf16x8_t hi = *reinterpret_cast<const bf16x8_t*>(Pw + col * LDP + c + quad * 8);
      const bf16x8_t rem = *reinterpret_cast<const bf16x8_t*>(Pw + (16 + col) * LDP + c + quad * 8);
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const bf16x8_t b = *reinterpret_cast<const bf16x8_t*>(Vt + (t * 16 + col) * LDP + c + quad * 8);
        o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(rem, b, o[t], 0, 0, 0);
        o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, b, o[t], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int r = q0 + wave * 16 + quad * 4 + e;
    if (r < n) {
      const float inv = 1.0f / l[e];
#pragma unroll
      for (int t = 0; t < NT; ++t) out[(size_t)r * p.ldo + (size_t)h * DV + t * 16 + col] = (bf16_t)(o[t][e] * inv);
    }
  }
}

size_t tile_lds(int dk, int dv) {
  return ((size_t)(QT + KT) * (dk + 8) + (size_t)dv * (KT + 8) + (size_t)4 * 2 * 16 * (KT + 8)) * 2;
}

template <int DV>
int launch_tiles(void* out, const void* q, const void* k, const void* v, int n, int start, const window_args& p, hipStream_t st) {
  const size_t lds = tile_lds(p.dk, DV);
  LCU_REQUIRE(lds <= 160 * 1024, "lcu_attention_windowed: head size %d with value size %d", p.dk, DV);
  auto kernel = attention_tile_kernel<DV>;
  static bool raised[16] = {};  // per device, once
  int dev = 0;
  LCU_HIP(hipGetDevice(&dev));
  if (!raised[dev & 15]) {
    LCU_HIP(hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));
    raised[dev & 15] = true;
  }
  kernel<<<dim3((n + QT - 1) / QT, p.heads), 256, lds, st>>>((bf16_t*)out, (const bf16_t*)q, (const bf16_t*)k, (const bf16_t*)v, n,
                                                              start, p);
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

// ---- one new token, bfloat16 ----------------------------------------------------------------------------
// Workgroup (kv head, slice of the visible keys): 16 lanes share a key row and score it for every query
// head of the group (the row is read once for all of them); then the slice's maximum, sum and weighted
// values per head go to part[kv head][slice][head][dv + 2], and the last workgroup of a kv head to arrive
// adds the slices up (arrives_last).  Nobody waits.
__device__ __forceinline__ float load_device(const float* p) {
  return __hip_atomic_load(p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
}
// eight loads at device scope in flight together (see load_words_device_scope)
__device__ __forceinline__ void load8_device(float (&o)[8], const float* const (&p)[8]) {
  asm volatile(
      "global_load_dword %0, %8, off sc0 sc1\n\tglobal_load_dword %1, %9, off sc0 sc1\n\t"
      "global_load_dword %2, %10, off sc0 sc1\n\tglobal_load_dword %3, %11, off sc0 sc1\n\t"
      "global_load_dword %4, %12, off sc0 sc1\n\tglobal_load_dword %5, %13, off sc0 sc1\n\t"
      "global_load_dword %6, %14, off sc0 sc1\n\tglobal_load_dword %7, %15, off sc0 sc1\n\ts_waitcnt vmcnt(0)"
      : "=&v"(o[0]), "=&v"(o[1]), "=&v"(o[2]), "=&v"(o[3]), "=&v"(o[4]), "=&v"(o[5]), "=&v"(o[6]), "=&v"(o[7])
      : "v"(p[0]), "v"(p[1]), "v"(p[2]), "v"(p[3]), "v"(p[4]), "v"(p[5]), "v"(p[6]), "v"(p[7])
      : "memory");
}
constexpr int DEC_MAX_SLICE = 256;   // keys of a slice
constexpr int DEC_MAX_GROUP = 16;    // query heads per kv head

__global__ __launch_bounds__(256) void attention_decode_kernel(bf16_t* __restrict__ out, const bf16_t* __restrict__ q,
                                                               const bf16_t* __restrict__ k, const bf16_t* __restrict__ v,
                                                               const int* __restrict__ pos_dev, int max_pos,
                                                               float* __restrict__ part, uint32_t* __restrict__ arrived,
                                                               window_args p) {
  extern __shared__ float dec_lds[];
  const int R = p.heads / p.kv_heads;
  float* qs = dec_lds;                   // [R][dk]
  float* sc = qs + R * p.dk;             // [R][DEC_MAX_SLICE]
  float* ov = sc + R * DEC_MAX_SLICE;    // [4][R][dv]
  __shared__ bool last;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int g = blockIdx.x, slice = blockIdx.y, slices = gridDim.y;
  const int i = min(max(*pos_dev, 0), max_pos - 1);
  const int lo = window_begin(p, i), kept = min(p.keep, lo), n_keys = kept + i - lo + 1;
  const int per = (n_keys + slices - 1) / slices;
  const int x0 = slice * per, cnt = max(0, min(per, n_keys - x0));
  for (int c = tid; c < R * p.dk; c += 256) qs[c] = (float)q[(size_t)g * R * p.dk + c];
  __syncthreads();
  const int sub = lane & 15, grp = tid >> 4;
  for (int x = grp; x < cnt; x += 16) {
    const int xi = x0 + x, j = xi < kept ? xi : lo + xi - kept;
    const bf16_t* kr = k + ((size_t)j * p.kv_heads + g) * p.dk;
    float s[DEC_MAX_GROUP];
#pragma unroll
    for (int r = 0; r < DEC_MAX_GROUP; ++r) s[r] = 0.0f;
    for (int c = sub * 8; c < p.dk; c += 128) {
      const bf16x8_t kv = *reinterpret_cast<const bf16x8_t*>(kr + c);
#pragma unroll
      for (int r = 0; r < DEC_MAX_GROUP; ++r) {
        if (r < R) {
#pragma unroll
          for (int e = 0; e < 8; ++e) s[r] = fmaf(qs[r * p.dk + c + e], (float)kv[e], s[r]);
        }
      }
    }
#pragma unroll
    for (int r = 0; r < DEC_MAX_GROUP; ++r) {
      if (r < R) {
        const float d = row16_sum(s[r]);
        if (sub == 0) sc[r * DEC_MAX_SLICE + x] = d * p.scale - p.r1[g * R + r] * log1pf(p.r2[g * R + r] * (float)(i - j));
      }
    }
  }
  __syncthreads();
  float* pg = part + (size_t)(g * slices + slice) * R * (p.dv + 2);
  for (int r = wave; r < R; r += 4) {
    float m = -1e30f;
    for (int x = lane; x < cnt; x += WAVE) m = fmaxf(m, sc[r * DEC_MAX_SLICE + x]);
    m = wave_max_dpp(m);
    float l = 0.0f;
    for (int x = lane; x < cnt; x += WAVE) {
      const float e = expf(sc[r * DEC_MAX_SLICE + x] - m);
      sc[r * DEC_MAX_SLICE + x] = e;
      l += e;
    }
    l = wave_sum(l);
    if (lane == 0) {
      __hip_atomic_store(pg + r * (p.dv + 2) + p.dv, m, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      __hip_atomic_store(pg + r * (p.dv + 2) + p.dv + 1, l, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
  }
  __syncthreads();
  // weighted values: wavefront w takes keys w, w + 4, ...; a lane owns columns lane, lane + 64, ...
  for (int c = lane; c < p.dv; c += WAVE) {
    float o[DEC_MAX_GROUP];
#pragma unroll
    for (int r = 0; r < DEC_MAX_GROUP; ++r) o[r] = 0.0f;
#pragma unroll 4
    for (int x = wave; x < cnt; x += 4) {
      const int xi = x0 + x, j = xi < kept ? xi : lo + xi - kept;
      const float vv = (float)v[((size_t)j * p.kv_heads + g) * p.dv + c];
#pragma unroll
      for (int r = 0; r < DEC_MAX_GROUP; ++r) {
        if (r < R) o[r] = fmaf(sc[r * DEC_MAX_SLICE + x], vv, o[r]);
      }
    }
#pragma unroll
    for (int r = 0; r < DEC_MAX_GROUP; ++r) {
      if (r < R) ov[(wave * R + r) * p.dv + c] = o[r];
    }
  }
  __syncthreads();
  for (int c = tid; c < R * p.dv; c += 256) {
    const int rd = R * p.dv;
    const float o = (ov[c] + ov[rd + c]) + (ov[2 * rd + c] + ov[3 * rd + c]);
    __hip_atomic_store(pg + (c / p.dv) * (p.dv + 2) + c % p.dv, o, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // every wavefront's stores are out before the count goes up
  __syncthreads();
  if (tid == 0) last = arrives_last(arrived + (size_t)g * ARRIVAL_WORDS, slice, slices);
  __syncthreads();
  if (!last) return;
  // factor and share of every slice, per head; then the columns
  const float* all = part + (size_t)g * slices * R * (p.dv + 2);
  float* sm = sc;              // [R][slices]: maxima, then factors (a slice is at most DEC_MAX_SLICE keys, and so are the slices)
  float* sl = dec_lds;         // [R]: sums (q is done with)
  for (int c = tid; c < R * slices; c += 256) {
    const int r = c / slices, s = c % slices;
    sm[r * DEC_MAX_SLICE + s] = load_device(all + ((size_t)s * R + r) * (p.dv + 2) + p.dv);
  }
  __syncthreads();
  for (int r = wave; r < R; r += 4) {
    float m = -1e30f;
    for (int s = lane; s < slices; s += WAVE) m = fmaxf(m, sm[r * DEC_MAX_SLICE + s]);
    m = wave_max_dpp(m);
    float l = 0.0f;
    for (int s = lane; s < slices; s += WAVE) {
      const float f = expf(sm[r * DEC_MAX_SLICE + s] - m);
      l += f * load_device(all + ((size_t)s * R + r) * (p.dv + 2) + p.dv + 1);
      sm[r * DEC_MAX_SLICE + s] = f;
    }
    l = wave_sum(l);
    if (lane == 0) sl[r] = l;
  }
  __syncthreads();
  for (int c = tid; c < R * p.dv; c += 256) {
    const int r = c / p.dv, e = c % p.dv;
    float o = 0.0f;
    for (int s0 = 0; s0 < slices; s0 += 8) {
      float v[8];
      const float* at[8];
#pragma unroll
      for (int k = 0; k < 8; ++k) at[k] = all + ((size_t)min(s0 + k, slices - 1) * R + r) * (p.dv + 2) + e;
      load8_device(v, at);
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        if (s0 + k < slices) o = fmaf(sm[r * DEC_MAX_SLICE + s0 + k], v[k], o);
      }
    }
    out[(size_t)(g * R + r) * p.dv + e] = (bf16_t)(o / sl[r]);
  }
}

int check_window(const char* who, const lcu_window_params* w, int dtype) {
  LCU_REQUIRE(w && w->r1_dev && w->r2_dev, "%s: null pointer", who);
  LCU_REQUIRE(dtype == LCU_BF16 || dtype == LCU_F32, "%s: element type %d", who, dtype);
  LCU_REQUIRE(w->heads > 0 && w->kv_heads > 0 && w->heads % w->kv_heads == 0 && w->dk > 0 && w->dk % 32 == 0 && w->dk <= 256 &&
                  (w->dv == 32 || w->dv == 64 || w->dv == 128 || w->dv == 256),
              "%s: heads %d / %d, head size %d (a multiple of 32, at most 256), value size %d (32, 64, 128, 256)", who, w->heads,
              w->kv_heads, w->dk, w->dv);
  LCU_REQUIRE(w->window > 0 && w->keep >= 0 && w->heads <= 65535, "%s: window %d keep %d", who, w->window, w->keep);
  return LCU_OK;
}

window_args make_window(const lcu_window_params* w, int ldq, int ldo) {
  return window_args{w->heads, w->kv_heads, w->dk, w->dv, ldq, ldo, w->window, w->keep, w->scale, (const float*)w->r1_dev,
                     (const float*)w->r2_dev};
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
  const dim3 grid((k_cols + v_cols + 255) / 256, n);
  hipStream_t st = as_stream(stream);
  if (dtype == LCU_F32) {
    kv_store_kernel<float><<<grid, 256, 0, st>>>((float*)k_cache_dev, (float*)v_cache_dev, (const float*)qkv_dev, ldq, q_cols, k_cols,
                                                 v_cols, (float*)v_first_dev, v_mode, (const float*)lambda_dev,
                                                 (const int*)start_dev, max_positions);
  } else {
    kv_store_kernel<bf16_t><<<grid, 256, 0, st>>>((bf16_t*)k_cache_dev, (bf16_t*)v_cache_dev, (const bf16_t*)qkv_dev, ldq, q_cols,
                                                  k_cols, v_cols, (bf16_t*)v_first_dev, v_mode, (const float*)lambda_dev,
                                                  (const int*)start_dev, max_positions);
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
  switch (window->dv) {
    case 32: return launch_tiles<32>(out_dev, q_dev, k_cache_dev, v_cache_dev, n, start, p, st);
    case 64: return launch_tiles<64>(out_dev, q_dev, k_cache_dev, v_cache_dev, n, start, p, st);
    case 128: return launch_tiles<128>(out_dev, q_dev, k_cache_dev, v_cache_dev, n, start, p, st);
    default: return launch_tiles<256>(out_dev, q_dev, k_cache_dev, v_cache_dev, n, start, p, st);
  }
}

int lcu_attention_windowed_decode(void* out_dev, const void* q_dev, const void* k_cache_dev, const void* v_cache_dev,
                                  const void* pos_dev, int max_positions, const lcu_window_params* window, void* arrived_dev,
                                  void* stream) {
  LCU_REQUIRE(out_dev && q_dev && k_cache_dev && v_cache_dev && pos_dev && arrived_dev, "lcu_attention_windowed_decode: null pointer");
  const int rc = check_window("lcu_attention_windowed_decode", window, LCU_BF16);
  if (rc) return rc;
  const int R = window->heads / window->kv_heads;
  LCU_REQUIRE(R <= DEC_MAX_GROUP && max_positions > 0, "lcu_attention_windowed_decode: %d query heads per kv head (at most %d)", R,
              DEC_MAX_GROUP);
  hipStream_t st = as_stream(stream);
  const workspace_t ws = workspace_for(st);
  if (ws.ptr == nullptr) return set_error(LCU_E_NOINIT, "lcu_attention_windowed_decode: lcu_init has not run on this device");
  const long seen = (long)window->window + window->keep;
  const int most = (int)(seen < max_positions ? seen : max_positions);  // visible keys of any position
  // slices: enough workgroups for the chip, at least 32 keys each, never more keys than a slice holds
  int slices = std::min((most + 31) / 32, (256 + window->kv_heads - 1) / window->kv_heads);
  slices = std::max(slices, (most + DEC_MAX_SLICE - 1) / DEC_MAX_SLICE);
  const size_t need = (size_t)window->heads * slices * (window->dv + 2) * sizeof(float);
  const size_t lds = ((size_t)R * (window->dk + DEC_MAX_SLICE + 4 * window->dv)) * sizeof(float);
  LCU_REQUIRE(need <= ws.bytes && slices <= DEC_MAX_SLICE, "lcu_attention_windowed_decode: %d slices do not fit the workspace", slices);
  LCU_REQUIRE(lds <= 128 * 1024, "lcu_attention_windowed_decode: %d heads of %d / %d per kv head", R, window->dk, window->dv);
  static bool raised[16] = {};
  int dev = 0;
  LCU_HIP(hipGetDevice(&dev));
  if (!raised[dev & 15]) {
    LCU_HIP(hipFuncSetAttribute((const void*)attention_decode_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024));
    raised[dev & 15] = true;
  }
  const window_args p = make_window(window, window->heads * window->dk, window->heads * window->dv);
  attention_decode_kernel<<<dim3(window->kv_heads, slices), 256, lds, st>>>((bf16_t*)out_dev, (const bf16_t*)q_dev,
                                                                           (const bf16_t*)k_cache_dev, (const bf16_t*)v_cache_dev,
                                                                           (const int*)pos_dev, max_positions, (float*)ws.ptr,
                                                                           (uint32_t*)arrived_dev, p);
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

}  // extern "C"
