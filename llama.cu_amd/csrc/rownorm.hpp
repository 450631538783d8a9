// Grouped RMS norm of one row by one workgroup, the row in registers.
#pragma once
#include "common.hpp"

namespace lcu {

constexpr int ROW_THREADS = 256;    // many rows: a workgroup each
constexpr int STEP_THREADS = 1024;  // a single row: the launch is nothing but latency
constexpr int ROW_MAX_WIDTH = 12288;
constexpr int ROW_MAX_GROUPS = 2048;
constexpr int ROW_PIECE = WAVE * 4;  // columns a wavefront holds per register piece

struct row_shape {
  int width, ld, groups;  // elements of a row, row stride in memory, equal consecutive parts
  float eps;
};

// where a sublayer left its result
struct sublayer_rows {
  const float* out;
  const int* inverse;  // top rows of out per token: rows inverse[r * top + k], or r * top + k when NULL
  int top;
  const float* shared;
  const float* shared_gate;
};

// A row spread over the workgroup's registers: piece j of thread t holds the four columns from
// (t + TH j) * 4 (TH threads).  Columns at or beyond the width hold zeros.
template <int NV, int TH>
struct row_t {
  float4_t v[NV];
  static __device__ __forceinline__ int column(int j) { return (int)(threadIdx.x + TH * j) * 4; }
};

__device__ __forceinline__ float4_t load4(const float* p) { return *reinterpret_cast<const float4_t*>(p); }
__device__ __forceinline__ float4_t load4(const bf16_t* p) {
  typedef uint32_t uint2_t __attribute__((ext_vector_type(2)));
  const uint2_t u = *reinterpret_cast<const uint2_t*>(p);
  float4_t r;
  r[0] = __builtin_bit_cast(float, u[0] << 16);
  r[1] = __builtin_bit_cast(float, u[0] & 0xffff0000u);
  r[2] = __builtin_bit_cast(float, u[1] << 16);
  r[3] = __builtin_bit_cast(float, u[1] & 0xffff0000u);
  return r;
}
__device__ __forceinline__ void store4(float* p, float4_t v) { *reinterpret_cast<float4_t*>(p) = v; }
__device__ __forceinline__ void store4(bf16_t* p, float4_t v) {
  typedef bf16_t bf16x4_t __attribute__((ext_vector_type(4)));
  *reinterpret_cast<bf16x4_t*>(p) = __builtin_convertvector(v, bf16x4_t);
}

// Rows have a padded stride (a multiple of 64 elements), so whole pieces up to ld may be read and written;
// vectors of the width (norm weights) are padded by their owners to ld too.
template <int NV, int TH, class T>
__device__ __forceinline__ void load_row(row_t<NV, TH>& r, const T* p, const row_shape& rs) {
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = r.column(j);
    r.v[j] = c < rs.ld ? load4(p + c) : (float4_t)(0.0f);
  }
}
template <int NV, int TH, class T>
__device__ __forceinline__ void store_row(T* p, const row_t<NV, TH>& r, const row_shape& rs) {
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = r.column(j);
    if (c < rs.ld) store4(p + c, r.v[j]);
  }
}

// LDS a workgroup needs for scale_row
inline size_t row_lds_bytes(const row_shape& rs) {
  const size_t quads = (size_t)rs.ld / 4;                        // general form: a partial sum per four columns ...
  const size_t pieces = (rs.ld + ROW_PIECE - 1) / ROW_PIECE;     // ... or one per piece of a wavefront
  const bool whole = rs.width % rs.groups == 0 && (rs.width / rs.groups) % ROW_PIECE == 0;
  return ((whole ? pieces : quads * 4) + rs.groups) * sizeof(float);
}

// row <- row / sqrt(mean of its part's squares + eps) * w.  Parts that are whole pieces of a wavefront (256
// columns) are summed in registers; other sizes go through LDS column by column.  `lds` may be reused right
// after an earlier call.
template <int NV, int TH>
__device__ __forceinline__ void scale_row(row_t<NV, TH>& r, const row_shape& rs, float* lds, const row_t<NV, TH>& w) {
  constexpr int WAVES = TH / WAVE;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, part = rs.width / rs.groups;
  if (part % ROW_PIECE == 0) {
    float* piece = lds;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const float4_t q = r.v[j] * r.v[j];
      const float s = wave_sum((q[0] + q[1]) + (q[2] + q[3]));
      if (lane == 0 && r.column(j) < rs.ld) piece[j * WAVES + wave] = s;
    }
    __syncthreads();
    const int per = part / ROW_PIECE;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int g = __builtin_amdgcn_readfirstlane((j * WAVES + wave) / per);
      if (g < rs.groups) {
        float total = 0.0f;
        for (int k = 0; k < per; ++k) total += piece[g * per + k];
        r.v[j] *= (1.0f / sqrtf(total / (float)part + rs.eps)) * w.v[j];
      }
    }
    __syncthreads();
    return;
  }
  float* sq = lds;                     // [ld] squares
  float* inv = lds + rs.ld;            // [groups]
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = r.column(j);
    if (c < rs.ld) store4(sq + c, r.v[j] * r.v[j]);
  }
  __syncthreads();
  for (int g = wave; g < rs.groups; g += WAVES) {
    float s = 0.0f;
    for (int i = lane; i < part; i += WAVE) s += sq[g * part + i];
    s = wave_sum(s);
    if (lane == 0) inv[g] = 1.0f / sqrtf(s / (float)part + rs.eps);
  }
  __syncthreads();
#pragma unroll
  for (int j = 0; j < NV; ++j) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int c = r.column(j) + e;
      r.v[j][e] = c < rs.width ? r.v[j][e] * inv[c / part] * w.v[j][e] : 0.0f;
    }
  }
  __syncthreads();
}

// calls f with the number of pieces per thread that covers the row stride
template <class F>
void with_row_pieces(int ld, F&& f) {
  if (ld <= 1024) {
    f(std::integral_constant<int, 1>{});
  } else if (ld <= 2048) {
    f(std::integral_constant<int, 2>{});
  } else if (ld <= 4096) {
    f(std::integral_constant<int, 4>{});
  } else if (ld <= 8192) {
    f(std::integral_constant<int, 8>{});
  } else {
    f(std::integral_constant<int, 12>{});
  }
}
// the same for STEP_THREADS threads
template <class F>
void with_step_pieces(int ld, F&& f) {
  if (ld <= 4096) {
    f(std::integral_constant<int, 1>{});
  } else if (ld <= 8192) {
    f(std::integral_constant<int, 2>{});
  } else {
    f(std::integral_constant<int, 3>{});
  }
}

}  // namespace lcu
