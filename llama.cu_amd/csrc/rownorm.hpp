// Grouped RMS norm of one row held in LDS by one workgroup.
#pragma once
#include "common.hpp"

namespace lcu {

constexpr int ROW_THREADS = 256;
constexpr int ROW_WAVES = ROW_THREADS / WAVE;
constexpr int ROW_MAX_WIDTH = 12288;
constexpr int ROW_MAX_GROUPS = 2048;

struct row_shape {
  int width, ld, groups;  // elements of a row, row stride in memory, equal consecutive parts
  float eps;
};

// where a sublayer left its result
struct sublayer_rows {
  const float* out;
  const int* inverse;  // NULL: row r of out; else top rows of out per token
  int top;
  const float* shared;
  const float* shared_gate;
};

inline size_t row_lds_bytes(const row_shape& rs) {
  return ((size_t)rs.width + (rs.groups > ROW_WAVES ? rs.groups : ROW_WAVES)) * sizeof(float);
}

// row[c] <- row[c] / sqrt(mean of its part's squares + eps) * w[c].  Starts and ends with every thread's
// writes to row visible to the workgroup.  A part is summed by one wavefront, or by several when there are
// fewer parts than wavefronts.
__device__ __forceinline__ void group_scale(float* row, const row_shape& rs, float* scratch, const float* __restrict__ w) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int part = rs.width / rs.groups;
  __syncthreads();
  if (rs.groups >= ROW_WAVES) {
    for (int g = wave; g < rs.groups; g += ROW_WAVES) {
      float s = 0.0f;
      for (int i = lane; i < part; i += WAVE) s = fmaf(row[g * part + i], row[g * part + i], s);
      s = wave_sum(s);
      if (lane == 0) scratch[g] = 1.0f / sqrtf(s / (float)part + rs.eps);
    }
    __syncthreads();
    for (int c = threadIdx.x; c < rs.width; c += ROW_THREADS) row[c] = row[c] * scratch[c / part] * w[c];
  } else {
    const int share = ROW_WAVES / rs.groups;  // wavefronts of a part
    float s = 0.0f;
    if (wave < share * rs.groups) {
      const float* p = row + (wave / share) * part;
      for (int i = (wave % share) * WAVE + lane; i < part; i += share * WAVE) s = fmaf(p[i], p[i], s);
    }
    s = wave_sum(s);
    if (lane == 0) scratch[wave] = s;
    __syncthreads();
    for (int c = threadIdx.x; c < rs.width; c += ROW_THREADS) {
      const int g = c / part;
      float total = 0.0f;
      for (int k = 0; k < share; ++k) total += scratch[g * share + k];
      row[c] = row[c] * (1.0f / sqrtf(total / (float)part + rs.eps)) * w[c];
    }
  }
  __syncthreads();
}

}  // namespace lcu
