// Linear layers of the layered decoders: operand conventions and epilogues shared by the bfloat16
// matrix-core kernel (gemm.hip) and the 32-bit one (linear.hip).
//
// An activation is bfloat16 or fp32 ("element type", LCU_BF16 / LCU_F32); products accumulate in
// fp32.  Rows of activations and of weights are padded with zeros to a multiple of 64 elements, so
// every K is one.
#pragma once
#include "common.hpp"

namespace lcu {

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }

// 0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3)))
__device__ __forceinline__ float gelu_tanh(float z) {
  const float inner = 0.7978845608028654f * (z + 0.044715f * z * z * z);
  return 0.5f * z * (1.0f + tanhf(inner));
}

// min(g, limit), clamp(u, -limit, limit), then g sigmoid(alpha g) (u + up_shift)
struct clamped_gate {
  float limit, alpha, up_shift;
  __device__ __forceinline__ float operator()(float g, float u) const {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g * sigmoid_f32(alpha * g) * (u + up_shift);
  }
};

// GROUPED: rows are sorted by group (expert); row tile t belongs to group tile_group[t], starts at row
// tile_row[t] and ends at the group's end; group g multiplies matrix W + g * group_stride bytes; row r of lhs
// is row row_index[r] of the array when row_index is given.
// GATED: the matrix holds, in blocks of 64 rows, 32 gate rows and the 32 up rows of the same hidden columns.
template <bool GROUPED_, bool GATED_>
struct linear_epilogue {
  static constexpr bool BF16 = true, GROUPED = GROUPED_, GATED = GATED_;
  void* out;
  int ldo;
  bool out_f32;
  const float* bias;         // [N] or nullptr
  int gelu_cols;             // columns below this one pass through the GELU
  float* tail;               // fp32 rows [ld_tail] of the columns from tail_from on, or nullptr
  int tail_from, ld_tail;
  clamped_gate gate;
  const float* row_scale;    // factor of row r of lhs, or nullptr (gated products only)
  const int* tile_group;
  const int* tile_row;
  const int* group_end;
  const int* n_tiles;
  const int* row_index;
  size_t group_stride;
  int tile_rows;

  __device__ __forceinline__ void put(int m, int n, float v) const {
    const size_t at = (size_t)m * ldo + n;
    if (out_f32) {
      reinterpret_cast<float*>(out)[at] = v;
    } else {
      reinterpret_cast<bf16_t*>(out)[at] = (bf16_t)v;
    }
  }
  __device__ __forceinline__ void store(int m, int n, float v) const {
    if (bias) v += bias[n];
    if (n < gelu_cols) v = gelu_tanh(v);
    if (tail && n >= tail_from) {
      tail[(size_t)m * ld_tail + n - tail_from] = v;
      return;
    }
    put(m, n, v);
  }
  __device__ __forceinline__ void store_gated(int m, int n, float g, float u) const {
    const float s = row_scale ? row_scale[m] : 1.0f;
    put(m, n, gate(g * s, u * s));
  }
};

// gemm.hip
template <bool GATED>
int gemm_bf16(linear_epilogue<false, GATED> const& ep, const void* A, const void* W, int M, int K, int N, hipStream_t st);
template <bool GATED>
int gemm_bf16_grouped(linear_epilogue<true, GATED> const& ep, const void* A, const void* W, int max_tiles, int K, int N,
                      hipStream_t st);

// element access by type
template <class T>
__device__ __forceinline__ float to_f32(T v) { return (float)v; }

}  // namespace lcu
