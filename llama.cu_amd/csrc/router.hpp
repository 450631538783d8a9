// Choice of experts from router logits.
#pragma once
#include "linear.hpp"

namespace lcu {

constexpr int ROUTER_MAX_ROWS = 513;  // 512 experts and the shared expert's gate

struct router_step {
  const bf16_t* w;     // [rows][ld]; NULL: no router
  int rows, experts, top;
  int* expert;
  float* weight;
  float* shared_gate;  // NULL: no gate row behind the experts'
};

// One wavefront: the `top` largest of z (LDS; ties: the smaller index), with their scores sigmoid(z).  z is
// used up.
__device__ __forceinline__ void choose_experts(float* z, int n_experts, int top, int* __restrict__ expert, float* __restrict__ weight) {
  const int lane = threadIdx.x & 63;
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY;
    int idx = 0x7fffffff;
    for (int e = lane; e < n_experts; e += WAVE) {
      const float v = z[e];
      if (v > best || (v == best && e < idx)) {
        best = v;
        idx = e;
      }
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float ob = __shfl_xor(best, off, WAVE);
      const int oi = __shfl_xor(idx, off, WAVE);
      if (ob > best || (ob == best && oi < idx)) {
        best = ob;
        idx = oi;
      }
    }
    if (idx >= n_experts) idx = k;  // no finite logit left
    if (lane == 0) {
      expert[k] = idx;
      weight[k] = sigmoid_f32(best);
      z[idx] = -INFINITY;
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // z is LDS of this wavefront: its accesses are in order
  }
}

}  // namespace lcu
