// Mixture of experts: router (scores, choice of the largest, gate of the shared expert) and the
// plan that sorts the tokens' choices by expert for the grouped products (linear.hip).
#include "router.hpp"

using namespace lcu;

namespace {

constexpr int MAX_EXPERTS = ROUTER_MAX_ROWS - 1;

// One workgroup per token: logit e = row e of w . h in fp32, then the `top` largest (ties: the smaller
// index), their scores sigmoid(z), and sigmoid of the row behind the experts' (the shared gate).
template <class T>
__global__ __launch_bounds__(256) void router_kernel(int* __restrict__ expert, float* __restrict__ weight,
                                                     float* __restrict__ shared_gate, const T* __restrict__ h,
                                                     const T* __restrict__ w, int n_experts, int top, int K) {
  __shared__ float z[MAX_EXPERTS + 1];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, t = blockIdx.x;
  const T* ht = h + (size_t)t * K;
  const int n_rows = n_experts + (shared_gate ? 1 : 0);
  for (int e = wave; e < n_rows; e += 4) {
    const T* we = w + (size_t)e * K;
    float s = 0.0f;
    for (int k = lane; k < K; k += WAVE) s = fmaf(to_f32(ht[k]), to_f32(we[k]), s);
    s = wave_sum(s);
    if (lane == 0) z[e] = s;
  }
  __syncthreads();
  if (wave != 0) return;
  if (shared_gate && lane == 0) shared_gate[t] = sigmoid_f32(z[n_experts]);
  choose_experts(z, n_experts, top, expert + (size_t)t * top, weight + (size_t)t * top);
}

// The same for bfloat16 operands on the matrix cores: one workgroup takes 16 tokens and all rows of w, its eight
// wavefronts an eighth of K each, four tiles of 16 rows of w at a time; the eighths meet in LDS and are added
// in wavefront order, and every wavefront chooses for two of the tokens.
constexpr int ROUTER_TOKENS = 16, ROUTER_WAVES = 8;
template <int TILES>
__device__ __forceinline__ void router_tiles(float4_t (&acc)[4], const bf16_t* a, const bf16_t* const (&b)[4], int s0, int s1) {
#pragma unroll 8
  for (int s = s0; s < s1; ++s) {
    const bf16x8_t fa = *reinterpret_cast<const bf16x8_t*>(a + s * 32);
#pragma unroll
    for (int j = 0; j < TILES; ++j) {
      const bf16x8_t fb = *reinterpret_cast<const bf16x8_t*>(b[j] + s * 32);
      acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa, fb, acc[j], 0, 0, 0);
    }
  }
}

__global__ __launch_bounds__(64 * ROUTER_WAVES) void router_tile_kernel(int* __restrict__ expert, float* __restrict__ weight,
                                                          float* __restrict__ shared_gate, const bf16_t* __restrict__ h,
                                                          const bf16_t* __restrict__ w, int n, int n_experts, int top, int K) {
  extern __shared__ float zs[];  // [ROUTER_TOKENS][ldz]
  __shared__ float part[ROUTER_WAVES][ROUTER_TOKENS][64 + 1];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, t0 = blockIdx.x * ROUTER_TOKENS;
  const int n_rows = n_experts + (shared_gate ? 1 : 0), ldz = (n_rows + 15) / 16 * 16 + 1;
  const int col = lane & 15, quad = lane >> 4;
  const int steps = K / 32, s0 = wave * steps / ROUTER_WAVES, s1 = (wave + 1) * steps / ROUTER_WAVES;
  const bf16_t* a = h + (size_t)min(t0 + col, n - 1) * K + quad * 8;
  for (int e0 = 0; e0 < n_rows; e0 += 64) {
    float4_t acc[4];
    const bf16_t* b[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      acc[j] = (float4_t)(0.0f);
      b[j] = w + (size_t)min(e0 + j * 16 + col, n_rows - 1) * K + quad * 8;
    }
    const int tiles = min(4, (n_rows - e0 + 15) / 16);
    switch (tiles) {
      case 1: router_tiles<1>(acc, a, b, s0, s1); break;
      case 2: router_tiles<2>(acc, a, b, s0, s1); break;
      case 3: router_tiles<3>(acc, a, b, s0, s1); break;
      default: router_tiles<4>(acc, a, b, s0, s1); break;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
#pragma unroll
      for (int v = 0; v < 4; ++v) part[wave][quad * 4 + v][j * 16 + col] = acc[j][v];
    }
    __syncthreads();
    for (int i = tid; i < ROUTER_TOKENS * 64; i += 64 * ROUTER_WAVES) {
      const int t = i / 64, e = i % 64;
      float z = 0.0f;
#pragma unroll
      for (int x = 0; x < ROUTER_WAVES; ++x) z += part[x][t][e];
      if (e0 + e < n_rows) zs[t * ldz + e0 + e] = z;
    }
    __syncthreads();
  }
  for (int k = 0; k < ROUTER_TOKENS / ROUTER_WAVES; ++k) {
    const int t = t0 + wave * (ROUTER_TOKENS / ROUTER_WAVES) + k;
    if (t >= n) continue;
    float* z = zs + (t - t0) * ldz;
    if (shared_gate && lane == 0) shared_gate[t] = sigmoid_f32(z[n_experts]);
    choose_experts(z, n_experts, top, expert + (size_t)t * top, weight + (size_t)t * top);
  }
}

// One workgroup: counts per expert, their prefix sums, each choice's sorted row, and the row tiles.
__global__ __launch_bounds__(1024) void plan_kernel(const int* __restrict__ expert, const float* __restrict__ weight, int n, int top,
                                                    int n_experts, int tile_rows, int* __restrict__ row_token,
                                                    float* __restrict__ row_weight, int* __restrict__ inverse,
                                                    int* __restrict__ tile_expert, int* __restrict__ tile_row,
                                                    int* __restrict__ expert_end, int* __restrict__ n_tiles) {
  __shared__ int count[MAX_EXPERTS], next[MAX_EXPERTS], first_tile[MAX_EXPERTS];
  const int tid = threadIdx.x, rows = n * top;
  for (int e = tid; e < n_experts; e += 1024) count[e] = 0;
  __syncthreads();
  for (int i = tid; i < rows; i += 1024) atomicAdd(&count[expert[i]], 1);
  __syncthreads();
  if (tid == 0) {
    int at = 0, tiles = 0;
    for (int e = 0; e < n_experts; ++e) {
      next[e] = at;
      first_tile[e] = tiles;
      at += count[e];
      tiles += (count[e] + tile_rows - 1) / tile_rows;
    }
    *n_tiles = tiles;
  }
  __syncthreads();
  for (int e = tid; e < n_experts; e += 1024) {
    const int begin = next[e], end = begin + count[e];
    expert_end[e] = end;
    for (int r = begin, tl = first_tile[e]; r < end; r += tile_rows, ++tl) {
      tile_expert[tl] = e;
      tile_row[tl] = r;
    }
  }
  __syncthreads();
  for (int i = tid; i < rows; i += 1024) {
    const int r = atomicAdd(&next[expert[i]], 1);
    row_token[r] = i / top;
    row_weight[r] = weight[i];
    inverse[i] = r;
  }
}

}  // namespace

extern "C" {

int lcu_router(void* expert_dev, void* weight_dev, void* shared_gate_dev, const void* h_dev, const void* w_dev, int n_experts,
               int top, int dtype, int n, int K, void* stream) {
  LCU_REQUIRE(expert_dev && weight_dev && h_dev && w_dev, "lcu_router: null pointer");
  LCU_REQUIRE(n_experts > 0 && n_experts <= MAX_EXPERTS && top > 0 && top <= n_experts && n >= 0 && K > 0 && K % 64 == 0,
              "lcu_router: experts %d (at most %d), top %d", n_experts, MAX_EXPERTS, top);
  LCU_REQUIRE(dtype == LCU_BF16 || dtype == LCU_F32, "lcu_router: element type %d", dtype);
  if (n == 0) return LCU_OK;
  hipStream_t st = as_stream(stream);
  if (dtype == LCU_F32) {
    router_kernel<float><<<n, 256, 0, st>>>((int*)expert_dev, (float*)weight_dev, (float*)shared_gate_dev, (const float*)h_dev,
                                            (const float*)w_dev, n_experts, top, K);
  } else {
    const size_t lds = (size_t)ROUTER_TOKENS * ((n_experts + 1 + 15) / 16 * 16 + 1) * sizeof(float);
    static bool raised[16] = {};  // per device, once: hundreds of experts take more than 64 KB
    int dev = 0;
    LCU_HIP(hipGetDevice(&dev));
    if (!raised[dev & 15]) {
      LCU_HIP(hipFuncSetAttribute((const void*)router_tile_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024));
      raised[dev & 15] = true;
    }
    router_tile_kernel<<<(n + ROUTER_TOKENS - 1) / ROUTER_TOKENS, 64 * ROUTER_WAVES, lds, st>>>(
        (int*)expert_dev, (float*)weight_dev, (float*)shared_gate_dev, (const bf16_t*)h_dev, (const bf16_t*)w_dev, n, n_experts, top, K);
  }
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

int lcu_experts_plan(const lcu_expert_plan* plan, const void* expert_dev, const void* weight_dev, int n, int top, int n_experts,
                     void* stream) {
  LCU_REQUIRE(plan && expert_dev && weight_dev && plan->row_token_dev && plan->row_weight_dev && plan->inverse_dev &&
                  plan->tile_expert_dev && plan->tile_row_dev && plan->expert_end_dev && plan->n_tiles_dev,
              "lcu_experts_plan: null pointer");
  LCU_REQUIRE(n >= 0 && top > 0 && n_experts > 0 && n_experts <= MAX_EXPERTS && plan->tile_rows > 0,
              "lcu_experts_plan: n %d top %d experts %d", n, top, n_experts);
  // every expert may end in a partial tile
  LCU_REQUIRE((long)plan->max_tiles >= (long)n * top / plan->tile_rows + (n_experts < n * top ? n_experts : n * top),
              "lcu_experts_plan: room for %d tiles", plan->max_tiles);
  if (n == 0) return LCU_OK;
  plan_kernel<<<1, 1024, 0, as_stream(stream)>>>((const int*)expert_dev, (const float*)weight_dev, n, top, n_experts, plan->tile_rows,
                                                 (int*)plan->row_token_dev, (float*)plan->row_weight_dev, (int*)plan->inverse_dev,
                                                 (int*)plan->tile_expert_dev, (int*)plan->tile_row_dev,
                                                 (int*)plan->expert_end_dev, (int*)plan->n_tiles_dev);
  LCU_LAUNCH_CHECK();
  return LCU_OK;
}

}  // extern "C"
