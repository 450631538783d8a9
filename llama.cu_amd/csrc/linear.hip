// Linear layers of the layered decoders behind one interface for both element types: bfloat16
// operands go to the matrix-core kernel of gemm.hip, fp32 operands to the kernel here, which uses
// nothing narrower than fp32 anywhere (products by fused multiply-add, sums in k order).
#include "linear.hpp"

using namespace lcu;

namespace {

constexpr int FM = 32, FN = 64, FK = 32;  // tile rows, tile columns, K extent of a stage

// 256 threads; thread (column n = t % 64, row group t / 64) holds eight rows of one column.
template <class EP>
__global__ __launch_bounds__(256) void linear_f32_kernel(const float* __restrict__ A, const float* __restrict__ W, int M,
                                                         int K, int N, int tiles_m, EP ep) {
  __shared__ float As[FM][FK + 1];
  __shared__ float Ws[FN][FK + 1];
  __shared__ float Cs[EP::GATED ? FM : 1][EP::GATED ? FN : 1];
  const int tm = blockIdx.x % tiles_m, tn = blockIdx.x / tiles_m;
  int m0 = tm * FM;
  const int n0 = tn * FN;
  if constexpr (EP::GROUPED) {
    if (tm >= *ep.n_tiles) return;
    const int e = ep.tile_group[tm];
    m0 = ep.tile_row[tm];
    M = ep.group_end[e];
    W = reinterpret_cast<const float*>(reinterpret_cast<const char*>(W) + (size_t)e * ep.group_stride);
  }
  const int tid = threadIdx.x, nc = tid & 63, rg = tid >> 6;
  float acc[8];
#pragma unroll
  for (int r = 0; r < 8; ++r) acc[r] = 0.0f;
  for (int k0 = 0; k0 < K; k0 += FK) {
    __syncthreads();
    for (int c = tid; c < FM * FK; c += 256) {
      const int row = c / FK, k = c % FK;
      int gm = min(m0 + row, M - 1);
      if constexpr (EP::GROUPED) {
        if (ep.row_index) gm = ep.row_index[gm];
      }
      As[row][k] = A[(size_t)gm * K + k0 + k];
    }
    for (int c = tid; c < FN * FK; c += 256) {
      const int row = c / FK, k = c % FK;
      Ws[row][k] = W[(size_t)min(n0 + row, N - 1) * K + k0 + k];
    }
    __syncthreads();
#pragma unroll 8
    for (int k = 0; k < FK; ++k) {
      const float w = Ws[nc][k];
#pragma unroll
      for (int r = 0; r < 8; ++r) acc[r] = fmaf(As[rg * 8 + r][k], w, acc[r]);
    }
  }
  if constexpr (EP::GATED) {
#pragma unroll
    for (int r = 0; r < 8; ++r) Cs[rg * 8 + r][nc] = acc[r];
    __syncthreads();
    for (int c = tid; c < FM * 32; c += 256) {
      const int row = c / 32, j = c % 32;
      if (m0 + row < M && n0 < N) ep.store_gated(m0 + row, n0 / 2 + j, Cs[row][j], Cs[row][32 + j]);
    }
  } else {
#pragma unroll
    for (int r = 0; r < 8; ++r) {
      const int gm = m0 + rg * 8 + r, gn = n0 + nc;
      if (gm < M && gn < N) ep.store(gm, gn, acc[r]);
    }
  }
}

int check_linear(const char* who, int dtype, int M, int K, int N, int ldo) {
  LCU_REQUIRE(dtype == LCU_BF16 || dtype == LCU_F32, "%s: element type %d", who, dtype);
  LCU_REQUIRE(M >= 0 && N > 0 && K > 0 && K % 64 == 0 && ldo > 0, "%s: bad shape M %d K %d N %d (K %% 64 == 0)", who, M, K, N);
  const size_t es = dtype == LCU_F32 ? 4 : 2;
  LCU_REQUIRE((size_t)M * K * es < ((size_t)1 << 32) && (size_t)N * K * es < ((size_t)1 << 32),
              "%s: operands of 4 GiB or more are not supported", who);
  return LCU_OK;
}

template <bool GATED>
int run_linear(linear_epilogue<false, GATED> ep, int dtype, const void* lhs, const void* W, int M, int K, int N, hipStream_t st) {
  if (M == 0) return LCU_OK;
  if (dtype == LCU_F32) {
    const int tiles_m = (M + FM - 1) / FM, tiles_n = (N + FN - 1) / FN;
    linear_f32_kernel<<<tiles_m * tiles_n, 256, 0, st>>>((const float*)lhs, (const float*)W, M, K, N, tiles_m, ep);
    LCU_LAUNCH_CHECK();
    return LCU_OK;
  }
  return gemm_bf16<GATED>(ep, lhs, W, M, K, N, st);
}

template <bool GATED>
int run_grouped(linear_epilogue<true, GATED> ep, int dtype, const void* lhs, const void* W, int max_tiles, int K, int N,
                hipStream_t st) {
  if (dtype == LCU_F32) {
    linear_f32_kernel<<<max_tiles * ((N + FN - 1) / FN), 256, 0, st>>>((const float*)lhs, (const float*)W, 0, K, N,
                                                                      max_tiles, ep);
    LCU_LAUNCH_CHECK();
    return LCU_OK;
  }
  return gemm_bf16_grouped<GATED>(ep, lhs, W, max_tiles, K, N, st);
}

template <class EP>
void set_plan(EP& ep, const lcu_expert_plan* plan, const void* row_index, size_t group_stride) {
  ep.tile_group = (const int*)plan->tile_expert_dev;
  ep.tile_row = (const int*)plan->tile_row_dev;
  ep.group_end = (const int*)plan->expert_end_dev;
  ep.n_tiles = (const int*)plan->n_tiles_dev;
  ep.row_index = (const int*)row_index;
  ep.group_stride = group_stride;
  ep.tile_rows = plan->tile_rows;
}

bool plan_ok(const lcu_expert_plan* p, int dtype) {
  return p && p->tile_expert_dev && p->tile_row_dev && p->expert_end_dev && p->n_tiles_dev && p->row_token_dev &&
         p->max_tiles > 0 && (dtype == LCU_F32 ? p->tile_rows == FM : (p->tile_rows == 64 || p->tile_rows == 128 || p->tile_rows == 256));
}

}  // namespace

extern "C" {

int lcu_linear(void* out_dev, int out_f32, int ldo, const void* lhs_dev, const void* w_dev, const void* bias_dev,
               int gelu_cols, int dtype, int M, int K, int N, void* stream) {
  LCU_REQUIRE(out_dev && lhs_dev && w_dev, "lcu_linear: null pointer");
  const int rc = check_linear("lcu_linear", dtype, M, K, N, ldo);
  if (rc) return rc;
  LCU_REQUIRE(ldo >= N, "lcu_linear: row stride %d below N %d", ldo, N);
  linear_epilogue<false, false> ep{};
  ep.out = out_dev;
  ep.ldo = ldo;
  ep.out_f32 = out_f32 != 0 || dtype == LCU_F32;
  ep.bias = (const float*)bias_dev;
  ep.gelu_cols = gelu_cols;
  return run_linear<false>(ep, dtype, lhs_dev, w_dev, M, K, N, as_stream(stream));
}

int lcu_linear_tail(void* out_dev, int ldo, void* tail_f32_dev, int ld_tail, int tail_from, const void* lhs_dev, const void* w_dev,
                    int dtype, int M, int K, int N, void* stream) {
  LCU_REQUIRE(out_dev && tail_f32_dev && lhs_dev && w_dev, "lcu_linear_tail: null pointer");
  const int rc = check_linear("lcu_linear_tail", dtype, M, K, N, ldo);
  if (rc) return rc;
  LCU_REQUIRE(tail_from > 0 && tail_from < N && ldo >= tail_from && ld_tail >= N - tail_from,
              "lcu_linear_tail: columns from %d of %d, row strides %d %d", tail_from, N, ldo, ld_tail);
  linear_epilogue<false, false> ep{};
  ep.out = out_dev;
  ep.ldo = ldo;
  ep.out_f32 = dtype == LCU_F32;
  ep.tail = (float*)tail_f32_dev;
  ep.tail_from = tail_from;
  ep.ld_tail = ld_tail;
  return run_linear<false>(ep, dtype, lhs_dev, w_dev, M, K, N, as_stream(stream));
}

int lcu_linear_gated(void* out_dev, int ldo, const void* lhs_dev, const void* w_dev, const lcu_gate_params* gate, int dtype,
                     int M, int K, int N, void* stream) {
  LCU_REQUIRE(out_dev && lhs_dev && w_dev && gate, "lcu_linear_gated: null pointer");
  const int rc = check_linear("lcu_linear_gated", dtype, M, K, N, ldo);
  if (rc) return rc;
  LCU_REQUIRE(N % 64 == 0 && ldo >= N / 2, "lcu_linear_gated: N %d must be a multiple of 64, row stride %d at least N / 2", N, ldo);
  linear_epilogue<false, true> ep{};
  ep.out = out_dev;
  ep.ldo = ldo;
  ep.out_f32 = dtype == LCU_F32;
  ep.gate = clamped_gate{gate->limit, gate->alpha, gate->up_shift};
  return run_linear<true>(ep, dtype, lhs_dev, w_dev, M, K, N, as_stream(stream));
}

int lcu_experts_up(void* out_dev, int ldo, const void* lhs_dev, const void* w_dev, size_t expert_stride,
                   const lcu_gate_params* gate, const lcu_expert_plan* plan, int dtype, int n_tokens, int K, int N,
                   void* stream) {
  LCU_REQUIRE(out_dev && lhs_dev && w_dev && gate && plan_ok(plan, dtype), "lcu_experts_up: null pointer or bad plan");
  const int rc = check_linear("lcu_experts_up", dtype, n_tokens, K, N, ldo);
  if (rc) return rc;
  LCU_REQUIRE(N % 64 == 0 && ldo >= N / 2, "lcu_experts_up: N %d must be a multiple of 64, row stride %d at least N / 2", N, ldo);
  if (n_tokens == 0) return LCU_OK;
  linear_epilogue<true, true> ep{};
  ep.out = out_dev;
  ep.ldo = ldo;
  ep.out_f32 = dtype == LCU_F32;
  ep.gate = clamped_gate{gate->limit, gate->alpha, gate->up_shift};
  ep.row_scale = (const float*)plan->row_weight_dev;
  set_plan(ep, plan, plan->row_token_dev, expert_stride);
  return run_grouped<true>(ep, dtype, lhs_dev, w_dev, plan->max_tiles, K, N, as_stream(stream));
}

int lcu_experts_down(void* out_f32_dev, int ldo, const void* lhs_dev, const void* w_dev, size_t expert_stride,
                     const lcu_expert_plan* plan, int dtype, int n_rows, int K, int N, void* stream) {
  LCU_REQUIRE(out_f32_dev && lhs_dev && w_dev && plan_ok(plan, dtype), "lcu_experts_down: null pointer or bad plan");
  const int rc = check_linear("lcu_experts_down", dtype, n_rows, K, N, ldo);
  if (rc) return rc;
  LCU_REQUIRE(ldo >= N, "lcu_experts_down: row stride %d below N %d", ldo, N);
  if (n_rows == 0) return LCU_OK;
  linear_epilogue<true, false> ep{};
  ep.out = out_f32_dev;
  ep.ldo = ldo;
  ep.out_f32 = true;
  set_plan(ep, plan, nullptr, expert_stride);
  return run_grouped<false>(ep, dtype, lhs_dev, w_dev, plan->max_tiles, K, N, as_stream(stream));
}

}  // extern "C"
