// Weight-streaming products of a decode step's few rows (vy_rows.h) as launches of their own: y = act(x W^T + bias).
#include "vy_rows.h"

namespace {

using vy_rows::Dense;

template <int MB, int NW, int NT>
__global__ __launch_bounds__(64 * NW) void rows_linear_kernel(Dense a) {
  __shared__ f32x4 red[vy_rows::RED<NT, MB, NW>];
  vy_rows::dense<MB, NW, NT>(a, red, blockIdx.x);
}

template <int MB>
void rows_go(const Dense& a, hipStream_t st) {
  const unsigned tiles = (unsigned)((a.N + 15) / 16);
  // few workgroups with long rows: twice the waves each; many: two tiles each, for half the traffic of x
  if (a.N <= 4096 && a.K >= 2048) hipLaunchKernelGGL((rows_linear_kernel<MB, 8, 1>), dim3(tiles), dim3(512), 0, st, a);
  else if (MB == 1 || a.N < 8192) hipLaunchKernelGGL((rows_linear_kernel<MB, 4, 1>), dim3(tiles), dim3(256), 0, st, a);
  else hipLaunchKernelGGL((rows_linear_kernel<MB, 4, 2>), dim3((tiles + 1) / 2), dim3(256), 0, st, a);
}

}  // namespace

// internal (vy_hybrid.hip): bf16 y[M][N], 5 .. 32 rows of x (stride K) against w [N][K].  VY_ERR_UNSUPPORTED: other sizes.
int vy_rows_linear(const void* x, const void* w, const void* bias, int act, float act_arg, void* y, int64_t ldy, int64_t M, int64_t N,
                   int64_t K, hipStream_t st) {
  if (M < 5 || M > 32 || N > INT32_MAX || K > INT32_MAX || N < 16 || K < 8 || K % 8 || ldy % 8 || (uintptr_t)x % 16 || (uintptr_t)w % 16 ||
      (uintptr_t)y % 16 || (act != VY_ACT_NONE && act != VY_ACT_RELU2 && act != VY_ACT_SOFTCAP))
    return VY_ERR_UNSUPPORTED;
  const Dense a{(const bf16*)x, K, (int)M, (const bf16*)w, (int)N, (int)K, y, ldy, 0, (const bf16*)bias, act, act_arg};
  if (M <= 16) rows_go<1>(a, st);
  else rows_go<2>(a, st);
  VY_CHECK_LAUNCH("vy_rows_linear");
  return VY_OK;
}
