// Weight-streaming products of few rows (decode): a workgroup of four waves takes 16 NT rows of W [N][K] against 16 MB rows of X
// on mfma_f32_16x16x32_bf16 (A = weight rows, B = rows of X), both straight from memory into operand registers: a weight is used
// once, and X is small enough for L2.  The waves split K by whole 128-byte lines (two k-steps of 32); every wave requests its
// loads of up to STEPS k-steps before the first product, so a pass over K = 128 STEPS costs one memory latency.  W is streamed
// past the caches (non-temporal) unless other workgroups read it too.
#pragma once
#include "vy_common.h"

namespace vy_rows {

template <int NT, int MB> constexpr int RED = 3 * NT * MB * 64;   // f32x4 of LDS that stream() needs
template <int NT, int MB> constexpr int STEPS = NT * MB == 1 ? 16 : NT + MB <= 3 ? 8 : 4;

// acc[t][j] (in wave 0 only) = 16 rows ws[t] x 16 rows xs[j]; a lane's pointers are its row (lane & 15) + 8 (lane >> 4).
// D: a lane owns row lane & 15 of X and rows 4 (lane >> 4) .. + 3 of W.
template <int NT, int MB, bool ONCE = true>
__device__ __forceinline__ void stream(const bf16* const (&ws)[NT], const bf16* const (&xs)[MB], int K, f32x4 (&acc)[NT][MB],
                                       f32x4* red) {
  constexpr int U = STEPS<NT, MB>;
  const int lane = threadIdx.x & 63, kq = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const bf16x8 zero8 = {(bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f};
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int j = 0; j < MB; ++j) acc[t][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 64 * wave; k0 < K; k0 += 128 * U) {
    bf16x8 w[U][NT], x[U][MB];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + 256 * (u >> 1) + 32 * (u & 1);
      const bool in = k + 8 * kq < K;
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const bf16x8* at = reinterpret_cast<const bf16x8*>(ws[t] + k);
        if constexpr (ONCE) w[u][t] = in ? __builtin_nontemporal_load(at) : zero8;
        else w[u][t] = in ? *at : zero8;
      }
#pragma unroll
      for (int j = 0; j < MB; ++j) x[u][j] = in ? *reinterpret_cast<const bf16x8*>(xs[j] + k) : zero8;
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int j = 0; j < MB; ++j) acc[t][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[u][t], x[u][j], acc[t][j], 0, 0, 0);
  }
  __syncthreads();   // (red may still be read from the pass before)
  if (wave)
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int j = 0; j < MB; ++j) red[((wave - 1) * NT * MB + t * MB + j) * 64 + lane] = acc[t][j];
  __syncthreads();
  if (wave == 0)
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int j = 0; j < MB; ++j)
#pragma unroll
        for (int s = 0; s < 3; ++s) {
          const f32x4 v = red[(s * NT * MB + t * MB + j) * 64 + lane];
#pragma unroll
          for (int r = 0; r < 4; ++r) acc[t][j][r] += v[r];
        }
}

struct Dense {
  const bf16* x; int64_t ldx; int M;   // M <= 16 MB
  const bf16* w; int N, K;             // [N][K]
  void* y; int64_t ldy; int f32;       // f32: fp32 results
};

// rows 16 tile .. + 15 of W against all of X
template <int MB>
__device__ __forceinline__ void dense(const Dense& a, f32x4* red, int tile) {
  const int lane = threadIdx.x & 63, r16 = lane & 15, kq = lane >> 4;
  const bf16* ws[1] = {a.w + (int64_t)min(16 * tile + r16, a.N - 1) * a.K + 8 * kq};
  const bf16* xs[MB];
#pragma unroll
  for (int j = 0; j < MB; ++j) xs[j] = a.x + (int64_t)min(16 * j + r16, a.M - 1) * a.ldx + 8 * kq;
  f32x4 acc[1][MB];
  stream<1, MB>(ws, xs, a.K, acc, red);
  if (threadIdx.x >= 64) return;
  const int n = 16 * tile + 4 * kq;
#pragma unroll
  for (int j = 0; j < MB; ++j) {
    const int m = 16 * j + r16;
    if (m >= a.M) continue;
    const f32x4 v = acc[0][j];
    if (a.f32) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (n + r < a.N) ((float*)a.y)[(int64_t)m * a.ldy + n + r] = v[r];
    } else if (n + 4 <= a.N) {
      bf16x4 w4;
#pragma unroll
      for (int r = 0; r < 4; ++r) w4[r] = (bf16)v[r];
      *reinterpret_cast<bf16x4*>((bf16*)a.y + (int64_t)m * a.ldy + n) = w4;
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (n + r < a.N) ((bf16*)a.y)[(int64_t)m * a.ldy + n + r] = (bf16)v[r];
    }
  }
}

}  // namespace vy_rows
