// Weight-streaming products of few rows (decode): a workgroup of NW = 4 (or 8) waves takes 16 NT rows of W [N][K] against 16 MB rows of X
// on mfma_f32_16x16x32_bf16 (A = weight rows, B = rows of X), both straight from memory into operand registers: a weight is used
// once, and X is small enough for L2.  The waves split K by whole 128-byte lines (two k-steps of 32); every wave requests its
// loads of up to STEPS k-steps before the first product, so a pass over K = 32 NW STEPS costs one memory latency.  W is streamed
// past the caches (non-temporal) unless other workgroups read it too.
#pragma once
#include "vy_common.h"

namespace vy_rows {

template <int NT, int MB, int NW = 4> constexpr int RED = (NW - 1) * NT * MB * 64;   // f32x4 of LDS that stream() needs
template <int NT, int MB> constexpr int STEPS = NT * MB == 1 ? 16 : NT + MB <= 3 ? 8 : 4;

// acc[t][j] (in wave 0 only) = 16 rows ws[t] x 16 rows xs[j]; a lane's pointers are its row (lane & 15) + 8 (lane >> 4).
// D: a lane owns row lane & 15 of X and rows 4 (lane >> 4) .. + 3 of W.
template <int NT, int MB, bool ONCE = true, int NW = 4>
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
  for (int k0 = 64 * wave; k0 < K; k0 += 32 * NW * U) {
    bf16x8 w[U][NT], x[U][MB];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + 64 * NW * (u >> 1) + 32 * (u & 1);
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
        for (int s = 0; s < NW - 1; ++s) {
          const f32x4 v = red[(s * NT * MB + t * MB + j) * 64 + lane];
#pragma unroll
          for (int r = 0; r < 4; ++r) acc[t][j][r] += v[r];
        }
}

struct Dense {
  const bf16* x; int64_t ldx; int M;   // M <= 16 MB
  const bf16* w; int N, K;             // [N][K]
  void* y; int64_t ldy; int f32;       // f32: fp32 results
  const bf16* bias; int act; float act_arg;   // of bf16 results: act(x W^T + bias), act none, VY_ACT_RELU2 or VY_ACT_SOFTCAP
};

__device__ __forceinline__ float finish(const Dense& a, float v, int n) {
  if (a.bias) v += (float)a.bias[n];
  if (a.act == VY_ACT_RELU2) v = vy_act_fwd<VY_ACT_RELU2>(v);
  else if (a.act == VY_ACT_SOFTCAP) v = vy_act_fwd<VY_ACT_SOFTCAP>(v, a.act_arg);
  return v;
}

// rows 16 NT tile .. + 16 NT - 1 of W against all of X
template <int MB, int NW = 4, int NT = 1>
__device__ __forceinline__ void dense(const Dense& a, f32x4* red, int tile) {
  const int lane = threadIdx.x & 63, r16 = lane & 15, kq = lane >> 4;
  const bf16* ws[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) ws[t] = a.w + (int64_t)min(16 * (NT * tile + t) + r16, a.N - 1) * a.K + 8 * kq;
  const bf16* xs[MB];
#pragma unroll
  for (int j = 0; j < MB; ++j) xs[j] = a.x + (int64_t)min(16 * j + r16, a.M - 1) * a.ldx + 8 * kq;
  f32x4 acc[NT][MB];
  stream<NT, MB, true, NW>(ws, xs, a.K, acc, red);
  if (threadIdx.x >= 64) return;
#pragma unroll
  for (int i = 0; i < NT * MB; ++i) {
    const int m = 16 * (i % MB) + r16, n = 16 * (NT * tile + i / MB) + 4 * kq;
    if (m >= a.M) continue;
    const f32x4 v = acc[i / MB][i % MB];
    if (a.f32) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (n + r < a.N) ((float*)a.y)[(int64_t)m * a.ldy + n + r] = v[r];
    } else if (n + 4 <= a.N) {
      bf16x4 w4;
#pragma unroll
      for (int r = 0; r < 4; ++r) w4[r] = (bf16)finish(a, v[r], n + r);
      *reinterpret_cast<bf16x4*>((bf16*)a.y + (int64_t)m * a.ldy + n) = w4;
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (n + r < a.N) ((bf16*)a.y)[(int64_t)m * a.ldy + n + r] = (bf16)finish(a, v[r], n + r);
    }
  }
}

// ---- one row of X: a wave per two weight rows ---------------------------------------------------
// Whole 1 KiB pieces of a row per instruction and no sharing between waves: many small, even pieces of work, which a single
// token's stream needs to reach every CU equally (16-row tiles leave some with half as much again as others).
__device__ __forceinline__ float dot8(const bf16x8 a, const bf16x8 b, float s) {
#pragma unroll
  for (int i = 0; i < 8; i += 2) s = __builtin_amdgcn_fdot2_f32_bf16(bf16x2{a[i], a[i + 1]}, bf16x2{b[i], b[i + 1]}, s, false);
  return s;
}
__device__ __forceinline__ void gemv2(const bf16* w0, const bf16* w1, const bf16* x, int K, float& s0, float& s1) {
  constexpr int U = 4;
  const int lane = threadIdx.x & 63;
  s0 = s1 = 0.f;
  int k = lane * 8;
  for (; k - lane * 8 + 512 * U <= K; k += 512 * U) {   // (wave-uniform)
    bf16x8 a[U], b[U], v[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      a[u] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(w0 + k + 512 * u));
      b[u] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(w1 + k + 512 * u));
    }
#pragma unroll
    for (int u = 0; u < U; ++u) v[u] = *reinterpret_cast<const bf16x8*>(x + k + 512 * u);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      s0 = dot8(a[u], v[u], s0);
      s1 = dot8(b[u], v[u], s1);
    }
  }
#pragma unroll 2
  for (; k < K; k += 512) {
    const bf16x8 a = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(w0 + k));
    const bf16x8 b = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(w1 + k));
    const bf16x8 v = *reinterpret_cast<const bf16x8*>(x + k);
    s0 = dot8(a, v, s0);
    s1 = dot8(b, v, s1);
  }
  s0 = vy_wave_sum(s0);
  s1 = vy_wave_sum(s1);
}

// rows 8 tile .. + 7 of W against the one row of X
__device__ __forceinline__ void dense1(const Dense& a, int tile) {
  const int n = 8 * tile + 2 * (threadIdx.x >> 6);
  if (n >= a.N) return;
  const bf16* w = a.w + (int64_t)n * a.K;
  float s0, s1;
  gemv2(w, n + 1 < a.N ? w + a.K : w, a.x, a.K, s0, s1);
  if (threadIdx.x & 63) return;
  if (a.f32) {
    ((float*)a.y)[n] = s0;
    if (n + 1 < a.N) ((float*)a.y)[n + 1] = s1;
  } else {
    ((bf16*)a.y)[n] = (bf16)s0;
    if (n + 1 < a.N) ((bf16*)a.y)[n + 1] = (bf16)s1;
  }
}

}  // namespace vy_rows
