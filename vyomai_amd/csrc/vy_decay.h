// Shared by the linear attentions whose only memory of the past is an fp32 state S (one dk x dv matrix per head and sequence):
// vy_lightning.hip (a constant decay per head) and vy_gated.hip (a forget gate per key channel, GATED).  The arguments, the
// token-by-token recurrence, the scan of the chunked form along the chunks, and the fragments' helpers.
#pragma once
#include "vy_common.h"

namespace vy_decay {

constexpr int C = VY_DECAY_CHUNK;

struct DecayArgs {
  const void* p; int64_t ldp; int64_t oq, ok, ov;
  float* state; const float* pow;          // [slot][h][dk][dv]; [h][C + 1]
  const int* slots; const int* start; const int* count;
  void* out; int64_t ldo;
  int B, L, h, dk, dv, silu, nc;
  float* U;                                // [B * h][nc][dk][dv]
  const float2* rope; int half, rope_len;  // half = 0: no rotation; pairs of neighbouring columns
  float k_scale;
  const float* f_bias; const float* f_lower;   // GATED: [h][dk] (f_bias nullable); the gate's logits lie in the place of k
  float* D;                                    // GATED: decay of a whole chunk, [B * h][nc][dk]
};

// forget gate f = lower + (1 - lower) sigmoid(z) and what it lets in, k = 1 - f = (1 - lower) sigmoid(-z)
__device__ __forceinline__ void forget_gate(float z, float lower, float& f, float& k) {
  const float e = expf(-fabsf(z)), big = 1.f / (1.f + e), small = e * big;
  f = fmaf(1.f - lower, z >= 0.f ? big : small, lower);
  k = (1.f - lower) * (z >= 0.f ? small : big);
}

// (cos, sin) of the first pair of a token's row of the table (clamped: padding rows only)
__device__ __forceinline__ const float2* trig_row(const DecayArgs& a, int pos) {
  return a.rope + (int64_t)(pos < a.rope_len ? pos : a.rope_len - 1) * a.half;
}
// N consecutive columns d0 .. (both even) of a row
template <int N>
__device__ __forceinline__ void rotate(const float2* trig, int half, int d0, float (&v)[N]) {
  if (d0 + N <= 2 * half && (half & 1) == 0 && N % 4 == 0) {   // whole 16-byte pieces of the table's row
#pragma unroll
    for (int e = 0; e < N; e += 4) {
      const f32x4 cs = *reinterpret_cast<const f32x4*>(trig + ((d0 + e) >> 1));
      const float u = v[e], w = v[e + 1], x = v[e + 2], y = v[e + 3];
      v[e] = u * cs[0] - w * cs[1];
      v[e + 1] = w * cs[0] + u * cs[1];
      v[e + 2] = x * cs[2] - y * cs[3];
      v[e + 3] = y * cs[2] + x * cs[3];
    }
    return;
  }
#pragma unroll
  for (int e = 0; e < N; e += 2) {
    const int i = (d0 + e) >> 1;
    if (i < half) {
      const float2 cs = trig[i];
      const float u = v[e], w = v[e + 1];
      v[e] = u * cs.x - w * cs.y;
      v[e + 1] = w * cs.x + u * cs.y;
    }
  }
}

__device__ __forceinline__ float activate(float x, int silu) { return silu ? vy_silu(x) : x; }
__device__ __forceinline__ void split_bf16(float x, bf16& hi, bf16& lo) {
  const float h = vy_round_bf16(x);
  hi = (bf16)h;
  lo = (bf16)(x - h);
}

// ---- recurrence ------------------------------------------------------------------------------
// workgroup = COLS value columns of one (b, head); thread (rg, col) keeps rows rg, rg + RG, ... of the state column.
// TT tokens are staged at a time; the RG partial dot products of an output are added after each stage.
template <typename T, int COLS, int RPT, int TT, bool GATED>
__global__ __launch_bounds__(256) void decay_recurrent_kernel(DecayArgs a) {
  constexpr int RG = 256 / COLS, DK = RG * RPT;
  __shared__ float qs[TT][DK], ks[TT][DK], fs[GATED ? TT : 1][DK];
  __shared__ float vs[TT][COLS];
  __shared__ float red[TT][RG][COLS + 1];
  const int col = threadIdx.x % COLS, rg = threadIdx.x / COLS;
  const int head = blockIdx.y, b = blockIdx.z;
  const int c0 = (int)blockIdx.x * COLS, vc = c0 + col;
  const int slot = a.slots ? a.slots[b] : b;
  const int n = a.count ? min(a.count[b], a.L) : a.L;
  const float decay = GATED ? 0.f : a.pow[(int64_t)head * (C + 1) + 1];
  float* S = a.state + ((int64_t)slot * a.h + head) * a.dk * a.dv;
  float s[RPT];
  const int first = a.start[slot];
  const bool fresh = first == 0;
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg + RG * i;
    s[i] = r < a.dk && vc < a.dv ? S[(int64_t)r * a.dv + vc] : 0.f;
  }
  const T* P = (const T*)a.p + (int64_t)b * a.L * a.ldp;
  T* O = (T*)a.out + (int64_t)b * a.L * a.ldo + head * a.dv;
  for (int t0 = 0; t0 < n; t0 += TT) {
    const int m = min(TT, n - t0);
    for (int i = threadIdx.x; i < m * DK; i += 256) {
      const int t = i / DK, d = i % DK;
      const T* row = P + (int64_t)(t0 + t) * a.ldp + head * a.dk + d;
      const bool ok = d < a.dk;
      if constexpr (GATED) {
        float f = 1.f, k = 0.f;
        if (ok) {
          const int64_t at = (int64_t)head * a.dk + d;
          forget_gate(VyT<T>::ld(row + a.ok) + (a.f_bias ? a.f_bias[at] : 0.f), a.f_lower[at], f, k);
        }
        qs[t][d] = ok ? activate(VyT<T>::ld(row + a.oq), a.silu) : 0.f;
        fs[t][d] = f;
        ks[t][d] = k;
        continue;
      }
      float q = ok ? activate(VyT<T>::ld(row + a.oq), a.silu) : 0.f;
      float k = ok ? activate(VyT<T>::ld(row + a.ok), a.silu) : 0.f;
      if (d < 2 * a.half) {
        const int to = d & 1 ? -1 : 1;   // the other column of the pair
        const float2 cs = trig_row(a, first + t0 + t)[d >> 1];
        const float s = d & 1 ? cs.y : -cs.y;
        q = q * cs.x + activate(VyT<T>::ld(row + a.oq + to), a.silu) * s;
        k = k * cs.x + activate(VyT<T>::ld(row + a.ok + to), a.silu) * s;
      }
      qs[t][d] = q;
      ks[t][d] = k * a.k_scale;
    }
    for (int i = threadIdx.x; i < m * COLS; i += 256) {
      const int t = i / COLS, d = c0 + i % COLS;
      vs[t][i % COLS] = d < a.dv ? activate(VyT<T>::ld(P + (int64_t)(t0 + t) * a.ldp + a.ov + head * a.dv + d), GATED ? 0 : a.silu) : 0.f;
    }
    __syncthreads();
    for (int t = 0; t < m; ++t) {
      const float v = vs[t][col];
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < RPT; ++i) {
        const float before = fresh && t0 + t == 0 ? 0.f : s[i];   // an empty slot's state is zero, whatever lies there
        s[i] = fmaf(GATED ? fs[t][rg + RG * i] : decay, before, ks[t][rg + RG * i] * v);
        o = fmaf(s[i], qs[t][rg + RG * i], o);
      }
      red[t][rg][col] = o;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < m * COLS; i += 256) {
      const int t = i / COLS, cc = i % COLS;
      float o = 0.f;
#pragma unroll
      for (int r = 0; r < RG; ++r) o += red[t][r][cc];
      if (c0 + cc < a.dv) VyT<T>::st(O + (int64_t)(t0 + t) * a.ldo + c0 + cc, o);
    }
  }
  // the padding behind a short sequence: finite values for whatever reads whole batches
  for (int64_t t = n + rg; t < a.L; t += RG)
    if (vc < a.dv) VyT<T>::st(O + t * a.ldo + vc, 0.f);
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg + RG * i;
    if (r < a.dk && vc < a.dv) S[(int64_t)r * a.dv + vc] = s[i];
  }
}

// ---- chunked form ----------------------------------------------------------------------------
__device__ __forceinline__ bf16x8 load8(const bf16* p, bool ok, int silu) {
  bf16x8 r = {};
  if (ok) {
    r = *reinterpret_cast<const bf16x8*>(p);
    if (silu) {
#pragma unroll
      for (int e = 0; e < 8; ++e) r[e] = (bf16)vy_silu((float)r[e]);
    }
  }
  return r;
}

// fragment of a transposed operand: 16 columns (block n) x 32 rows (block tt) of a row-major LDS tile
template <int OFF>
__device__ __forceinline__ bf16x8 tr_frag(unsigned lane_addr, int pitch) {
  union { struct { s16x4 a, b; } s; bf16x8 v; } u;
  u.s.a = vy_lds_tr16_off<OFF>(lane_addr);
  u.s.b = vy_lds_tr16_off<OFF>(lane_addr + 16 * pitch);
  return u.v;
}

// S_c as hi / lo quads in place of the four floats of U_c: one 16-byte element per thread and chunk
template <bool GATED>
__global__ __launch_bounds__(256) void chunk_scan_kernel(DecayArgs a) {
  const int bh = blockIdx.y, b = bh / a.h, head = bh - b * a.h;
  const int64_t elems = (int64_t)a.dk * a.dv;
  const int64_t e0 = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (e0 >= elems) return;
  const int slot = a.slots ? a.slots[b] : b;
  const int n = a.count ? min(a.count[b], a.L) : a.L;
  const float* pw = GATED ? a.D + (int64_t)bh * a.nc * a.dk + e0 / a.dv : a.pow + (int64_t)head * (C + 1);   // (dv % 4 == 0: one row)
  float* S = a.state + ((int64_t)slot * a.h + head) * elems + e0;
  float* U = a.U + (int64_t)bh * a.nc * elems + e0;
  f32x4 s = {0.f, 0.f, 0.f, 0.f};
  if (a.start[slot] != 0) s = *reinterpret_cast<const f32x4*>(S);
  const float full = GATED ? 0.f : pw[C];
  constexpr int UN = 4;                       // chunks per batch of loads; the next batch is requested before this one is used
  f32x4 u[UN], nx[UN];
  float dc[UN], dn[UN];
  auto fetch = [&](int c0, f32x4 (&r)[UN], float (&d)[UN]) {
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      r[i] = *reinterpret_cast<const f32x4*>(U + min(c0 + i, a.nc - 1) * elems);
      if constexpr (GATED) d[i] = pw[(int64_t)min(c0 + i, a.nc - 1) * a.dk];
    }
  };
  fetch(0, u, dc);
  for (int c0 = 0; c0 < a.nc; c0 += UN) {
    if (c0 + UN < a.nc) fetch(c0 + UN, nx, dn);
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      if (c0 + i >= a.nc) break;
      union { struct { bf16x4 hi, lo; } h; f32x4 f; } w;
#pragma unroll
      for (int e = 0; e < 4; ++e) { bf16 x, y; split_bf16(s[e], x, y); w.h.hi[e] = x; w.h.lo[e] = y; }
      *reinterpret_cast<f32x4*>(U + (c0 + i) * elems) = w.f;
      const int m = max(0, min(C, n - (c0 + i) * C));
      const float d = GATED ? dc[i] : m == C ? full : pw[m];
#pragma unroll
      for (int e = 0; e < 4; ++e) s[e] = fmaf(d, s[e], u[i][e]);
    }
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      u[i] = nx[i];
      if constexpr (GATED) dc[i] = dn[i];
    }
  }
  *reinterpret_cast<f32x4*>(S) = s;
}

inline bool chunked(int64_t L, int dk, int dtype) { return dtype == VY_BF16 && L > 1 && dk <= 128; }

template <typename T, bool GATED>
int recurrent_go(const DecayArgs& a, hipStream_t st) {
  const dim3 grid((unsigned)vy_cdiv(a.dv, 16), a.h, a.B), block(256);
  if (a.L == 1) {
    // a decode step streams the state: whole 256-byte row pieces where enough workgroups remain, else narrow columns
    const int64_t wide = vy_cdiv(a.dv, 64) * a.h * a.B;
    const dim3 wgrid((unsigned)vy_cdiv(a.dv, 64), a.h, a.B);
    if (wide >= 512 && a.dk <= 64) hipLaunchKernelGGL((decay_recurrent_kernel<T, 64, 16, 1, GATED>), wgrid, block, 0, st, a);
    else if (wide >= 512 && a.dk <= 128) hipLaunchKernelGGL((decay_recurrent_kernel<T, 64, 32, 1, GATED>), wgrid, block, 0, st, a);
    else if (a.dk <= 64) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 4, 1, GATED>), grid, block, 0, st, a);
    else if (a.dk <= 128) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 8, 1, GATED>), grid, block, 0, st, a);
    else if (a.dk <= 256) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 16, 1, GATED>), grid, block, 0, st, a);
    else if (a.dk <= 512) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 32, 1, GATED>), grid, block, 0, st, a);
    else return 1;
    return 0;
  }
  if (a.dk <= 64) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 4, 16, GATED>), grid, block, 0, st, a);
  else if (a.dk <= 128) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 8, 16, GATED>), grid, block, 0, st, a);
  else if (a.dk <= 256) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 16, 8, GATED>), grid, block, 0, st, a);
  else if (a.dk <= 512) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 32, 8, GATED>), grid, block, 0, st, a);
  else return 1;
  return 0;
}

}  // namespace vy_decay
