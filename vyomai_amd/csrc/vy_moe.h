// Mixture of experts, the device code of decode steps: the choice of a token's experts and the weight-streaming products of few
// tokens.  Used by vy_moe.hip (launches of their own), vy_parallel.hip and vy_route.hip (one launch with other work of the same step).
#pragma once
#include "vy_rows.h"
#include <float.h>

namespace vy_moe_dev {

constexpr int MAX_E = 1024, MAX_ENTRIES = 1024;

struct ChooseArgs {
  const float* logits; int64_t M;
  int E, top, groups, keep;
  int sigmoid, best, normalize;       // scores sigmoid or softmax; largest scores summed for a group's (1 or 2)
  float scale;
  const int* count; int L;            // tokens l >= count[b] of a sequence are padding: no expert
  int* ids; float* weight;            // [M][top]; id -1: none
  int* pos;                           // nullable: choice -> its row where rows lie in the order of the choices
  int* counts; int* rank;             // nullable: tokens per expert (zeroed by the caller), a choice's rank among its expert's
};

__device__ __forceinline__ unsigned ordered(float z) {
  const unsigned u = __builtin_bit_cast(unsigned, z);
  return u & 0x80000000u ? ~u : u | 0x80000000u;
}

// one wave per token; lane holds experts lane + 64 i.  Both scores are monotone: the choice is made on the logits (of groups only
// if a group's score is its best expert's).  logits: the token's, in global memory or
// LDS; gmax: 2 * 64 EPL floats of LDS of the wave's own
template <int EPL>
__device__ __forceinline__ void choose_one(const ChooseArgs& a, int64_t m, const float* logits, int lane, float* gmax, int (&my_id),
                                           float (&my_w)) {
  my_id = -1;
  my_w = 0.f;
  const int b = a.count ? (int)(m / a.L) : 0;
  if (a.count && (int)(m - (int64_t)b * a.L) >= a.count[b]) return;
  float z[EPL], zmax = -INFINITY;
#pragma unroll
  for (int i = 0; i < EPL; ++i) {
    const int e = lane + 64 * i;
    z[i] = e < a.E ? logits[e] : -INFINITY;
    zmax = fmaxf(zmax, z[i]);
  }
  float sum = 1.f;
  if (!a.sigmoid) {
    zmax = vy_wave_max(zmax);
    sum = 0.f;
#pragma unroll
    for (int i = 0; i < EPL; ++i) sum += expf(z[i] - zmax);   // (exp(-inf) = 0 behind the last expert)
    sum = vy_wave_sum(sum);
  }
  auto score = [&](float x) { return a.sigmoid ? 1.f / (1.f + expf(-x)) : expf(x - zmax) / sum; };
  unsigned key[EPL];
#pragma unroll
  for (int i = 0; i < EPL; ++i) key[i] = lane + 64 * i < a.E ? ordered(z[i]) : 0u;
  if (a.keep < a.groups) {
    // a group stays if fewer than `keep` others are better (ties: the earlier one)
    const int size = a.E / a.groups;
    float* zs = gmax + 64 * EPL;
#pragma unroll
    for (int i = 0; i < EPL; ++i)
      if (lane + 64 * i < a.E) zs[lane + 64 * i] = a.best == 1 ? z[i] : score(z[i]);
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    for (int g = lane; g < a.groups; g += 64) {
      float best = -INFINITY, second = -INFINITY;
      for (int j = 0; j < size; ++j) {
        const float s = zs[g * size + j];
        second = fmaxf(second, fminf(best, s));
        best = fmaxf(best, s);
      }
      gmax[g] = a.best == 1 || size == 1 ? best : best + second;
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
#pragma unroll
    for (int i = 0; i < EPL; ++i) {
      const int e = lane + 64 * i;
      if (e < a.E) {
        const int g = e / size;
        const float mine = gmax[g];
        int better = 0;
        for (int j = 0; j < a.groups; ++j) better += gmax[j] > mine || (gmax[j] == mine && j < g);
        if (better >= a.keep) key[i] = 0u;
      }
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  }
  float total = 0.f;
  for (int k = 0; k < a.top; ++k) {
    // best remaining key, the lower expert of equal ones
    unsigned bk = 0u;
    int be = MAX_E;
#pragma unroll
    for (int i = 0; i < EPL; ++i)
      if (key[i] > bk) { bk = key[i]; be = lane + 64 * i; }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const unsigned ok = (unsigned)__shfl_xor((int)bk, o, 64);
      const int oe = __shfl_xor(be, o, 64);
      if (ok > bk || (ok == bk && oe < be)) { bk = ok; be = oe; }
    }
    if (bk == 0u) break;
    float ze = 0.f;
#pragma unroll
    for (int i = 0; i < EPL; ++i)
      if (lane + 64 * i == be) { ze = z[i]; key[i] = 0u; }
    ze = __shfl(ze, be & 63, 64);
    const float s = score(ze);
    total += s;
    if (lane == k) { my_id = be; my_w = s; }
  }
  my_w = (a.normalize ? my_w / (total + 1e-20f) : my_w) * a.scale;
}

// what an expert product does with its rows
constexpr int DOWN = 0;      // rows by choice in and out
constexpr int GATE_UP = 1;   // rows by token in, pairs of neighbouring results -> clamped gated activation
constexpr int UP = 2;        // rows by token in, exact GELU

__device__ __forceinline__ float clamped_act(float g, float u, float limit, float alpha) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * vy_sigmoid(alpha * g) * (u + 1.f);
}

// ---- the experts, few tokens ------------------------------------------------------------------
struct ExpertRows {
  const bf16* x; int64_t ldx;          // DOWN: activation rows by choice; else rows of h by token
  const int* ids; int n, top;          // n = tokens * top choices
  const bf16* w; int N, K;             // [E][N][K]
  bf16* y; int64_t ldy;                // rows by choice
  float limit, alpha;
};

template <int NT> struct ExpertLds {
  unsigned used[MAX_E / 32];
  int who, found, list[MAX_ENTRIES];
  f32x4 red[vy_rows::RED<NT, 1>];
};

// The y-th expert in use (in order of its number; of a single token: its y-th choice) x 16 NT weight rows.
template <int KIND, int NT>
__device__ __forceinline__ void expert_rows(const ExpertRows& a, ExpertLds<NT>& lds, int x, int y) {
  const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, kq = lane >> 4;
  int e, cnt;
  if (a.n == a.top) {
    e = a.ids[y];
    cnt = 1;
    if (e < 0) return;
  } else {
    if (tid < MAX_E / 32) lds.used[tid] = 0u;
    if (tid == 0) { lds.who = -1; lds.found = 0; }
    __syncthreads();
    for (int i = tid; i < a.n; i += 256) {
      const int id = a.ids[i];
      if (id >= 0) atomicOr(&lds.used[id >> 5], 1u << (id & 31));
    }
    __syncthreads();
    if (tid < 32) {
      const unsigned bits = lds.used[tid];
      int before = __popc(bits);
#pragma unroll
      for (int o = 1; o < 32; o <<= 1) {
        const int v = __shfl_up(before, o, 32);
        if (lane >= o) before += v;
      }
      before -= __popc(bits);
      int want = y - before;
      if (want >= 0 && want < __popc(bits)) {
        unsigned rest = bits;
        while (want--) rest &= rest - 1;
        lds.who = tid * 32 + __ffs((int)rest) - 1;
      }
    }
    __syncthreads();
    e = lds.who;
    if (e < 0) return;
    for (int i = tid; i < a.n; i += 256)
      if (a.ids[i] == e) lds.list[atomicAdd(&lds.found, 1)] = i;   // (any order: rows do not touch each other)
    __syncthreads();
    cnt = lds.found;
  }
  const int n0 = x * 16 * NT;
  const bf16* ws[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) ws[t] = a.w + ((int64_t)e * a.N + min(n0 + 16 * t + r16, a.N - 1)) * a.K + 8 * kq;
  for (int m0 = 0; m0 < cnt; m0 += 16) {
    const int mine = a.n == a.top ? y : lds.list[m0 + r16 < cnt ? m0 + r16 : cnt - 1];
    const bf16* xs[1] = {a.x + (int64_t)(KIND != DOWN ? mine / a.top : mine) * a.ldx + 8 * kq};
    f32x4 acc[NT][1];
    vy_rows::stream<NT, 1>(ws, xs, a.K, acc, lds.red);
    if (tid < 64 && m0 + r16 < cnt) {
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const f32x4 v = acc[t][0];
        const int n = n0 + 16 * t + 4 * kq;
        if (n < a.N) {
          bf16* yr = a.y + (int64_t)mine * a.ldy;
          if constexpr (KIND == GATE_UP) {
            bf16x2 w2;
            w2[0] = (bf16)clamped_act(v[0], v[1], a.limit, a.alpha);
            w2[1] = (bf16)clamped_act(v[2], v[3], a.limit, a.alpha);
            *reinterpret_cast<bf16x2*>(yr + n / 2) = w2;
          } else {
            bf16x4 w4;
#pragma unroll
            for (int r = 0; r < 4; ++r) w4[r] = (bf16)(KIND == UP ? vy_gelu_erf_fast(v[r]) : v[r]);
            *reinterpret_cast<bf16x4*>(yr + n) = w4;
          }
        }
      }
    }
  }
}

// a single token: its y-th choice x 8 weight rows (GATE_UP: 4 pairs)
template <int KIND>
__device__ __forceinline__ void expert_rows1(const ExpertRows& a, int x, int y) {
  const int e = a.ids[y], n = 8 * x + 2 * (threadIdx.x >> 6);
  if (e < 0 || n >= a.N) return;   // (N is a multiple of 8)
  const bf16* w = a.w + ((int64_t)e * a.N + n) * a.K;
  float s0, s1;
  vy_rows::gemv2(w, w + a.K, a.x + (KIND != DOWN ? 0 : (int64_t)y * a.ldx), a.K, s0, s1);
  if (threadIdx.x & 63) return;
  bf16* yr = a.y + (int64_t)y * a.ldy;
  if constexpr (KIND == GATE_UP) {
    yr[n / 2] = (bf16)clamped_act(s0, s1, a.limit, a.alpha);
  } else if constexpr (KIND == UP) {
    yr[n] = (bf16)vy_gelu_erf_fast(s0);
    yr[n + 1] = (bf16)vy_gelu_erf_fast(s1);
  } else {
    yr[n] = (bf16)s0;
    yr[n + 1] = (bf16)s1;
  }
}

}  // namespace vy_moe_dev
