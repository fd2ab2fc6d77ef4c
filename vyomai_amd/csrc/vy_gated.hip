// Linear attention with a forget gate per key channel, tied to the input gate 1 - f (HGRN2):
//   f = lower + (1 - lower) sigmoid(z + bias),   S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T ,   o_t = S_t^T q_t ,   q = silu
//
// Two forms, as in vy_lightning.hip: the recurrence (vy_decay.h) for decode steps, fp32 models and wide keys, and chunks of
// C = 64 tokens on MFMA for bf16 prompts, in three launches:
//   gated_kv_kernel    U_c = sum_j (prod_{t > j} f_t) k_j v_j^T , D_c = prod f over chunk c, k = 1 - f          (all chunks at once)
//   chunk_scan_kernel  S_(c+1) = diag(D_c) S_c + U_c, leaves S_c where U_c was
//   gated_out_kernel   O = A V + (q prefix) S_c ,  A_ij = sum_d q_id k_jd prod_{j < t <= i} f_td  for j <= i      (all chunks at once)
//
// The gates depend on the channel, so A is no masked Q K^T.  A chunk is cut into four blocks of 16 tokens.  Between blocks the
// product of gates splits at block borders into (prefix inside the query's block) x (whole blocks between) x (suffix inside the
// key's block); each factor is at most 1, so nothing overflows however small a gate is, and A's block is an MFMA product of
// scaled queries and keys.  Inside a block each lane carries w_j = k_j prod f down the rows i (16 steps, fp32): no quotient,
// no logarithm and no exponential of a sum of logarithms appears anywhere.
//
// 32-bit: gates, their products, the state, A.  What enters MFMA is split into hi + lo bf16 (scaled q and k, A, S_c); only v, a
// projection, is plain bf16.
#include "vy_decay.h"

namespace {

using namespace vy_decay;

constexpr int BT = 16, NB = C / BT;     // tokens per block, blocks per chunk

// gates, written keys (and queries) of the 16 tokens of block s, channels c and c + 1
struct Gates { float f[BT][2], k[BT][2], q[BT][2]; };
template <bool Q>
__device__ __forceinline__ void load_gates(const DecayArgs& a, const bf16* P, int head, int s, int c, int m, Gates& g) {
  bf16x2 z[BT], q[BT];
  const bool in = c < a.dk;
  const int64_t at = (int64_t)head * a.dk + (in ? c : 0);
#pragma unroll
  for (int t = 0; t < BT; ++t) {
    z[t] = q[t] = bf16x2{(bf16)0.f, (bf16)0.f};
    if (in && BT * s + t < m) {
      const bf16* row = P + (int64_t)(BT * s + t) * a.ldp + at;
      z[t] = *reinterpret_cast<const bf16x2*>(row + a.ok);
      if constexpr (Q) q[t] = *reinterpret_cast<const bf16x2*>(row + a.oq);
    }
  }
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    const float b = a.f_bias ? a.f_bias[at + e] : 0.f, lower = a.f_lower[at + e];
#pragma unroll
    for (int t = 0; t < BT; ++t) {
      g.f[t][e] = 1.f;
      g.k[t][e] = 0.f;
      if (in && BT * s + t < m) forget_gate((float)z[t][e] + b, lower, g.f[t][e], g.k[t][e]);
      if constexpr (Q) g.q[t][e] = activate((float)q[t][e], a.silu);
    }
  }
}
__device__ __forceinline__ void store_split2(char* hi, char* lo, float x, float y) {
  bf16 h0, l0, h1, l1;
  split_bf16(x, h0, l0);
  split_bf16(y, h1, l1);
  *reinterpret_cast<bf16x2*>(hi) = bf16x2{h0, h1};
  *reinterpret_cast<bf16x2*>(lo) = bf16x2{l0, l1};
}

// grid (chunks, B * h)
template <int DKP>
__global__ __launch_bounds__(256) void gated_kv_kernel(DecayArgs a) {
  constexpr int KP = (DKP + 8) * 2, VP = (64 + 8) * 2, PAIRS = DKP / 2, ITEMS = NB * PAIRS;
  __shared__ __attribute__((aligned(16))) char smem[C * (2 * KP + VP) + NB * DKP * 4];
  char* kh = smem;
  char* kl = smem + C * KP;
  char* vt = smem + 2 * C * KP;
  float* F = reinterpret_cast<float*>(vt + C * VP);    // [block][channel]: product of a block's gates
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r16 = lane & 15, kq = lane >> 4;
  const int ch = blockIdx.x, bh = blockIdx.y, b = bh / a.h, head = bh - b * a.h;
  const int n = a.count ? min(a.count[b], a.L) : a.L;
  const int m = max(0, min(C, n - ch * C));            // tokens of this chunk
  const bf16* P = (const bf16*)a.p + ((int64_t)b * a.L + ch * C) * a.ldp;
  const int it = threadIdx.x, s = it / PAIRS, c = (it % PAIRS) * 2;
  static_assert(ITEMS <= 256, "one item per thread");
  Gates g;
  bf16x8 v8[2];
  auto fetch = [&](int v0) {
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int x = threadIdx.x + 256 * i, t = x >> 3, d = (x & 7) * 8;
      v8[i] = load8(P + (int64_t)t * a.ldp + a.ov + head * a.dv + v0 + d, t < m && v0 + d < a.dv, 0);
    }
  };
  fetch(0);
  float sfx[2] = {1.f, 1.f};
  if (it < ITEMS) {
    load_gates<false>(a, P, head, s, c, m, g);
#pragma unroll
    for (int t = BT - 1; t >= 0; --t)
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        g.k[t][e] *= sfx[e];
        sfx[e] *= g.f[t][e];
      }
    F[s * DKP + c] = sfx[0];
    F[s * DKP + c + 1] = sfx[1];
  }
  __syncthreads();
  if (it < ITEMS) {
    float later[2] = {1.f, 1.f};
    for (int o = s + 1; o < NB; ++o) {
      later[0] *= F[o * DKP + c];
      later[1] *= F[o * DKP + c + 1];
    }
#pragma unroll
    for (int t = 0; t < BT; ++t) {
      const int at = (BT * s + t) * KP + c * 2;
      store_split2(kh + at, kl + at, g.k[t][0] * later[0], g.k[t][1] * later[1]);
    }
    if (s == 0 && c < a.dk) {
      float* D = a.D + ((int64_t)bh * a.nc + ch) * a.dk + c;
      D[0] = sfx[0] * later[0];
      D[1] = sfx[1] * later[1];
    }
  }
  float* U = a.U + ((int64_t)bh * a.nc + ch) * a.dk * a.dv;
  const int lr = 4 * kq + (r16 >> 2), lc = (4 * (r16 & 3)) * 2;
  const unsigned khb = vy_lds_addr(kh) + lr * KP + lc, klb = vy_lds_addr(kl) + lr * KP + lc, vb = vy_lds_addr(vt) + lr * VP + lc;
  for (int v0 = 0; v0 < a.dv; v0 += 64) {
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int x = threadIdx.x + 256 * i;
      *reinterpret_cast<bf16x8*>(vt + (x >> 3) * VP + (x & 7) * 16) = v8[i];
    }
    __syncthreads();
    if (v0 + 64 < a.dv) fetch(v0 + 64);
    for (int blk = wave; blk < DKP / 16; blk += 4) {      // 16 key rows of the state
      if (blk * 16 >= a.dk) break;
      f32x4 acc[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int tt = 0; tt < C / 32; ++tt) {
        bf16x8 fh = tr_frag<0>(khb + tt * 32 * KP + blk * 32, KP), fl = tr_frag<0>(klb + tt * 32 * KP + blk * 32, KP);
        bf16x8 fv[4];
        vy_static_for<4>([&](auto i_c) {
          constexpr int i = decltype(i_c)::value;
          fv[i] = tr_frag<i * 32>(vb + tt * 32 * VP, VP);
        });
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        vy_tie(fh);
        vy_tie(fl);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          vy_tie(fv[i]);
          acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fl, fv[i], acc[i], 0, 0, 0);
          acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fh, fv[i], acc[i], 0, 0, 0);
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int r = blk * 16 + 4 * kq + e, col = v0 + 16 * i + r16;
          if (r < a.dk && col < a.dv) U[(int64_t)r * a.dv + col] = acc[i][e];
        }
    }
    __syncthreads();   // the tile has been read
  }
}

// a lane of a wave (jp = lane & 7, dg = lane >> 3) holds 24 partial sums; the eight lanes of equal jp are added up and share them
// out: afterwards a[0 .. 2] are the sums of index 12 bit5 + 6 bit4 + 3 bit3 + 0 .. 2
__device__ __forceinline__ void share_out(float (&a)[24], int lane) {
  auto half = [&](auto n_c, int bit) {
    constexpr int N = decltype(n_c)::value;
    const bool up = lane & bit;
#pragma unroll
    for (int v = 0; v < N; ++v) {
      const float keep = up ? a[v + N] : a[v], send = up ? a[v] : a[v + N];
      a[v] = keep + __shfl_xor(send, bit, 64);
    }
  };
  half(std::integral_constant<int, 12>{}, 32);
  half(std::integral_constant<int, 6>{}, 16);
  half(std::integral_constant<int, 3>{}, 8);
}

// grid (chunks, B * h): wave w computes rows 16 w .. + 15 of the chunk, block w
template <int DKP>
__global__ __launch_bounds__(256, 1) void gated_out_kernel(DecayArgs a) {
  static_assert(NB == 4, "one block per wave");
  constexpr int KP = (DKP + 8) * 2, VP = (64 + 8) * 2, PAIRS = DKP / 2, ITEMS = NB * PAIRS;
  constexpr int KS = DKP / 32, QP = DKP + 4, AP = 20;   // QP, AP: pitches in floats
  constexpr int RAW = C * QP * 4;                       // bytes of an fp32 image
  constexpr int SN = DKP * 16 / 256;                    // quads of S per thread and value block
  static_assert(2 * DKP * VP + C * VP <= 2 * RAW, "the state and value tiles fit over the raw gates and keys");
  __shared__ __attribute__((aligned(16))) char smem[3 * RAW + 2 * C * KP + NB * BT * AP * 4 + NB * DKP * 4];
  float* qs = reinterpret_cast<float*>(smem);           // queries, then times their prefix
  float* fs = reinterpret_cast<float*>(smem + RAW);
  float* ks = reinterpret_cast<float*>(smem + 2 * RAW);
  char* kh = smem + 3 * RAW;                            // keys times their suffix, hi and lo
  char* kl = kh + C * KP;
  float* A = reinterpret_cast<float*>(kl + C * KP);     // [block][i][j] inside a block
  float* F = A + NB * BT * AP;                          // [block][channel]
  char* sh = smem + RAW;                                // over fs and ks: state tile hi, lo, value tile
  char* sl = sh + DKP * VP;
  char* vt = sl + DKP * VP;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r16 = lane & 15, kq = lane >> 4;
  const int ch = blockIdx.x, bh = blockIdx.y, b = bh / a.h, head = bh - b * a.h;
  const int n = a.count ? min(a.count[b], a.L) : a.L;
  const int m = max(0, min(C, n - ch * C)), rows = min(C, a.L - ch * C);
  const bf16* P = (const bf16*)a.p + ((int64_t)b * a.L + ch * C) * a.ldp;
  const float* Sg = a.U + ((int64_t)bh * a.nc + ch) * a.dk * a.dv;

  f32x4 s4[SN];
  bf16x8 v8[2];
  auto fetch = [&](int v0) {
#pragma unroll
    for (int i = 0; i < SN; ++i) {
      const int x = threadIdx.x + 256 * i, r = x >> 4, col = v0 + (x & 15) * 4;
      s4[i] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (r < a.dk && col < a.dv) s4[i] = *reinterpret_cast<const f32x4*>(Sg + (int64_t)r * a.dv + col);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int x = threadIdx.x + 256 * i, t = x >> 3, d = (x & 7) * 8;
      v8[i] = load8(P + (int64_t)t * a.ldp + a.ov + head * a.dv + v0 + d, t < m && v0 + d < a.dv, 0);
    }
  };
  // ---- gates, keys, queries
  const int it = threadIdx.x, s = it / PAIRS, c = (it % PAIRS) * 2;
  static_assert(ITEMS <= 256, "one item per thread");
  {
    Gates g;
    if (it < ITEMS) load_gates<true>(a, P, head, s, c, m, g);
    fetch(0);
    if (it < ITEMS) {
#pragma unroll
      for (int t = 0; t < BT; ++t) {
        const int at = (BT * s + t) * QP + c;
        *reinterpret_cast<float2*>(qs + at) = make_float2(g.q[t][0], g.q[t][1]);
        *reinterpret_cast<float2*>(fs + at) = make_float2(g.f[t][0], g.f[t][1]);
        *reinterpret_cast<float2*>(ks + at) = make_float2(g.k[t][0], g.k[t][1]);
      }
    }
  }
  __syncthreads();
  // ---- A inside the wave's block: lane (jp, dg) has keys jp and jp + 8, DKP / 8 channels
  {
    constexpr int DG = DKP / 8;
    const int jp = lane & 7, d0 = (lane >> 3) * DG;
    float k0[DG], k1[DG], w0[DG], w1[DG], part[24];
    auto row = [&](const float* p, int t, float (&v)[DG]) {
#pragma unroll
      for (int e = 0; e < DG; e += 4) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(p + (BT * wave + t) * QP + d0 + e);
#pragma unroll
        for (int i = 0; i < 4; ++i) v[e + i] = x[i];
      }
    };
    row(ks, jp, k0);
    row(ks, jp + 8, k1);
#pragma unroll
    for (int e = 0; e < DG; ++e) w0[e] = w1[e] = 0.f;
#pragma unroll
    for (int i = 0; i < BT; ++i) {
      float f[DG], q[DG], p0 = 0.f, p1 = 0.f;
      row(fs, i, f);
      row(qs, i, q);
#pragma unroll
      for (int e = 0; e < DG; ++e) {
        w0[e] *= f[e];
        if (i < 8) w0[e] = i == jp ? k0[e] : w0[e];
        p0 = fmaf(q[e], w0[e], p0);
        if (i >= 8) {
          w1[e] *= f[e];
          w1[e] = i - 8 == jp ? k1[e] : w1[e];
          p1 = fmaf(q[e], w1[e], p1);
        }
      }
      part[i] = p0;
      if (i >= 8) part[8 + i] = p1;
    }
    share_out(part, lane);
    const int first = (lane & 32 ? 12 : 0) + (lane & 16 ? 6 : 0) + (lane & 8 ? 3 : 0);
#pragma unroll
    for (int v = 0; v < 3; ++v) {
      const int x = first + v, i = x < 16 ? x : x - 8, j = x < 16 ? jp : jp + 8;
      A[(wave * BT + i) * AP + j] = part[v];
    }
  }
  __syncthreads();
  // ---- queries times their prefix, keys times their suffix, products of whole blocks
  if (it < ITEMS) {
    float2 f[BT];
    float p0 = 1.f, p1 = 1.f;
#pragma unroll
    for (int t = 0; t < BT; ++t) {
      const int at = (BT * s + t) * QP + c;
      f[t] = *reinterpret_cast<const float2*>(fs + at);
      float2 q = *reinterpret_cast<const float2*>(qs + at);
      p0 *= f[t].x;
      p1 *= f[t].y;
      *reinterpret_cast<float2*>(qs + at) = make_float2(q.x * p0, q.y * p1);
    }
    F[s * DKP + c] = p0;
    F[s * DKP + c + 1] = p1;
    float s0 = 1.f, s1 = 1.f;
#pragma unroll
    for (int t = BT - 1; t >= 0; --t) {
      const float2 k = *reinterpret_cast<const float2*>(ks + (BT * s + t) * QP + c);
      const int at = (BT * s + t) * KP + c * 2;
      store_split2(kh + at, kl + at, k.x * s0, k.y * s1);
      s0 *= f[t].x;
      s1 *= f[t].y;
    }
  }
  __syncthreads();
  // ---- A between blocks; the query operand takes in one block's gates after the other, at last the whole prefix of the chunk
  float qv[KS][8];
  bf16x8 qh[KS], ql[KS];
  auto split_q = [&]() {
#pragma unroll
    for (int k = 0; k < KS; ++k)
#pragma unroll
      for (int e = 0; e < 8; ++e) { bf16 x, y; split_bf16(qv[k][e], x, y); qh[k][e] = x; ql[k][e] = y; }
  };
#pragma unroll
  for (int k = 0; k < KS; ++k)
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(qs + (BT * wave + r16) * QP + 32 * k + 16 * hf + 4 * kq);
#pragma unroll
      for (int e = 0; e < 4; ++e) qv[k][4 * hf + e] = x[e];
    }
  f32x4 sc[NB];
#pragma unroll
  for (int J = 0; J < NB; ++J) sc[J] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int J = NB - 2; J >= 0; --J) {
    if (J < wave) {   // wave-uniform
      split_q();
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        union { struct { bf16x4 a, b; } h; bf16x8 v; } h8, l8;
        const int at = (BT * J + r16) * KP + (32 * k + 4 * kq) * 2;
        h8.h.a = *reinterpret_cast<const bf16x4*>(kh + at);
        h8.h.b = *reinterpret_cast<const bf16x4*>(kh + at + 32);
        l8.h.a = *reinterpret_cast<const bf16x4*>(kl + at);
        l8.h.b = *reinterpret_cast<const bf16x4*>(kl + at + 32);
        sc[J] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(l8.v, qh[k], sc[J], 0, 0, 0);
        sc[J] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(h8.v, ql[k], sc[J], 0, 0, 0);
        sc[J] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(h8.v, qh[k], sc[J], 0, 0, 0);
      }
#pragma unroll
      for (int k = 0; k < KS; ++k)
#pragma unroll
        for (int hf = 0; hf < 2; ++hf) {
          const f32x4 x = *reinterpret_cast<const f32x4*>(F + J * DKP + 32 * k + 16 * hf + 4 * kq);
#pragma unroll
          for (int e = 0; e < 4; ++e) qv[k][4 * hf + e] *= x[e];
        }
    }
  }
  split_q();
  const f32x4 own = *reinterpret_cast<const f32x4*>(A + (wave * BT + r16) * AP + 4 * kq);
  bf16x8 ph[NB / 2], pl[NB / 2];
#pragma unroll
  for (int J = 0; J < NB; ++J)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float inside = 4 * kq + r <= r16 ? own[r] : 0.f;
      bf16 x, y;
      split_bf16(J < wave ? sc[J][r] : J == wave ? inside : 0.f, x, y);
      ph[J >> 1][4 * (J & 1) + r] = x;
      pl[J >> 1][4 * (J & 1) + r] = y;
    }
  // ---- outputs, 64 value columns at a time
  const int qi = BT * wave + r16;
  const int lr = 4 * kq + (r16 >> 2), lc = (4 * (r16 & 3)) * 2;
  const unsigned shb = vy_lds_addr(sh) + lr * VP + lc, slb = vy_lds_addr(sl) + lr * VP + lc, vb = vy_lds_addr(vt) + lr * VP + lc;
  for (int v0 = 0; v0 < a.dv; v0 += 64) {
#pragma unroll
    for (int i = 0; i < SN; ++i) {
      const int x = threadIdx.x + 256 * i, at = (x >> 4) * VP + (x & 15) * 8;
      union { struct { bf16x4 hi, lo; } h; f32x4 f; } w;
      w.f = s4[i];
      *reinterpret_cast<bf16x4*>(sh + at) = w.h.hi;
      *reinterpret_cast<bf16x4*>(sl + at) = w.h.lo;
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int x = threadIdx.x + 256 * i;
      *reinterpret_cast<bf16x8*>(vt + (x >> 3) * VP + (x & 7) * 16) = v8[i];
    }
    __syncthreads();
    if (v0 + 64 < a.dv) fetch(v0 + 64);
    f32x4 o[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    // O^T += S^T (prefix Q)^T
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      bf16x8 fh[4], fl[4];
      vy_static_for<4>([&](auto i_c) {
        constexpr int i = decltype(i_c)::value;
        fh[i] = tr_frag<i * 32>(shb + k * 32 * VP, VP);
        fl[i] = tr_frag<i * 32>(slb + k * 32 * VP, VP);
      });
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        vy_tie(fh[i]);
        vy_tie(fl[i]);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fl[i], qh[k], o[i], 0, 0, 0);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fh[i], ql[k], o[i], 0, 0, 0);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fh[i], qh[k], o[i], 0, 0, 0);
      }
    }
    // O^T += V^T A^T over 32 keys at a time
#pragma unroll
    for (int tt = 0; tt < NB / 2; ++tt) {
      if (2 * tt > wave) break;
      bf16x8 fv[4];
      vy_static_for<4>([&](auto i_c) {
        constexpr int i = decltype(i_c)::value;
        fv[i] = tr_frag<i * 32>(vb + tt * 32 * VP, VP);
      });
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        vy_tie(fv[i]);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fv[i], pl[tt], o[i], 0, 0, 0);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fv[i], ph[tt], o[i], 0, 0, 0);
      }
    }
    if (qi < rows) {
      bf16* O = (bf16*)a.out + ((int64_t)b * a.L + ch * C + qi) * a.ldo + head * a.dv + v0;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int col = 16 * i + 4 * kq;
        if (v0 + col < a.dv) {
          bf16x4 w;
#pragma unroll
          for (int e = 0; e < 4; ++e) w[e] = (bf16)o[i][e];
          *reinterpret_cast<bf16x4*>(O + col) = w;
        }
      }
    }
    __syncthreads();   // the tiles have been read
  }
}

int64_t up256(int64_t x) { return (x + 255) / 256 * 256; }

}  // namespace

extern "C" int64_t vy_gated_attn_ws_bytes(int64_t B, int64_t L, int32_t h, int32_t dk, int32_t dv, int dtype) {
  return chunked(L, dk, dtype) ? up256(B * h * vy_cdiv(L, C) * dk * dv * 4) + B * h * vy_cdiv(L, C) * dk * 4 : 0;
}

extern "C" int vy_gated_attn(const void* p, int64_t ldp, int64_t oq, int64_t of, int64_t ov, float* state, const float* bias,
                             const float* lower, const int32_t* slots, const int32_t* start, const int32_t* count, void* out,
                             int64_t ldo, int64_t B, int64_t L, int32_t h, int32_t dk, int32_t dv, int silu, void* ws,
                             int64_t ws_bytes, int dtype, void* stream) {
  const char* who = "vy_gated_attn";
  if (!p || !state || !lower || !start || !out) VY_FAIL(VY_ERR_ARG, "%s: null pointer", who);
  if (B <= 0 || L <= 0 || h <= 0 || dk <= 0 || dv <= 0 || L > INT32_MAX) VY_FAIL(VY_ERR_ARG, "%s: empty problem", who);
  if (dk % 8 || dv % 8 || ldp % 8 || ldo % 8 || oq % 8 || of % 8 || ov % 8) VY_FAIL(VY_ERR_ARG, "%s: widths, strides and offsets must be multiples of 8", who);
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  if (B * h > 65535) VY_FAIL(VY_ERR_UNSUPPORTED, "%s: %ld (sequence, head) pairs", who, (long)(B * h));
  hipStream_t st = (hipStream_t)stream;
  DecayArgs a{};
  a.p = p; a.ldp = ldp; a.oq = oq; a.ok = of; a.ov = ov; a.state = state; a.slots = slots; a.start = start; a.count = count;
  a.out = out; a.ldo = ldo; a.B = (int)B; a.L = (int)L; a.h = h; a.dk = dk; a.dv = dv; a.silu = silu; a.nc = (int)vy_cdiv(L, C);
  a.f_bias = bias; a.f_lower = lower;
  if (chunked(L, dk, dtype)) {
    if (!ws || ws_bytes < vy_gated_attn_ws_bytes(B, L, h, dk, dv, dtype)) VY_FAIL(VY_ERR_ARG, "%s: workspace too small", who);
    a.U = (float*)ws;
    a.D = (float*)((char*)ws + up256(B * h * a.nc * (int64_t)dk * dv * 4));
    const dim3 grid(a.nc, (unsigned)(B * h)), block(256), sgrid((unsigned)vy_cdiv((int64_t)dk * dv, 1024), (unsigned)(B * h));
#define GA_GO(D)                                                          \
  do {                                                                    \
    hipLaunchKernelGGL(gated_kv_kernel<D>, grid, block, 0, st, a);        \
    hipLaunchKernelGGL(chunk_scan_kernel<true>, sgrid, block, 0, st, a);  \
    hipLaunchKernelGGL(gated_out_kernel<D>, grid, block, 0, st, a);       \
  } while (0)
    if (dk <= 32) GA_GO(32);
    else if (dk <= 64) GA_GO(64);
    else GA_GO(128);
#undef GA_GO
  } else if (dtype == VY_BF16 ? recurrent_go<bf16, true>(a, st) : recurrent_go<float, true>(a, st)) {
    VY_FAIL(VY_ERR_UNSUPPORTED, "%s: key width %d > 512", who, dk);
  }
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}
