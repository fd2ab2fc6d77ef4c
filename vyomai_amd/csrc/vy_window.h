// Decode attention over a ring of keys and values: the device code of vy_window.hip (a launch of its own) and vy_parallel.hip
// (one launch with other work of the same step).  See vy_window.hip for what a ring is.
//
// WindowDecode (bf16): a workgroup takes one key/value head of one sequence with ALL its query heads (up to 16 per pass: the ring
// is streamed once, not once per query head) and a slice of the ring; its four waves walk units of 32 rows on their own.
// Swapped products as in attn_fwd_gen_kernel: S^T = K Q^T straight from global memory into MFMA operands (a key row is read
// once, nobody else needs it: no LDS), P stays in registers as the B operand of O^T = V^T P^T, V passes through a wave-private
// LDS tile for the transposing reads.  Rows of the next unit are requested before the arithmetic of this one.  The token's own
// key and value never make the trip to memory and back: they replace its row of the ring in registers / LDS.
//
// The norms over the whole query and key projection (DecodeArgs::q_norm) are part of it: every workgroup adds up the squares of
// the sequence's projection rows itself (a few KB from L2), in fp32, and the rotated operand is rounded once.  Norms over groups
// of columns (DecodeArgs::group) need no more than the group's own lanes.
//
// MAPS = 2, differential attention: a head's queries and keys are two maps side by side (a row of the ring is [key 1 | key 2 |
// value]), each with a softmax of its own over the same values: one stream of the ring, one value fragment for both.  The maps'
// partial results always go through window_finish_diff.
#pragma once
#include "vy_common.h"
#include <float.h>

namespace vy_window {

constexpr float LOG2E = 1.4426950408889634f;

struct DecodeArgs {
  const bf16* p; int64_t ldp, oq, ok, ov, og;
  bf16* ring; int64_t r_ss, r_sh; int R, keep;
  const float2* rope; int half, rope_len;
  const float* q_norm; const float* k_norm; int n_q, n_k; float eps;   // nullable: norms over the whole projections ...
  int group, temp_every; float temp_coef;                              // ... or (group > 0) over groups; temperature of the query
  const bf16* vm; int64_t ldm; float lambda;                           // nullable: values mixed in
  int n_v, m_v, m_vp;                                                  // used columns of v's heads and of vm's, and vm's padded ones
  bf16* vo; int64_t ldvo;                                              // nullable: receives the token's own values
  const int* slots; const int* start;
  bf16* out; int64_t ldo;
  int h, hk, dim, vdim, ns, passes, sink;   // ns slices of the ring, passes of 16 query heads per key/value head
  float scale;
  float* part_o; float* part_ml;            // ns > 1: [b][head][slice][vdim] and [b][head][slice][2] (head: head * MAPS + map)
  float lambda2, out_scale, eps_out;        // MAPS = 2: the difference's weight, the outputs' factor and norm
};

__device__ __forceinline__ float group_max(float v) {   // over the four lane groups (lane >> 4)
  const unsigned u = __builtin_bit_cast(unsigned, v);
  auto s = __builtin_amdgcn_permlane16_swap(u, u, false, false);
  v = fmaxf(__builtin_bit_cast(float, (unsigned)s[0]), __builtin_bit_cast(float, (unsigned)s[1]));
  const unsigned w = __builtin_bit_cast(unsigned, v);
  auto t = __builtin_amdgcn_permlane32_swap(w, w, false, false);
  return fmaxf(__builtin_bit_cast(float, (unsigned)t[0]), __builtin_bit_cast(float, (unsigned)t[1]));
}
__device__ __forceinline__ float group_sum(float v) {
  const unsigned u = __builtin_bit_cast(unsigned, v);
  auto s = __builtin_amdgcn_permlane16_swap(u, u, false, false);
  v = __builtin_bit_cast(float, (unsigned)s[0]) + __builtin_bit_cast(float, (unsigned)s[1]);
  const unsigned w = __builtin_bit_cast(unsigned, v);
  auto t = __builtin_amdgcn_permlane32_swap(w, w, false, false);
  return __builtin_bit_cast(float, (unsigned)t[0]) + __builtin_bit_cast(float, (unsigned)t[1]);
}

// row of position p in a ring of R rows whose first `keep` stay
__device__ __forceinline__ int ring_row(int p, int R, int keep) { return p < R ? p : keep + (p - keep) % (R - keep); }

// factor on the query of a position
__device__ __forceinline__ float query_temperature(int pos, int every, float coef) {
  return every > 0 ? 1.f + coef * logf((float)((pos + 1) / every + 1)) : 1.f;
}

// 8 columns d0 .. of a head times r w (w nullable: as they are), rotated, rounded once
__device__ __forceinline__ bf16x8 rotate8(const DecodeArgs& a, const float2* t, int d0, bf16x8 x, const float* w, float r) {
  if (!w && d0 >= 2 * a.half) return x;
  float v[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = (float)x[e];
  if (w) {
    float f[8];
    VyChunk<float>::load(w, f);
    VyChunk<float>::load(w + 4, f + 4);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] *= r * f[e];
  }
#pragma unroll
  for (int e = 0; e < 8; e += 2) {
    const int i = (d0 + e) >> 1;
    if (i < a.half) {
      const float2 cs = t[i];
      const float u = v[e], y = v[e + 1];
      v[e] = u * cs.x - y * cs.y;
      v[e + 1] = y * cs.x + u * cs.y;
    }
  }
  bf16x8 y;
#pragma unroll
  for (int e = 0; e < 8; ++e) y[e] = (bf16)v[e];
  return y;
}
// v <- (1 - lambda) v + lambda m on VEC columns d .. of head g; the rows m have heads of their own width (m_v of m_vp columns used,
// against n_v of vdim) and agree as flat rows of used columns
template <typename T, int VEC>
__device__ __forceinline__ void mix_values(float (&v)[VEC], const T* m, float lambda, int g, int d, int vdim, int n_v, int m_v, int m_vp) {
  float x[VEC];
  if (m_v == n_v) {
    VyChunk<T>::load(m + g * vdim + d, x);
  } else {
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const int f = g * n_v + d + e;
      x[e] = d + e < n_v ? VyT<T>::ld(m + (f / m_v) * m_vp + f % m_v) : 0.f;
    }
  }
#pragma unroll
  for (int e = 0; e < VEC; ++e) v[e] = (1.f - lambda) * v[e] + lambda * x[e];
}
__device__ __forceinline__ float rms_factor(float sum, int n, float eps) {
  const float ms = sum / (float)n + eps, r = rsqrtf(ms);
  return r * (1.5f - 0.5f * ms * r * r);
}

// DHP, DVP: padded widths of a map's keys and of the values (DecodeArgs::dim is a map's)
template <int DHP, int DVP, int MAPS = 1>
struct WindowDecode {
  static constexpr int KS = DHP / 32, NDB = DVP / 16;
  static constexpr int VPITCH = (DVP + 8) * 2;              // bytes per row of a wave's value tile
  static constexpr int VROWS = 32 * VPITCH, VC = DVP / 8;   // 16-byte chunks per value row
  static constexpr int VPL = 32 * VC / 64;                  // value chunks per lane and unit
  static constexpr int QP = DHP + 8;                        // query pitch (elements)
  // [value tiles, later the waves' results | queries | new key | new value | m, l of the waves]
  static constexpr int O_Q = 4 * VROWS, O_K = O_Q + MAPS * 16 * QP * 2, O_V = O_K + MAPS * DHP * 2, O_ML = O_V + DVP * 2;
  static_assert(4 * 16 * DVP * 4 <= 4 * VROWS, "the waves' results fit over the value tiles");
  static_assert(2 * 64 * 4 >= 8 * 4, "the norms' partial sums fit over m, l");
  static constexpr int LDS = O_ML + 2 * 64 * 4;

  // slice of the ring, y = key/value head * passes + pass, b = sequence
  static __device__ __forceinline__ void run(const DecodeArgs& a, char* smem, int slice, int y, int b) {
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r16 = lane & 15, kq = lane >> 4;
  const int g = y / a.passes, pass = y - g * a.passes;
  const int rep = a.h / a.hk, h0 = g * rep + pass * 16, nh = min(16, rep - pass * 16);
  const int slot = a.slots ? a.slots[b] : b;
  const int pos = a.start[slot];
  const int n = min(pos + 1, a.R), fresh = ring_row(pos, a.R, a.keep);
  const int KW = MAPS * a.dim, W = KW + a.vdim;
  const bf16* row = a.p + (int64_t)b * a.ldp;
  bf16* ring = a.ring + (int64_t)slot * a.r_ss + (int64_t)g * a.r_sh;
  const float2* trig = a.rope + (int64_t)min(pos, a.rope_len - 1) * a.half;
  const bf16x8 zero8 = {(bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f};
  const int units = (n + 31) / 32, step = a.ns * 4;
  int u = slice * 4 + wave;

  // keys and values of a unit in registers: key rows as MFMA operands, values chunk by chunk (whole rows per instruction)
  bf16x8 kf[MAPS][2][KS], vr[VPL];
  auto request = [&](int unit, bf16x8 (&kd)[MAPS][2][KS], bf16x8 (&vd)[VPL]) {
#pragma unroll
    for (int blk = 0; blk < 2; ++blk) {
      const int j = min(unit * 32 + 16 * blk + r16, n - 1);
#pragma unroll
      for (int m = 0; m < MAPS; ++m)
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          const int d0 = 32 * ks + 8 * kq;
          kd[m][blk][ks] = d0 < a.dim ? *reinterpret_cast<const bf16x8*>(ring + (int64_t)j * W + m * a.dim + d0) : zero8;
        }
    }
#pragma unroll
    for (int i = 0; i < VPL; ++i) {
      const int c = lane + 64 * i, j = min(unit * 32 + c / VC, n - 1), d0 = (c % VC) * 8;
      vd[i] = d0 < a.vdim ? *reinterpret_cast<const bf16x8*>(ring + (int64_t)j * W + KW + d0) : zero8;
    }
  };
  if (u < units) request(u, kf, vr);

  // sums of squares of the sequence's whole query and key projections
  float rq = 1.f, rk = 1.f;
  if (a.q_norm && a.group == 0) {
    float* red = reinterpret_cast<float*>(smem + O_ML);
    float sq = 0.f, sk = 0.f;
    auto squares = [&](const bf16* p, int cols, float& s) {
      for (int i = tid * 8; i < cols; i += 2048) {
        const bf16x8 x = *reinterpret_cast<const bf16x8*>(p + i);
#pragma unroll
        for (int e = 0; e < 8; ++e) s = fmaf((float)x[e], (float)x[e], s);
      }
    };
    squares(row + a.oq, a.h * a.dim, sq);
    squares(row + a.ok, a.hk * a.dim, sk);
    sq = vy_wave_sum(sq);
    sk = vy_wave_sum(sk);
    if (lane == 0) { red[wave] = sq; red[4 + wave] = sk; }
    __syncthreads();
    rq = rms_factor(red[0] + red[1] + red[2] + red[3], a.n_q, a.eps);
    rk = rms_factor(red[4] + red[5] + red[6] + red[7], a.n_k, a.eps);
  }

  // rotated queries, new key, new value
  bf16* lq = reinterpret_cast<bf16*>(smem + O_Q);
  bf16* lk = reinterpret_cast<bf16*>(smem + O_K);
  bf16* lv = reinterpret_cast<bf16*>(smem + O_V);
  constexpr int CPG = DHP / 8;                 // lanes (chunks) of a head's map, neighbours
  auto group_factor = [&](const bf16x8 x, int count) {   // every lane of the wave is here: rms of the map's columns
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) s = fmaf((float)x[e], (float)x[e], s);
#pragma unroll
    for (int o = CPG / 2; o > 0; o >>= 1) s += __shfl_xor(s, o, 64);
    return rms_factor(s, count, a.eps);
  };
  const float temp = query_temperature(pos, a.temp_every, a.temp_coef);
  static_assert(MAPS * 16 * CPG % 64 == 0, "whole waves");
  for (int i = tid; i < MAPS * 16 * CPG; i += 256) {
    const int hm = i / CPG, hh = hm / MAPS, mp = hm % MAPS, d0 = (i % CPG) * 8;
    const bool ok = hh < nh && d0 < a.dim;
    bf16x8 q = zero8;
    const int at = (h0 + hh) * KW + mp * a.dim + d0;
    if (ok) q = *reinterpret_cast<const bf16x8*>(row + a.oq + at);
    float f = rq;
    if (a.q_norm && a.group) f = group_factor(q, a.n_q) * temp;
    if (ok) q = rotate8(a, trig, d0, q, a.q_norm ? a.q_norm + at : nullptr, f);
    *reinterpret_cast<bf16x8*>(lq + (mp * 16 + hh) * QP + d0) = q;
  }
  const bool owner = pass == 0 && (fresh / 32) % step / 4 == slice;   // the workgroup whose units hold the new row
  static_assert(MAPS * CPG <= 64, "a new key is one wave's");
  if (tid >= 192) {
    const int mp = (tid - 192) / CPG, d0 = (tid - 192) % CPG * 8;
    const bool ok = mp < MAPS && d0 < a.dim;
    bf16x8 k8 = zero8;
    const int at = g * KW + mp * a.dim + d0;
    if (ok) k8 = *reinterpret_cast<const bf16x8*>(row + a.ok + at);
    float f = rk;
    if (a.k_norm && a.group) f = group_factor(k8, a.n_k);
    if (ok) {
      k8 = rotate8(a, trig, d0, k8, a.k_norm ? a.k_norm + at : nullptr, f);
      if (owner) *reinterpret_cast<bf16x8*>(ring + (int64_t)fresh * W + mp * a.dim + d0) = k8;
    }
    if (mp < MAPS) *reinterpret_cast<bf16x8*>(lk + mp * DHP + d0) = k8;
  } else if (tid >= 128 && tid < 192 && tid - 128 < VC) {
    const int d0 = (tid - 128) * 8;
    bf16x8 v8 = zero8;
    if (d0 < a.vdim) {
      v8 = *reinterpret_cast<const bf16x8*>(row + a.ov + (int64_t)g * a.vdim + d0);
      if (owner && a.vo) *reinterpret_cast<bf16x8*>(a.vo + (int64_t)b * a.ldvo + (int64_t)g * a.vdim + d0) = v8;
      if (a.vm) {
        float v[8];
        VyChunk<bf16>::unpack(v8, v);
        mix_values(v, a.vm + (int64_t)b * a.ldm, a.lambda, g, d0, a.vdim, a.n_v, a.m_v, a.m_vp);
#pragma unroll
        for (int e = 0; e < 8; ++e) v8[e] = (bf16)v[e];
      }
      if (owner) *reinterpret_cast<bf16x8*>(ring + (int64_t)fresh * W + KW + d0) = v8;
    }
    *reinterpret_cast<bf16x8*>(lv + d0) = v8;
  }
  __syncthreads();
  bf16x8 qf[MAPS][KS];
#pragma unroll
  for (int m = 0; m < MAPS; ++m)
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) qf[m][ks] = *reinterpret_cast<const bf16x8*>(lq + (m * 16 + r16) * QP + 32 * ks + 8 * kq);

  f32x4 o[MAPS][NDB];
  float m_run[MAPS], l_run[MAPS];
#pragma unroll
  for (int m = 0; m < MAPS; ++m) {
    m_run[m] = -FLT_MAX;
    l_run[m] = 0.f;
#pragma unroll
    for (int d = 0; d < NDB; ++d) o[m][d] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const float c = a.scale * LOG2E;
  char* vt = smem + wave * VROWS;
  const unsigned vtr = vy_lds_addr(vt) + (4 * kq + (r16 >> 2)) * VPITCH + (4 * (r16 & 3)) * 2;
  for (; u < units; u += step) {
    const int j0 = u * 32;
    if (fresh >= j0 && fresh < j0 + 32) {   // wave-uniform
      if (r16 == (fresh & 15)) {
#pragma unroll
        for (int blk = 0; blk < 2; ++blk)
          if (blk == ((fresh >> 4) & 1))
#pragma unroll
            for (int m = 0; m < MAPS; ++m)
#pragma unroll
              for (int ks = 0; ks < KS; ++ks) kf[m][blk][ks] = *reinterpret_cast<const bf16x8*>(lk + m * DHP + 32 * ks + 8 * kq);
      }
#pragma unroll
      for (int i = 0; i < VPL; ++i) {
        const int cc = lane + 64 * i;
        if (cc / VC == (fresh & 31)) vr[i] = *reinterpret_cast<const bf16x8*>(lv + (cc % VC) * 8);
      }
    }
    if (j0 + 32 > n) {   // rows behind the last one weigh 0, whatever an earlier owner of the slot left there
#pragma unroll
      for (int i = 0; i < VPL; ++i)
        if (j0 + (lane + 64 * i) / VC >= n) vr[i] = zero8;
    }
#pragma unroll
    for (int i = 0; i < VPL; ++i) {
      const int cc = lane + 64 * i;
      *reinterpret_cast<bf16x8*>(vt + (cc / VC) * VPITCH + (cc % VC) * 16) = vr[i];
    }
    f32x4 sc[MAPS][2];
#pragma unroll
    for (int m = 0; m < MAPS; ++m)
#pragma unroll
      for (int blk = 0; blk < 2; ++blk) {
        sc[m][blk] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) sc[m][blk] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[m][blk][ks], qf[m][ks], sc[m][blk], 0, 0, 0);
      }
    if (u + step < units) request(u + step, kf, vr);   // lands under this unit's softmax and value product
    bf16x8 pf[MAPS];
#pragma unroll
    for (int m = 0; m < MAPS; ++m) {
      float tmax = -INFINITY;
#pragma unroll
      for (int blk = 0; blk < 2; ++blk)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          if (j0 + 16 * blk + 4 * kq + r >= n) sc[m][blk][r] = -INFINITY;
          tmax = fmaxf(tmax, sc[m][blk][r]);
        }
      const float m_new = fmaxf(m_run[m], group_max(tmax) * c);
      const float alpha = __builtin_amdgcn_exp2f(m_run[m] - m_new);
      m_run[m] = m_new;
      l_run[m] *= alpha;
#pragma unroll
      for (int d = 0; d < NDB; ++d)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[m][d][r] *= alpha;
#pragma unroll
      for (int blk = 0; blk < 2; ++blk)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float e = __builtin_amdgcn_exp2f(fmaf(sc[m][blk][r], c, -m_run[m]));
          l_run[m] += e;
          pf[m][4 * blk + r] = (bf16)e;
        }
    }
    vy_static_for<NDB>([&](auto d_c) {
      constexpr int d = decltype(d_c)::value;
      union { struct { s16x4 a, b; } hh; bf16x8 v; } uu;
      uu.hh.a = vy_lds_tr16_off<d * 32>(vtr);
      uu.hh.b = vy_lds_tr16_off<d * 32 + 16 * VPITCH>(vtr);
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      vy_tie(uu.v);
#pragma unroll
      for (int m = 0; m < MAPS; ++m) o[m][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(uu.v, pf[m], o[m][d], 0, 0, 0);
    });
  }

  // the four waves' results through LDS, map by map
#pragma unroll
  for (int mp = 0; mp < MAPS; ++mp) {
  l_run[mp] = group_sum(l_run[mp]);
  __syncthreads();
  float* lo = reinterpret_cast<float*>(smem);                    // [wave][head][DVP]
  float* lml = reinterpret_cast<float*>(smem + O_ML);            // m [wave][16], l [wave][16]
#pragma unroll
  for (int d = 0; d < NDB; ++d) *reinterpret_cast<f32x4*>(lo + (wave * 16 + r16) * DVP + 16 * d + 4 * kq) = o[mp][d];
  if (kq == 0) {
    lml[wave * 16 + r16] = m_run[mp];
    lml[64 + wave * 16 + r16] = l_run[mp];
  }
  __syncthreads();
  for (int i = tid; i < nh * (a.vdim / 8); i += 256) {
    const int hh = i / (a.vdim / 8), d0 = (i % (a.vdim / 8)) * 8, head = h0 + hh;
    float m = fmaxf(fmaxf(lml[hh], lml[16 + hh]), fmaxf(lml[32 + hh], lml[48 + hh]));
    if (MAPS == 1 && a.ns == 1 && a.sink) m = fmaxf(m, 0.f);
    float l = MAPS == 1 && a.ns == 1 && a.sink ? __builtin_amdgcn_exp2f(-m) : 0.f, v[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float s = __builtin_amdgcn_exp2f(lml[w * 16 + hh] - m);
      l += s * lml[64 + w * 16 + hh];
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = fmaf(s, lo[(w * 16 + hh) * DVP + d0 + e], v[e]);
    }
    if (MAPS == 1 && a.ns == 1) {
      const float inv = 1.f / l;
      bf16x8 w8;
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] *= inv;
      if (a.og >= 0) {
        const bf16x8 g8 = *reinterpret_cast<const bf16x8*>(row + a.og + (int64_t)head * a.vdim + d0);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] *= vy_sigmoid((float)g8[e]);
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) w8[e] = (bf16)v[e];
      *reinterpret_cast<bf16x8*>(a.out + (int64_t)b * a.ldo + (int64_t)head * a.vdim + d0) = w8;
    } else {
      const int64_t at = (((int64_t)b * a.h + head) * MAPS + mp) * a.ns + slice;
      VyChunk<float>::store(a.part_o + at * a.vdim + d0, v);
      VyChunk<float>::store(a.part_o + at * a.vdim + d0 + 4, v + 4);
      if (d0 == 0) { a.part_ml[2 * at] = m; a.part_ml[2 * at + 1] = l; }
    }
  }
  }
}
};

// one workgroup per (sequence, head): sink, slices, gate
constexpr int FINISH_LDS = 256 * 4 * 4;
__device__ __forceinline__ void window_finish(const DecodeArgs& a, float* red, int head, int b) {
  const int tid = threadIdx.x;
  const float* ml = a.part_ml + ((int64_t)b * a.h + head) * a.ns * 2;
  const float* po = a.part_o + ((int64_t)b * a.h + head) * a.ns * a.vdim;
  const int nc = a.vdim / 4, lanes = nc <= 64 ? 64 : nc <= 128 ? 128 : 256, groups = 256 / lanes;
  const int ch = tid % lanes, grp = tid / lanes;
  float m = a.sink ? 0.f : -FLT_MAX;
  for (int s = 0; s < a.ns; ++s) m = fmaxf(m, ml[2 * s]);
  float l = a.sink ? __builtin_amdgcn_exp2f(-m) : 0.f;
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int s = 0; s < a.ns; ++s) l += ml[2 * s + 1] * __builtin_amdgcn_exp2f(ml[2 * s] - m);
  if (ch < nc) {
#pragma unroll 4
    for (int s = grp; s < a.ns; s += groups) {
      const float f = __builtin_amdgcn_exp2f(ml[2 * s] - m);
      const f32x4 x = *reinterpret_cast<const f32x4*>(po + (int64_t)s * a.vdim + ch * 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = fmaf(f, x[e], v[e]);
    }
  }
  *reinterpret_cast<f32x4*>(red + tid * 4) = v;
  __syncthreads();
  if (grp == 0 && ch < nc) {
    for (int s = 1; s < groups; ++s) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(red + (s * lanes + ch) * 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] += x[e];
    }
    const float inv = 1.f / l;
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] *= inv;
    if (a.og >= 0) {
      const bf16x4 g4 = *reinterpret_cast<const bf16x4*>(a.p + (int64_t)b * a.ldp + a.og + (int64_t)head * a.vdim + ch * 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] *= vy_sigmoid((float)g4[e]);
    }
    bf16x4 w;
#pragma unroll
    for (int e = 0; e < 4; ++e) w[e] = (bf16)v[e];
    *reinterpret_cast<bf16x4*>(a.out + (int64_t)b * a.ldo + (int64_t)head * a.vdim + ch * 4) = w;
  }
}

// one workgroup per (sequence, head): both maps' slices, their difference, the head's norm.  vdim <= 1024.
// A lane holds one slice's statistics (at most 64): one memory latency for all of them, and every partial row's factor is known
// before the first is added.
constexpr int FINISH_DIFF_LDS = FINISH_LDS + 16 + 2 * 64 * 4;
__device__ __forceinline__ void window_finish_diff(const DecodeArgs& a, float* red, int head, int b) {
  const int tid = threadIdx.x;
  const int nc = a.vdim / 4, lanes = nc <= 64 ? 64 : nc <= 128 ? 128 : 256, groups = 256 / lanes;
  const int ch = tid % lanes, grp = tid / lanes;
  float* sw = red + 1024 + 4;                // [map][slice]
  const int64_t at = ((int64_t)b * a.h + head) * 2 * a.ns;
  if (tid < 128) {
    const int mp = tid >> 6, s = tid & 63;
    const float2 ml = s < a.ns ? *reinterpret_cast<const float2*>(a.part_ml + (at + mp * a.ns + s) * 2) : make_float2(-FLT_MAX, 0.f);
    const float e = __builtin_amdgcn_exp2f(ml.x - vy_wave_max(ml.x));
    sw[mp * 64 + s] = e * (mp ? -a.lambda2 : 1.f) / vy_wave_sum(e * ml.y);
  }
  // the maps' slices as one list: 2 ns rows; the first batch is requested ahead of the factors
  const float* po = a.part_o + at * a.vdim;
  constexpr int UB = 8;
  f32x4 x[UB];
  auto fetch = [&](int k0) {
#pragma unroll
    for (int u = 0; u < UB; ++u) x[u] = *reinterpret_cast<const f32x4*>(po + (int64_t)min(k0 + u * groups, 2 * a.ns - 1) * a.vdim + (ch < nc ? ch : 0) * 4);
  };
  fetch(grp);
  __syncthreads();
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = grp; k0 < 2 * a.ns; k0 += UB * groups) {
#pragma unroll
    for (int u = 0; u < UB; ++u) {
      const int k = k0 + u * groups;
      const float f = k < 2 * a.ns ? sw[k < a.ns ? k : 64 + k - a.ns] : 0.f;
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = fmaf(f, x[u][e], o[e]);
    }
    if (k0 + UB * groups < 2 * a.ns) fetch(k0 + UB * groups);
  }
  *reinterpret_cast<f32x4*>(red + tid * 4) = o;
  __syncthreads();
  float sq = 0.f;
  if (grp == 0 && ch < nc) {
    for (int s = 1; s < groups; ++s) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(red + (s * lanes + ch) * 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] += x[e];
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) sq = fmaf(o[e], o[e], sq);   // (padded columns are zero)
  }
  sq = vy_wave_sum(sq);
  if ((tid & 63) == 0) red[1024 + (tid >> 6)] = sq;
  __syncthreads();
  if (grp == 0 && ch < nc) {
    const float f = rms_factor(red[1024] + red[1025] + red[1026] + red[1027], a.n_v, a.eps_out) * a.out_scale;
    bf16x4 w;
#pragma unroll
    for (int e = 0; e < 4; ++e) w[e] = (bf16)(o[e] * f);
    *reinterpret_cast<bf16x4*>(a.out + (int64_t)b * a.ldo + (int64_t)head * a.vdim + ch * 4) = w;
  }
}

// slices of the ring: about 512 workgroups in all, at least 128 rows (one unit per wave) each
inline int slices_of(int64_t workgroups, int64_t rows) {
  int64_t ns = (512 + workgroups - 1) / workgroups;
  const int64_t most = (rows + 127) / 128;
  if (ns > most) ns = most;
  return (int)(ns < 1 ? 1 : ns > 64 ? 64 : ns);
}

}  // namespace vy_window
