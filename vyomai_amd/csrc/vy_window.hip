// Sliding-window attention over a ring of keys and values, for decoders whose queries see only the last `window` tokens.
//
// Memory: per sequence (slot) and key/value head a ring of R rows [key (dim) | value (vdim)], R = the window (or less while
// sequences are shorter): position p lives in row p % R, so a sequence never holds more than its window.
//
//   vy_window_rows     prefill: rotary positions on the new keys (in place in the packed projection rows) and the last R new
//                      rows to the ring
//   vy_window_context  prefill behind a past: the ring's rows and the new ones as one contiguous context for vy_attn_fwd_ex
//   vy_window_decode   one query token per sequence: rotation of query and key, the new row to the ring, attention over the
//                      ring, sink, output gate.  Every row of the ring that holds a token is inside the window, so decode
//                      needs no mask but the row count -- and no order: softmax does not care where a row lies.
//
// window_decode_kernel (bf16): a workgroup takes one key/value head of one sequence with ALL its query heads (up to 16 per
// pass: the ring is streamed once, not once per query head) and a slice of the ring; its four waves walk units of 32 rows on
// their own.  Swapped products as in attn_fwd_gen_kernel: S^T = K Q^T straight from global memory into MFMA operands (a key
// row is read once, nobody else needs it: no LDS), P stays in registers as the B operand of O^T = V^T P^T, V passes through a
// wave-private LDS tile for the transposing reads.  Rows of the next unit are requested before the arithmetic of this one.
// The token's own key and value never make the trip to memory and back: they replace row p % R in registers / LDS.
#include "vy_common.h"
#include <float.h>

namespace {

constexpr float LOG2E = 1.4426950408889634f;

struct RowsArgs {
  const void* p; int64_t ldp, ok, ov;       // packed rows; key / value columns
  void* ring; int64_t r_ss, r_sh; int R;    // ring rows of dim + vdim elements
  const float2* rope; int half, rope_len;
  const int* slots; const int* start; const int* count;
  int64_t M; int L, hk, dim, vdim, rotate, store;
};

// one 16-byte chunk of a token's keys or values per thread
template <typename T>
__global__ __launch_bounds__(256) void window_rows_kernel(RowsArgs a) {
  constexpr int VEC = VyChunk<T>::VEC;
  const int kc = a.dim / VEC, vc = a.vdim / VEC, per_head = kc + vc, per_row = per_head * a.hk;
  const int64_t total = a.M * per_row;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
    const int64_t row = i / per_row;
    const int r = (int)(i - row * per_row), g = r / per_head, c = r - g * per_head;
    const int b = (int)(row / a.L), l = (int)(row - (int64_t)b * a.L);
    const int slot = a.slots ? a.slots[b] : b;
    const int first = a.start ? a.start[slot] : 0, n = a.count ? a.count[b] : a.L;
    const int pos = first + l;
    const bool keep = a.store && l < n && l + a.R >= n;
    const bool key = c < kc;
    if (!keep && !(key && a.rotate)) continue;
    T* src = (T*)a.p + row * a.ldp + (key ? a.ok + (int64_t)g * a.dim + c * VEC : a.ov + (int64_t)g * a.vdim + (c - kc) * VEC);
    float v[VEC];
    VyChunk<T>::load(src, v);
    if (key && a.rotate && c * VEC < 2 * a.half) {
      const float2* t = a.rope + (int64_t)(pos < a.rope_len ? pos : a.rope_len - 1) * a.half;   // (clamped: padding rows only)
#pragma unroll
      for (int e = 0; e < VEC; e += 2) {
        const int j = (c * VEC + e) >> 1;
        if (j < a.half) {
          const float2 cs = t[j];
          const float u = v[e], w = v[e + 1];
          v[e] = u * cs.x - w * cs.y;
          v[e + 1] = w * cs.x + u * cs.y;
        }
      }
      VyChunk<T>::store(src, v);
    }
    if (keep) VyChunk<T>::store((T*)a.ring + (int64_t)slot * a.r_ss + (int64_t)g * a.r_sh + (int64_t)(pos % a.R) * (a.dim + a.vdim) + c * VEC, v);
  }
}

struct ContextArgs {
  const void* p; int64_t ldp, ok, ov;
  const void* ring; int64_t r_ss, r_sh; int R;
  void* ctx; int S, past;                   // ctx [B][hk][S][dim + vdim]; past rows of the ring at most
  const int* slots; const int* start;
  int B, L, hk, dim, vdim;
};

// row s of sequence b: position (start - k) + s with k = min(start, past); the first k rows come from the ring
template <typename T>
__global__ __launch_bounds__(256) void window_context_kernel(ContextArgs a) {
  constexpr int VEC = VyChunk<T>::VEC;
  const int W = a.dim + a.vdim, nc = W / VEC;
  const int64_t total = (int64_t)a.B * a.hk * a.S * nc;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
    const int c = (int)(i % nc) * VEC;
    int64_t r = i / nc;
    const int s = (int)(r % a.S);
    r /= a.S;
    const int g = (int)(r % a.hk), b = (int)(r / a.hk);
    const int slot = a.slots ? a.slots[b] : b;
    const int first = a.start[slot], k = first < a.past ? first : a.past;
    float v[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = 0.f;
    if (s < k) {
      VyChunk<T>::load((const T*)a.ring + (int64_t)slot * a.r_ss + (int64_t)g * a.r_sh + (int64_t)((first - k + s) % a.R) * W + c, v);
    } else if (s - k < a.L) {
      const T* row = (const T*)a.p + ((int64_t)b * a.L + s - k) * a.ldp;
      VyChunk<T>::load(c < a.dim ? row + a.ok + (int64_t)g * a.dim + c : row + a.ov + (int64_t)g * a.vdim + (c - a.dim), v);
    }
    VyChunk<T>::store((T*)a.ctx + (((int64_t)b * a.hk + g) * a.S + s) * W + c, v);
  }
}

// ---- decode ---------------------------------------------------------------------------------
struct DecodeArgs {
  const bf16* p; int64_t ldp, oq, ok, ov, og;
  bf16* ring; int64_t r_ss, r_sh; int R;
  const float2* rope; int half, rope_len;
  const int* slots; const int* start;
  bf16* out; int64_t ldo;
  int h, hk, dim, vdim, ns, passes, sink;   // ns slices of the ring, passes of 16 query heads per key/value head
  float scale;
  float* part_o; float* part_ml;            // ns > 1: [b][head][slice][vdim] and [b][head][slice][2]
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

__device__ __forceinline__ bf16x8 rotate8(const DecodeArgs& a, const float2* t, int d0, bf16x8 x) {
  if (d0 >= 2 * a.half) return x;
  bf16x8 y = x;
#pragma unroll
  for (int e = 0; e < 8; e += 2) {
    const int i = (d0 + e) >> 1;
    if (i < a.half) {
      const float2 cs = t[i];
      const float u = (float)x[e], w = (float)x[e + 1];
      y[e] = (bf16)(u * cs.x - w * cs.y);
      y[e + 1] = (bf16)(w * cs.x + u * cs.y);
    }
  }
  return y;
}

template <int DHP, int DVP>
__global__ __launch_bounds__(256) void window_decode_kernel(DecodeArgs a) {
  constexpr int KS = DHP / 32, NDB = DVP / 16;
  constexpr int VPITCH = (DVP + 8) * 2;              // bytes per row of a wave's value tile
  constexpr int VROWS = 32 * VPITCH, VC = DVP / 8;   // 16-byte chunks per value row
  constexpr int VPL = 32 * VC / 64;                  // value chunks per lane and unit
  constexpr int QP = DHP + 8;                        // query pitch (elements)
  // [value tiles, later the waves' results | queries | new key | new value | m, l of the waves]
  constexpr int O_Q = 4 * VROWS, O_K = O_Q + 16 * QP * 2, O_V = O_K + DHP * 2, O_ML = O_V + DVP * 2;
  static_assert(4 * 16 * DVP * 4 <= 4 * VROWS, "the waves' results fit over the value tiles");
  __shared__ __attribute__((aligned(16))) char smem[O_ML + 2 * 64 * 4];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r16 = lane & 15, kq = lane >> 4;
  const int slice = blockIdx.x, b = blockIdx.z;
  const int g = (int)blockIdx.y / a.passes, pass = (int)blockIdx.y - g * a.passes;
  const int rep = a.h / a.hk, h0 = g * rep + pass * 16, nh = min(16, rep - pass * 16);
  const int slot = a.slots ? a.slots[b] : b;
  const int pos = a.start[slot];
  const int n = min(pos + 1, a.R), fresh = pos % a.R;
  const int W = a.dim + a.vdim;
  const bf16* row = a.p + (int64_t)b * a.ldp;
  bf16* ring = a.ring + (int64_t)slot * a.r_ss + (int64_t)g * a.r_sh;
  const float2* trig = a.rope + (int64_t)min(pos, a.rope_len - 1) * a.half;
  const bf16x8 zero8 = {(bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f};
  const int units = (n + 31) / 32, step = a.ns * 4;
  int u = slice * 4 + wave;

  // keys and values of a unit in registers: key rows as MFMA operands, values chunk by chunk (whole rows per instruction)
  bf16x8 kf[2][KS], vr[VPL];
  auto request = [&](int unit, bf16x8 (&kd)[2][KS], bf16x8 (&vd)[VPL]) {
#pragma unroll
    for (int blk = 0; blk < 2; ++blk) {
      const int j = min(unit * 32 + 16 * blk + r16, n - 1);
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const int d0 = 32 * ks + 8 * kq;
        kd[blk][ks] = d0 < a.dim ? *reinterpret_cast<const bf16x8*>(ring + (int64_t)j * W + d0) : zero8;
      }
    }
#pragma unroll
    for (int i = 0; i < VPL; ++i) {
      const int c = lane + 64 * i, j = min(unit * 32 + c / VC, n - 1), d0 = (c % VC) * 8;
      vd[i] = d0 < a.vdim ? *reinterpret_cast<const bf16x8*>(ring + (int64_t)j * W + a.dim + d0) : zero8;
    }
  };
  if (u < units) request(u, kf, vr);

  // rotated queries, new key, new value
  bf16* lq = reinterpret_cast<bf16*>(smem + O_Q);
  bf16* lk = reinterpret_cast<bf16*>(smem + O_K);
  bf16* lv = reinterpret_cast<bf16*>(smem + O_V);
  for (int i = tid; i < 16 * (DHP / 8); i += 256) {
    const int hh = i / (DHP / 8), d0 = (i % (DHP / 8)) * 8;
    const bool ok = hh < nh && d0 < a.dim;
    bf16x8 q = zero8;
    if (ok) q = rotate8(a, trig, d0, *reinterpret_cast<const bf16x8*>(row + a.oq + (int64_t)(h0 + hh) * a.dim + d0));
    *reinterpret_cast<bf16x8*>(lq + hh * QP + d0) = q;
  }
  const bool owner = pass == 0 && (fresh / 32) % step / 4 == slice;   // the workgroup whose units hold the new row
  if (tid >= 192 && tid - 192 < DHP / 8) {
    const int d0 = (tid - 192) * 8;
    bf16x8 k8 = zero8;
    if (d0 < a.dim) {
      k8 = rotate8(a, trig, d0, *reinterpret_cast<const bf16x8*>(row + a.ok + (int64_t)g * a.dim + d0));
      if (owner) *reinterpret_cast<bf16x8*>(ring + (int64_t)fresh * W + d0) = k8;
    }
    *reinterpret_cast<bf16x8*>(lk + d0) = k8;
  } else if (tid >= 128 && tid < 192 && tid - 128 < VC) {
    const int d0 = (tid - 128) * 8;
    bf16x8 v8 = zero8;
    if (d0 < a.vdim) {
      v8 = *reinterpret_cast<const bf16x8*>(row + a.ov + (int64_t)g * a.vdim + d0);
      if (owner) *reinterpret_cast<bf16x8*>(ring + (int64_t)fresh * W + a.dim + d0) = v8;
    }
    *reinterpret_cast<bf16x8*>(lv + d0) = v8;
  }
  __syncthreads();
  bf16x8 qf[KS];
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) qf[ks] = *reinterpret_cast<const bf16x8*>(lq + r16 * QP + 32 * ks + 8 * kq);

  f32x4 o[NDB];
#pragma unroll
  for (int d = 0; d < NDB; ++d) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = -FLT_MAX, l_run = 0.f;
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
            for (int ks = 0; ks < KS; ++ks) kf[blk][ks] = *reinterpret_cast<const bf16x8*>(lk + 32 * ks + 8 * kq);
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
    f32x4 sc[2];
#pragma unroll
    for (int blk = 0; blk < 2; ++blk) {
      sc[blk] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) sc[blk] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[blk][ks], qf[ks], sc[blk], 0, 0, 0);
    }
    if (u + step < units) request(u + step, kf, vr);   // lands under this unit's softmax and value product
    float tmax = -INFINITY;
#pragma unroll
    for (int blk = 0; blk < 2; ++blk)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (j0 + 16 * blk + 4 * kq + r >= n) sc[blk][r] = -INFINITY;
        tmax = fmaxf(tmax, sc[blk][r]);
      }
    const float m_new = fmaxf(m_run, group_max(tmax) * c);
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
    m_run = m_new;
    l_run *= alpha;
#pragma unroll
    for (int d = 0; d < NDB; ++d)
#pragma unroll
      for (int r = 0; r < 4; ++r) o[d][r] *= alpha;
    bf16x8 pf;
#pragma unroll
    for (int blk = 0; blk < 2; ++blk)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float e = __builtin_amdgcn_exp2f(fmaf(sc[blk][r], c, -m_run));
        l_run += e;
        pf[4 * blk + r] = (bf16)e;
      }
    vy_static_for<NDB>([&](auto d_c) {
      constexpr int d = decltype(d_c)::value;
      union { struct { s16x4 a, b; } hh; bf16x8 v; } uu;
      uu.hh.a = vy_lds_tr16_off<d * 32>(vtr);
      uu.hh.b = vy_lds_tr16_off<d * 32 + 16 * VPITCH>(vtr);
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      vy_tie(uu.v);
      o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(uu.v, pf, o[d], 0, 0, 0);
    });
  }
  l_run = group_sum(l_run);

  // the four waves' results through LDS
  __syncthreads();
  float* lo = reinterpret_cast<float*>(smem);                    // [wave][head][DVP]
  float* lml = reinterpret_cast<float*>(smem + O_ML);            // m [wave][16], l [wave][16]
#pragma unroll
  for (int d = 0; d < NDB; ++d) *reinterpret_cast<f32x4*>(lo + (wave * 16 + r16) * DVP + 16 * d + 4 * kq) = o[d];
  if (kq == 0) {
    lml[wave * 16 + r16] = m_run;
    lml[64 + wave * 16 + r16] = l_run;
  }
  __syncthreads();
  for (int i = tid; i < nh * (a.vdim / 8); i += 256) {
    const int hh = i / (a.vdim / 8), d0 = (i % (a.vdim / 8)) * 8, head = h0 + hh;
    float m = fmaxf(fmaxf(lml[hh], lml[16 + hh]), fmaxf(lml[32 + hh], lml[48 + hh]));
    if (a.ns == 1 && a.sink) m = fmaxf(m, 0.f);
    float l = a.ns == 1 && a.sink ? __builtin_amdgcn_exp2f(-m) : 0.f, v[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float s = __builtin_amdgcn_exp2f(lml[w * 16 + hh] - m);
      l += s * lml[64 + w * 16 + hh];
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = fmaf(s, lo[(w * 16 + hh) * DVP + d0 + e], v[e]);
    }
    if (a.ns == 1) {
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
      const int64_t at = ((int64_t)b * a.h + head) * a.ns + slice;
      VyChunk<float>::store(a.part_o + at * a.vdim + d0, v);
      VyChunk<float>::store(a.part_o + at * a.vdim + d0 + 4, v + 4);
      if (d0 == 0) { a.part_ml[2 * at] = m; a.part_ml[2 * at + 1] = l; }
    }
  }
}

// one workgroup per (sequence, head): sink, slices, gate
__global__ __launch_bounds__(256) void window_finish_kernel(DecodeArgs a) {
  __shared__ float red[256 * 4];
  const int head = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
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

// slices of the ring: about 512 workgroups in all, at least 128 rows (one unit per wave) each
int slices_of(int64_t workgroups, int64_t rows) {
  int64_t ns = (512 + workgroups - 1) / workgroups;
  const int64_t most = (rows + 127) / 128;
  if (ns > most) ns = most;
  return (int)(ns < 1 ? 1 : ns > 64 ? 64 : ns);
}

template <int DHP>
void decode_go(const DecodeArgs& a, dim3 grid, hipStream_t st) {
  const dim3 block(256);
  if (a.vdim <= 64) hipLaunchKernelGGL((window_decode_kernel<DHP, 64>), grid, block, 0, st, a);
  else if (a.vdim <= 128) hipLaunchKernelGGL((window_decode_kernel<DHP, 128>), grid, block, 0, st, a);
  else hipLaunchKernelGGL((window_decode_kernel<DHP, 256>), grid, block, 0, st, a);
}

int check_ring(const char* who, const void* ring, int64_t r_ss, int64_t r_sh, int32_t R, int32_t hk, int32_t dim, int32_t vdim,
               int vec) {
  if (!ring || R < 1 || hk < 1 || dim < 1 || vdim < 1) VY_FAIL(VY_ERR_ARG, "%s: bad ring", who);
  if (dim % vec || vdim % vec || r_ss % vec || r_sh % vec) VY_FAIL(VY_ERR_ARG, "%s: widths and strides must be multiples of %d", who, vec);
  if (r_sh < (int64_t)R * (dim + vdim) || r_ss < hk * r_sh) VY_FAIL(VY_ERR_ARG, "%s: ring strides do not hold %d rows", who, R);
  return VY_OK;
}

int check_rope(const char* who, const float* rope, int32_t rope_dims, int32_t rope_len, int32_t dim) {
  if (rope_dims < 0 || rope_dims % 2 || rope_dims > dim || (rope_dims && (!rope || rope_len < 1)))
    VY_FAIL(VY_ERR_ARG, "%s: rotary table of %d columns, %d positions for heads of %d", who, rope_dims, rope_len, dim);
  return VY_OK;
}

}  // namespace

extern "C" int vy_window_rows(void* p, int64_t ldp, int64_t ok, int64_t ov, void* ring, int64_t r_ss, int64_t r_sh, int32_t R,
                              const float* rope, int32_t rope_dims, int32_t rope_len, int rotate, int store,
                              const int32_t* slots, const int32_t* start, const int32_t* count, int64_t B, int64_t L, int32_t hk,
                              int32_t dim, int32_t vdim, int dtype, void* stream) {
  const char* who = "vy_window_rows";
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!p || B <= 0 || L <= 0 || hk <= 0 || dim <= 0 || vdim <= 0 || dim % vec || vdim % vec || ldp % vec || ok % vec || ov % vec)
    VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (store) {
    if (!start) VY_FAIL(VY_ERR_ARG, "%s: ring without start positions", who);
    if (int rc = check_ring(who, ring, r_ss, r_sh, R, hk, dim, vdim, vec)) return rc;
  }
  if (rotate)
    if (int rc = check_rope(who, rope, rope_dims, rope_len, dim)) return rc;
  if (!rotate && !store) return VY_OK;
  RowsArgs a{p, ldp, ok, ov, ring, r_ss, r_sh, store ? R : 1, (const float2*)rope, rope_dims / 2, rope_len, slots, start, count,
             B * L, (int)L, hk, dim, vdim, rotate && rope_dims > 0, store};
  const int64_t want = vy_cdiv(a.M * hk * ((dim + vdim) / vec), 256);
  const dim3 grid((unsigned)(want < 16384 ? want : 16384)), block(256);
  if (dtype == VY_BF16) hipLaunchKernelGGL((window_rows_kernel<bf16>), grid, block, 0, (hipStream_t)stream, a);
  else hipLaunchKernelGGL((window_rows_kernel<float>), grid, block, 0, (hipStream_t)stream, a);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}

extern "C" int vy_window_context(const void* p, int64_t ldp, int64_t ok, int64_t ov, const void* ring, int64_t r_ss, int64_t r_sh,
                                 int32_t R, void* ctx, int32_t S, int32_t past, const int32_t* slots, const int32_t* start,
                                 int64_t B, int64_t L, int32_t hk, int32_t dim, int32_t vdim, int dtype, void* stream) {
  const char* who = "vy_window_context";
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!p || !ctx || !start || B <= 0 || L <= 0 || S < L || past < 0 || past > R || ldp % vec || ok % vec || ov % vec)
    VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (int rc = check_ring(who, ring, r_ss, r_sh, R, hk, dim, vdim, vec)) return rc;
  ContextArgs a{p, ldp, ok, ov, ring, r_ss, r_sh, R, ctx, S, past, slots, start, (int)B, (int)L, hk, dim, vdim};
  const int64_t want = vy_cdiv(B * hk * S * ((dim + vdim) / vec), 256);
  const dim3 grid((unsigned)(want < 16384 ? want : 16384)), block(256);
  if (dtype == VY_BF16) hipLaunchKernelGGL((window_context_kernel<bf16>), grid, block, 0, (hipStream_t)stream, a);
  else hipLaunchKernelGGL((window_context_kernel<float>), grid, block, 0, (hipStream_t)stream, a);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}

extern "C" int64_t vy_window_decode_ws_bytes(int32_t B, int32_t h, int32_t hk, int32_t vdim, int32_t R) {
  if (B < 1 || h < 1 || hk < 1 || vdim < 1 || R < 1) return 0;
  const int ns = slices_of((int64_t)B * hk * ((h / hk + 15) / 16), R);
  return ns == 1 ? 0 : (int64_t)B * h * ns * (vdim + 2) * 4 + 256;
}

extern "C" int vy_window_decode(void* p, int64_t ldp, int64_t oq, int64_t ok, int64_t ov, int64_t og, void* ring, int64_t r_ss,
                                int64_t r_sh, int32_t R, const float* rope, int32_t rope_dims, int32_t rope_len,
                                const int32_t* slots, const int32_t* start, int64_t max_keys, void* out, int64_t ldo, int64_t B,
                                int32_t h, int32_t hk, int32_t dim, int32_t vdim, float scale, int32_t sink, void* ws,
                                int64_t ws_bytes, int dtype, void* stream) {
  const char* who = "vy_window_decode";
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!p || !out || !start || B <= 0 || h <= 0 || hk <= 0 || h % hk || max_keys < 1 || !(scale > 0.f))
    VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (ldp % vec || oq % vec || ok % vec || ov % vec || ldo % vec || (og >= 0 && og % vec))
    VY_FAIL(VY_ERR_ARG, "%s: columns and strides must be multiples of %d", who, vec);
  if (int rc = check_ring(who, ring, r_ss, r_sh, R, hk, dim, vdim, vec)) return rc;
  if (int rc = check_rope(who, rope, rope_dims, rope_len, dim)) return rc;
  if (rope_dims && max_keys > rope_len) VY_FAIL(VY_ERR_ARG, "%s: %ld positions, rotary table of %d", who, (long)max_keys, rope_len);
  hipStream_t st = (hipStream_t)stream;
  if (dtype == VY_F32 || dim > 256 || vdim > 256) {
    // row-wise kernel over the ring: the new row goes in first
    if (int rc = vy_window_rows(p, ldp, ok, ov, ring, r_ss, r_sh, R, rope, rope_dims, rope_len, 1, 1, slots, start, nullptr, B, 1,
                                hk, dim, vdim, dtype, stream)) return rc;
    const int64_t e = dtype == VY_BF16 ? 2 : 4;
    const vy_attn_window win{0, sink, 1, INT32_MAX, rope, rope_dims, rope_len};
    const char* gate = og >= 0 ? (const char*)p + og * e : nullptr;
    return vy_attn_fwd_ex((const char*)p + oq * e, ldp, dim, ldp, ring, r_ss, r_sh, dim + vdim, (const char*)ring + (int64_t)dim * e,
                          r_ss, r_sh, dim + vdim, out, ldo, ldo, gate, ldp, ldp, start, slots, B, h, hk, 1, R, dim, vdim, scale,
                          &win, dtype, stream);
  }
  DecodeArgs a{};
  a.p = (const bf16*)p; a.ldp = ldp; a.oq = oq; a.ok = ok; a.ov = ov; a.og = og;
  a.ring = (bf16*)ring; a.r_ss = r_ss; a.r_sh = r_sh; a.R = R;
  a.rope = (const float2*)rope; a.half = rope_dims / 2; a.rope_len = rope_len > 0 ? rope_len : 1;
  a.slots = slots; a.start = start; a.out = (bf16*)out; a.ldo = ldo;
  a.h = h; a.hk = hk; a.dim = dim; a.vdim = vdim; a.scale = scale; a.sink = sink;
  a.passes = (h / hk + 15) / 16;
  const int64_t rows = max_keys < R ? max_keys : R;
  a.ns = slices_of(B * hk * a.passes, rows);
  if (a.ns > 1) {
    const int64_t need = B * h * a.ns * ((int64_t)vdim + 2) * 4;
    if (!ws || ws_bytes < need || (uintptr_t)ws % 16) VY_FAIL(VY_ERR_ARG, "%s: workspace too small or unaligned", who);
    a.part_o = (float*)ws;
    a.part_ml = a.part_o + B * h * a.ns * (int64_t)vdim;
  }
  const dim3 grid((unsigned)a.ns, (unsigned)(hk * a.passes), (unsigned)B);
  if (dim <= 64) decode_go<64>(a, grid, st);
  else if (dim <= 128) decode_go<128>(a, grid, st);
  else decode_go<256>(a, grid, st);
  if (a.ns > 1) hipLaunchKernelGGL(window_finish_kernel, dim3((unsigned)h, (unsigned)B), dim3(256), 0, st, a);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}
