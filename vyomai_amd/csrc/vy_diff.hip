// Differential attention over prompts: a head's queries and keys are two maps side by side, each map a causal softmax attention of
// its own over the SAME values; with their outputs a1, a2
//   o = a1 - lambda a2 ,   out = o / rms(o) * out_scale        (rms over the head's value columns)
// Keys and values are read where they live, in the slot's ring, which holds every token of the sequence (a full-attention ring
// never wraps: row = position; vy_qkv_rows has put the new tokens there): rows [key 1 | key 2 | value] per key/value head.  So a
// prompt behind a past needs no copy of it.  Decode steps are vy_window_decode's.
//
// All kernels walk the keys once for both maps: one fetch of a row, one value fragment for two products.  Difference and norm are
// part of the epilogue, in fp32, on accumulators that were never rounded.
//   diff_mfma_kernel  bf16, heads whose two key maps together are as wide as their values, 64 or 128: attn_fwd_mfma_kernel's
//                     structure (vy_attn.hip) -- 128 query rows per workgroup, 64-key tiles through a three-deep LDS-DMA ring,
//                     swapped products on mfma_f32_32x32x16, probabilities in registers, transposing reads of the values
//   diff_gen_kernel   bf16, any widths up to 256: attn_fwd_gen_kernel's structure, 64 query rows, one tile in LDS
//   diff_row_kernel   fp32 and wider heads: a workgroup per query row and head, 256 keys at a time
#include "vy_window.h"

namespace {

using vy_window::LOG2E;
using vy_window::group_max;
using vy_window::group_sum;
using vy_window::rms_factor;

struct DiffArgs {
  const void* q; int64_t ldq;               // rows b L + l, head a at column a 2 dim
  const void* ring; int64_t r_ss, r_sh;
  const int* slots; const int* start; const int* count;
  void* out; int64_t ldo;
  int B, L, h, hk, dim, vdim, n_v;          // dim: columns of one map
  float scale, lambda, out_scale, eps;
};

// ---- two maps of DV / 2 columns, values of DV -------------------------------------------------
template <int DV>
__global__ __launch_bounds__(256, 1) void diff_mfma_kernel(DiffArgs p) {
  constexpr int RB = DV * 2;            // bytes per key pair / value row
  constexpr int TILE = 64 * RB;         // bytes per 64-key tile
  constexpr int NP = TILE / 1024 / 4;   // 1-KiB LDS-DMA pieces per wave per tile
  constexpr int KS = DV / 16;           // k-steps of both maps' contractions together
  constexpr int KM = KS / 2;            // of one
  constexpr int ND = DV / 32;           // 32-wide blocks of O^T (2 or 4)
  constexpr int NS = 3;                 // tiles in the ring
  __shared__ __attribute__((aligned(16))) char smem[2 * NS * TILE];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int head = (int)blockIdx.x % p.h, b = (int)blockIdx.x / p.h;   // (heaviest query blocks of every head first)
  const int q0 = ((int)gridDim.y - 1 - (int)blockIdx.y) * 128;
  const int fr = lane & 31, fh = lane >> 5;
  const int qi = q0 + wave * 32 + fr, qrow = min(qi, p.L - 1);
  const int slot = p.slots ? p.slots[b] : b;
  const int start = p.start[slot], S = start + (p.count ? min(p.count[b], p.L) : p.L);
  const int64_t W = 2 * DV;             // a row of the ring
  const bf16* Q = (const bf16*)p.q + ((int64_t)b * p.L + qrow) * p.ldq + head * DV;
  const bf16* Kb = (const bf16*)p.ring + (int64_t)slot * p.r_ss + (int64_t)(head / (p.h / p.hk)) * p.r_sh;
  const bf16* Vb = Kb + DV;

  // LDS-DMA source geometry: piece pc covers LDS bytes [pc * 1024, + 1024); swizzles as in attn_fwd_mfma_kernel
  int ld_row[NP], ld_koff[NP], ld_voff[NP];
#pragma unroll
  for (int t = 0; t < NP; ++t) {
    const int P = (wave * NP + t) * 1024 + lane * 16;
    const int row = P / RB, off = P % RB;
    const int ksw = RB == 128 ? (row >> 1) & 7 : row & 15;
    const int vsw = RB == 128 ? ((row >> 1) & 1) << 6 : (row & 3) << 6;
    ld_row[t] = row;
    ld_koff[t] = (((off >> 4) ^ ksw) << 4) >> 1;
    ld_voff[t] = (off ^ vsw) >> 1;
  }
  auto stage = [&](int tile, int buf) {
    const int k0 = tile * 64;
#pragma unroll
    for (int t = 0; t < NP; ++t) {
      const bf16* row = Kb + (int64_t)min(k0 + ld_row[t], S - 1) * W;   // (rows past the end: the last one, weight 0)
      __builtin_amdgcn_global_load_lds((const VY_GLOBAL void*)(row + ld_koff[t]),
                                       (VY_LDS void*)(smem + buf * TILE + (wave * NP + t) * 1024), 16, 0, 0);
      __builtin_amdgcn_global_load_lds((const VY_GLOBAL void*)(row + DV + ld_voff[t]),
                                       (VY_LDS void*)(smem + (NS + buf) * TILE + (wave * NP + t) * 1024), 16, 0, 0);
    }
  };
  const int k_sw = RB == 128 ? (fr >> 1) & 7 : fr & 15;
  const int li = lane & 15, g16 = (lane >> 4) & 1;
  const int v_sw = RB == 128 ? ((li >> 3) & 1) << 6 : ((li >> 2) & 3) << 6;
  const int v_lane_row = 4 * fh + (li >> 2), v_lane_off = 32 * g16 + 8 * (li & 3);
  unsigned k_lds[KS], v_lds[ND];
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) k_lds[ks] = vy_lds_addr(smem) + fr * RB + (((2 * ks + fh) ^ k_sw) << 4);
#pragma unroll
  for (int n = 0; n < ND; ++n) v_lds[n] = vy_lds_addr(smem) + v_lane_row * RB + ((64 * n + v_lane_off) ^ v_sw);

  f32x16 o[2][ND];
  float m_run[2], l_run[2];
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    m_run[m] = -FLT_MAX;
    l_run[m] = 0.f;
#pragma unroll
    for (int n = 0; n < ND; ++n)
#pragma unroll
      for (int r = 0; r < 16; ++r) o[m][n][r] = 0.f;
  }
  const float c = p.scale * LOG2E;
  const int nt = max(1, (min(S, start + q0 + 128) + 63) / 64);
  const int wave_first = q0 + wave * 32, wave_last = wave_first + 31;
  bf16x8 qf[KS];

  auto compute = [&](int tile, int buf) {
    const int k0 = tile * 64;
    if (k0 > start + wave_last) return;   // wave-uniform: wholly above this wave's diagonal
    // Hidden (asm) LDS reads retired by counted waits: map 1's key fragments first; behind each of its products one of map 2's is
    // requested, behind those the values'.  The products of map 1's probabilities with the values run under map 2's softmax.
    f32x16 st[2];
    bf16x8 kfr[2][KS];                    // [map][KM kb + k]
    auto kread = [&](auto m_c, auto i_c) {
      constexpr int m = decltype(m_c)::value, i = decltype(i_c)::value;
      kfr[m][i] = vy_lds_read128_off<(i / KM) * 32 * RB>(k_lds[m * KM + i % KM] + buf * TILE);
    };
    vy_static_for<KS>([&](auto i_c) { kread(std::integral_constant<int, 0>{}, i_c); });
    bf16x8 vfr[4 * ND];
    auto vread = [&](auto f_c) {
      constexpr int f = decltype(f_c)::value;
      if constexpr (f < 4 * ND) {
        constexpr int n = f >> 2, kb = (f >> 1) & 1, s_ = f & 1;
        vfr[f] = vy_lds_tr16_pair_off<NS * TILE + (32 * kb + 16 * s_) * RB, NS * TILE + (32 * kb + 16 * s_ + 8) * RB>(v_lds[n] + buf * TILE);
      }
    };
    constexpr int VPM = (4 * ND + KS - 1) / KS;   // value fragments requested behind each product of map 2
    const bool need_mask = k0 + 64 > S || k0 + 63 > start + wave_first;
    const int klim = min(S - 1, qi + start) - k0 - 4 * fh;   // register r of block kb: key k0 + 4 fh + 32 kb + (r & 3) + 8 (r >> 2)
    float neg_m;
    auto scores = [&](auto m_c) {
      constexpr int m = decltype(m_c)::value;
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int r = 0; r < 16; ++r) st[kb][r] = 0.f;
      vy_static_for<KS>([&](auto i_c) {
        constexpr int i = decltype(i_c)::value;
        constexpr int allow = (KS - 1 - i) + (m == 0 ? i : 2 * VPM * i);   // requested behind fragment i so far
        if constexpr (allow <= 15) asm volatile("s_waitcnt lgkmcnt(%0)" ::"n"(allow) : "memory");
        else asm volatile("s_waitcnt lgkmcnt(15)" ::: "memory");
        vy_tie(kfr[m][i]);
        st[i / KM] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kfr[m][i], qf[m * KM + i % KM], st[i / KM], 0, 0, 0);
        if constexpr (m == 0) kread(std::integral_constant<int, 1>{}, i_c);
        else vy_static_for<VPM>([&](auto j_c) { vread(std::integral_constant<int, i * VPM + decltype(j_c)::value>{}); });
      });
      if (need_mask) {
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
          for (int r = 0; r < 16; ++r) st[kb][r] = 32 * kb + (r & 3) + 8 * (r >> 2) > klim ? -INFINITY : st[kb][r];
      }
      float tmax = -INFINITY;
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int r = 0; r < 16; ++r) tmax = fmaxf(tmax, st[kb][r]);
      tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
      const float tmax_s = tmax * c;
      if (__any(tmax_s > m_run[m] + 8.f)) {   // lazy rescale: exp2 arguments stay <= 8
        const float m_new = fmaxf(m_run[m], tmax_s);
        const float alpha = __builtin_amdgcn_exp2f(m_run[m] - m_new);
        m_run[m] = m_new;
        l_run[m] *= alpha;
#pragma unroll
        for (int n = 0; n < ND; ++n)
#pragma unroll
          for (int r = 0; r < 16; ++r) o[m][n][r] *= alpha;
      }
      neg_m = -m_run[m];
    };
    bf16x8 pf[2][4];                          // [map][2 kb + half]
    auto weigh = [&](auto m_c, int i, float& rs) {   // probabilities i and i + 1 of the lane's 32
      constexpr int m = decltype(m_c)::value;
      const float e0 = __builtin_amdgcn_exp2f(fmaf(st[i >> 4][i & 15], c, neg_m));
      const float e1 = __builtin_amdgcn_exp2f(fmaf(st[i >> 4][(i & 15) + 1], c, neg_m));
      rs += e0 + e1;
      pf[m][i >> 3][i & 7] = (bf16)e0;
      pf[m][i >> 3][(i & 7) + 1] = (bf16)e1;
    };
    constexpr std::integral_constant<int, 0> map0{};
    constexpr std::integral_constant<int, 1> map1{};
    scores(map0);
    float rs = 0.f;
#pragma unroll
    for (int i = 0; i < 32; i += 2) weigh(map0, i, rs);
    l_run[0] += rs;                           // this half's keys; the halves are added at the end
    scores(map1);
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
    for (int f = 0; f < 4 * ND; ++f) vy_tie(vfr[f]);
    rs = 0.f;
    vy_static_for<16>([&](auto i_c) {
      constexpr int i = decltype(i_c)::value;
      weigh(map1, 2 * i, rs);
      vy_static_for<ND / 4 + (ND % 4 && (i & 1) ? 1 : 0)>([&](auto j_c) {
        constexpr int f = ND >= 4 ? i * (ND / 4) + decltype(j_c)::value : i >> 1;
        o[0][f >> 2] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vfr[f], pf[0][f & 3], o[0][f >> 2], 0, 0, 0);
      });
    });
    l_run[1] += rs;
#pragma unroll
    for (int f = 0; f < 4 * ND; ++f) o[1][f >> 2] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vfr[f], pf[1][f & 3], o[1][f >> 2], 0, 0, 0);
  };
  auto wait_tile = [&](int younger) {   // `younger` tiles (2 NP LDS-DMA instructions each) may stay in flight
    if (younger >= 1) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(2 * NP) : "memory");
    else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  };
#pragma unroll
  for (int s_ = 0; s_ < NS - 1; ++s_)
    if (s_ < nt) stage(s_, s_);
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) qf[ks] = *reinterpret_cast<const bf16x8*>(Q + ks * 16 + fh * 8);
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) asm volatile("" ::"v"(qf[ks]));   // retired here: a wait inside the loop would drain the ring
  for (int t = 0; t < nt; ++t) {
    wait_tile(min(NS - 2, nt - 1 - t));
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    if (t + NS - 1 < nt) stage(t + NS - 1, (t + NS - 1) % NS);   // the buffer tile t - 1 was read from
    compute(t, t % NS);
  }
  const float i1 = 1.f / (l_run[0] + __shfl_xor(l_run[0], 32, 64));
  const float i2 = p.lambda / (l_run[1] + __shfl_xor(l_run[1], 32, 64));
  float sq = 0.f;
#pragma unroll
  for (int n = 0; n < ND; ++n)
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const float d = o[0][n][r] * i1 - o[1][n][r] * i2;
      o[0][n][r] = d;
      sq = fmaf(d, d, sq);   // (padded value columns are zero)
    }
  sq += __shfl_xor(sq, 32, 64);
  const float f = rms_factor(sq, p.n_v, p.eps) * p.out_scale;
  // through LDS: whole 16-byte pieces of rows to memory
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
  constexpr int OROW = RB + 16, LPR = RB / 16;
  static_assert(4 * 32 * OROW <= 2 * NS * TILE, "the waves' rows fit over the ring");
  char* ot = smem + wave * (32 * OROW);
#pragma unroll
  for (int n = 0; n < ND; ++n)
#pragma unroll
    for (int rg = 0; rg < 4; ++rg) {
      bf16x4 w;
#pragma unroll
      for (int e = 0; e < 4; ++e) w[e] = (bf16)(o[0][n][4 * rg + e] * f);
      *reinterpret_cast<bf16x4*>(ot + fr * OROW + (32 * n + 8 * rg + 4 * fh) * 2) = w;
    }
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");   // wave-private
#pragma unroll
  for (int it = 0; it < 32 * LPR / 64; ++it) {
    const int r = (it * 64 + lane) / LPR, ch = (it * 64 + lane) % LPR, row = q0 + wave * 32 + r;
    const bf16x8 v = *reinterpret_cast<const bf16x8*>(ot + r * OROW + ch * 16);
    if (row < p.L) *reinterpret_cast<bf16x8*>((bf16*)p.out + ((int64_t)b * p.L + row) * p.ldo + head * DV + ch * 8) = v;
  }
}

// ---- any widths up to 256 --------------------------------------------------------------------
template <int DHP, int DVP>
__global__ __launch_bounds__(256) void diff_gen_kernel(DiffArgs p) {
  constexpr int KPITCH = (DHP + 8) * 2, VPITCH = (DVP + 8) * 2;   // bytes per LDS row
  constexpr int KS = DHP / 32, NDB = DVP / 16, KCPR = DHP / 8, VCPR = DVP / 8;
  constexpr int KCPT = 2 * 64 * KCPR / 256, VCPT = 64 * VCPR / 256;   // 16-byte chunks per thread and tile
  __shared__ __attribute__((aligned(16))) char smem[64 * (2 * KPITCH + VPITCH)];
  char* kt = smem;                       // [map][key]
  char* vt = smem + 2 * 64 * KPITCH;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r16 = lane & 15, kq = lane >> 4;
  const int head = (int)blockIdx.x % p.h, b = (int)blockIdx.x / p.h;
  const int q0 = ((int)gridDim.y - 1 - (int)blockIdx.y) * 64;
  const int qi = q0 + wave * 16 + r16, qrow = min(qi, p.L - 1);
  const int slot = p.slots ? p.slots[b] : b;
  const int start = p.start[slot], S = start + (p.count ? min(p.count[b], p.L) : p.L);
  const int W = 2 * p.dim + p.vdim;
  const bf16* Q = (const bf16*)p.q + ((int64_t)b * p.L + qrow) * p.ldq + head * 2 * p.dim;
  const bf16* Kb = (const bf16*)p.ring + (int64_t)slot * p.r_ss + (int64_t)(head / (p.h / p.hk)) * p.r_sh;
  const bf16x8 zero8 = {};
  bf16x8 qf[2][KS];
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d0 = 32 * ks + 8 * kq;
      qf[m][ks] = d0 < p.dim ? *reinterpret_cast<const bf16x8*>(Q + m * p.dim + d0) : zero8;
    }
  f32x4 o[2][NDB];
  float m_run[2], l_run[2];
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    m_run[m] = -FLT_MAX;
    l_run[m] = 0.f;
#pragma unroll
    for (int n = 0; n < NDB; ++n) o[m][n] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const float c = p.scale * LOG2E;
  const int nt = max(1, (min(S, start + q0 + 64) + 63) / 64);
  const unsigned vtr = vy_lds_addr(vt) + (4 * kq + (r16 >> 2)) * VPITCH + (4 * (r16 & 3)) * 2;
  for (int t = 0; t < nt; ++t) {
    const int k0 = t * 64;
    bf16x8 kreg[KCPT], vreg[VCPT];
#pragma unroll
    for (int i = 0; i < KCPT; ++i) {
      const int x = tid + 256 * i, d0 = x % KCPR * 8, m = x / KCPR & 1, row = x / (2 * KCPR);
      kreg[i] = d0 < p.dim ? *reinterpret_cast<const bf16x8*>(Kb + (int64_t)min(k0 + row, S - 1) * W + m * p.dim + d0) : zero8;
    }
#pragma unroll
    for (int i = 0; i < VCPT; ++i) {
      const int x = tid + 256 * i, d0 = x % VCPR * 8, row = x / VCPR;   // (rows past the end: the last one, weight 0)
      vreg[i] = d0 < p.vdim ? *reinterpret_cast<const bf16x8*>(Kb + (int64_t)min(k0 + row, S - 1) * W + 2 * p.dim + d0) : zero8;
    }
    __syncthreads();   // the previous tile's fragments have been read
#pragma unroll
    for (int i = 0; i < KCPT; ++i) {
      const int x = tid + 256 * i;
      *reinterpret_cast<bf16x8*>(kt + ((x / KCPR & 1) * 64 + x / (2 * KCPR)) * KPITCH + (x % KCPR) * 16) = kreg[i];
    }
#pragma unroll
    for (int i = 0; i < VCPT; ++i) {
      const int x = tid + 256 * i;
      *reinterpret_cast<bf16x8*>(vt + (x / VCPR) * VPITCH + (x % VCPR) * 16) = vreg[i];
    }
    __syncthreads();
    bf16x8 pf[2][2];
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      f32x4 sc[4];
#pragma unroll
      for (int blk = 0; blk < 4; ++blk) {
        sc[blk] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          const bf16x8 kf = *reinterpret_cast<const bf16x8*>(kt + (m * 64 + 16 * blk + r16) * KPITCH + (32 * ks + 8 * kq) * 2);
          sc[blk] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[m][ks], sc[blk], 0, 0, 0);
        }
      }
      float tmax = -INFINITY;
#pragma unroll
      for (int blk = 0; blk < 4; ++blk)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int kj = k0 + 16 * blk + 4 * kq + r;
          sc[blk][r] = kj < S && kj <= qi + start ? sc[blk][r] : -INFINITY;
          tmax = fmaxf(tmax, sc[blk][r]);
        }
      const float m_new = fmaxf(m_run[m], group_max(tmax) * c);   // (-inf * c stays -inf; m_run is finite)
      const float alpha = __builtin_amdgcn_exp2f(m_run[m] - m_new);
      m_run[m] = m_new;
      l_run[m] *= alpha;
#pragma unroll
      for (int n = 0; n < NDB; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[m][n][r] *= alpha;
#pragma unroll
      for (int blk = 0; blk < 4; ++blk)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float e = __builtin_amdgcn_exp2f(fmaf(sc[blk][r], c, -m_run[m]));
          l_run[m] += e;
          pf[m][blk >> 1][4 * (blk & 1) + r] = (bf16)e;
        }
    }
#pragma unroll
    for (int tt = 0; tt < 2; ++tt)
      vy_static_for<NDB>([&](auto n_c) {
        constexpr int n = decltype(n_c)::value;
        union { struct { s16x4 a, b; } h; bf16x8 v; } u;
        u.h.a = vy_lds_tr16_off<n * 32>(vtr + (32 * tt) * VPITCH);
        u.h.b = vy_lds_tr16_off<n * 32>(vtr + (32 * tt + 16) * VPITCH);
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        vy_tie(u.v);
        o[0][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(u.v, pf[0][tt], o[0][n], 0, 0, 0);
        o[1][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(u.v, pf[1][tt], o[1][n], 0, 0, 0);
      });
  }
  const float i1 = 1.f / group_sum(l_run[0]), i2 = p.lambda / group_sum(l_run[1]);
  float sq = 0.f;
#pragma unroll
  for (int n = 0; n < NDB; ++n)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float d = o[0][n][r] * i1 - o[1][n][r] * i2;
      o[0][n][r] = d;
      sq = fmaf(d, d, sq);
    }
  const float f = rms_factor(group_sum(sq), p.n_v, p.eps) * p.out_scale;
  if (qi < p.L) {
    bf16* orow = (bf16*)p.out + ((int64_t)b * p.L + qi) * p.ldo + head * p.vdim;
#pragma unroll
    for (int n = 0; n < NDB; ++n) {
      const int d0 = 16 * n + 4 * kq;
      if (d0 < p.vdim) {
        bf16x4 w;
#pragma unroll
        for (int r = 0; r < 4; ++r) w[r] = (bf16)(o[0][n][r] * f);
        *reinterpret_cast<bf16x4*>(orow + d0) = w;
      }
    }
  }
}

// ---- row by row ------------------------------------------------------------------------------
// 256 keys at a time: a thread per key for both scores, then a thread per value column (256 / cols groups of keys)
constexpr int ROW_DIM = 1024;   // most columns of a map, and of the values
template <typename T>
__global__ __launch_bounds__(256) void diff_row_kernel(DiffArgs p) {
  constexpr int VEC = VyChunk<T>::VEC;
  __shared__ __attribute__((aligned(16))) float qs[2 * ROW_DIM];
  __shared__ float pr[2][256], red[2][4], acc[2][256];
  const int tid = threadIdx.x, wave = tid >> 6;
  const int qi = blockIdx.x, head = blockIdx.y, b = blockIdx.z;
  const int slot = p.slots ? p.slots[b] : b;
  const int start = p.start[slot], S = start + (p.count ? min(p.count[b], p.L) : p.L), n = min(S, start + qi + 1);
  const int W = 2 * p.dim + p.vdim;
  const T* Q = (const T*)p.q + ((int64_t)b * p.L + qi) * p.ldq + (int64_t)head * 2 * p.dim;
  const T* Kb = (const T*)p.ring + (int64_t)slot * p.r_ss + (int64_t)(head / (p.h / p.hk)) * p.r_sh;
  for (int i = tid; i < 2 * p.dim; i += 256) qs[i] = VyT<T>::ld(Q + i);
  int cols = 1;                          // threads per key group of the value sums
  while (cols < p.vdim && cols < 256) cols <<= 1;
  const int grp = tid / cols, groups = 256 / cols, col = tid % cols, NC = (p.vdim + cols - 1) / cols;
  constexpr int MC = ROW_DIM / 256;
  float o[2][MC] = {}, m[2] = {-FLT_MAX, -FLT_MAX}, l[2] = {0.f, 0.f};
  __syncthreads();
  auto both = [&](float (&v)[2], bool max) {   // over the workgroup
#pragma unroll
    for (int x = 0; x < 2; ++x) v[x] = max ? vy_wave_max(v[x]) : vy_wave_sum(v[x]);
    __syncthreads();
    if ((tid & 63) == 0) { red[0][wave] = v[0]; red[1][wave] = v[1]; }
    __syncthreads();
#pragma unroll
    for (int x = 0; x < 2; ++x)
      v[x] = max ? fmaxf(fmaxf(red[x][0], red[x][1]), fmaxf(red[x][2], red[x][3])) : red[x][0] + red[x][1] + red[x][2] + red[x][3];
  };
  for (int k0 = 0; k0 < n; k0 += 256) {
    const int kj = k0 + tid;
    float s[2] = {-FLT_MAX, -FLT_MAX};
    if (kj < n) {
      const T* k = Kb + (int64_t)kj * W;
#pragma unroll
      for (int x = 0; x < 2; ++x) {
        float d = 0.f;
        for (int c = 0; c < p.dim; c += VEC) {
          float v[VEC];
          VyChunk<T>::load(k + x * p.dim + c, v);
#pragma unroll
          for (int e = 0; e < VEC; ++e) d = fmaf(qs[x * p.dim + c + e], v[e], d);
        }
        s[x] = d * p.scale;
      }
    }
    float top[2] = {s[0], s[1]};
    both(top, true);
    float e[2];
#pragma unroll
    for (int x = 0; x < 2; ++x) {
      const float mn = fmaxf(m[x], top[x]), alpha = expf(m[x] - mn);
      m[x] = mn;
      e[x] = kj < n ? expf(s[x] - mn) : 0.f;
      pr[x][tid] = e[x];
      l[x] = l[x] * alpha + e[x];
#pragma unroll
      for (int c = 0; c < MC; ++c) o[x][c] *= alpha;
    }
    __syncthreads();
    const int last = min(256, n - k0);
    for (int j = grp; j < last; j += groups) {
      const T* v = Kb + (int64_t)(k0 + j) * W + 2 * p.dim;
#pragma unroll
      for (int c = 0; c < MC; ++c) {
        const int d = col + 256 * c;     // (NC > 1 only with cols = 256)
        if (c < NC && d < p.vdim) {
          const float x = VyT<T>::ld(v + d);
          o[0][c] = fmaf(pr[0][j], x, o[0][c]);
          o[1][c] = fmaf(pr[1][j], x, o[1][c]);
        }
      }
    }
  }
  both(l, false);
  float diff[MC], sq[2] = {0.f, 0.f};
#pragma unroll
  for (int c = 0; c < MC; ++c) {
    diff[c] = 0.f;
    if (c < NC) {                        // workgroup-uniform
      __syncthreads();
      acc[0][tid] = o[0][c];
      acc[1][tid] = o[1][c];
      __syncthreads();
      if (grp == 0 && col + 256 * c < p.vdim) {
        float a1 = 0.f, a2 = 0.f;
        for (int g = 0; g < groups; ++g) {
          a1 += acc[0][g * cols + col];
          a2 += acc[1][g * cols + col];
        }
        diff[c] = a1 / l[0] - p.lambda * (a2 / l[1]);
        sq[0] = fmaf(diff[c], diff[c], sq[0]);
      }
    }
  }
  both(sq, false);
  const float f = rms_factor(sq[0], p.n_v, p.eps) * p.out_scale;
  T* orow = (T*)p.out + ((int64_t)b * p.L + qi) * p.ldo + (int64_t)head * p.vdim;
#pragma unroll
  for (int c = 0; c < MC; ++c)
    if (c < NC && grp == 0 && col + 256 * c < p.vdim) VyT<T>::st(orow + col + 256 * c, diff[c] * f);
}

template <int DHP>
void gen_go(const DiffArgs& a, dim3 grid, hipStream_t st) {
  const dim3 block(256);
  if (a.vdim <= 64) hipLaunchKernelGGL((diff_gen_kernel<DHP, 64>), grid, block, 0, st, a);
  else if (a.vdim <= 128) hipLaunchKernelGGL((diff_gen_kernel<DHP, 128>), grid, block, 0, st, a);
  else hipLaunchKernelGGL((diff_gen_kernel<DHP, 256>), grid, block, 0, st, a);
}

}  // namespace

extern "C" int vy_diff_attn_fwd(const void* q, int64_t ldq, const void* ring, int64_t r_ss, int64_t r_sh, int32_t R, const vy_diff* diff,
                                const int32_t* slots, const int32_t* start, const int32_t* count, void* out, int64_t ldo, int64_t B,
                                int64_t L, int32_t h, int32_t hk, int32_t dim, int32_t vdim, float scale, int dtype, void* stream) {
  const char* who = "vy_diff_attn_fwd";
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!q || !ring || !diff || !start || !out || B <= 0 || L <= 0 || h <= 0 || hk <= 0 || h % hk || dim <= 0 || vdim <= 0 || !(scale > 0.f) ||
      L > R || L > INT32_MAX || B * h > INT32_MAX || B > 65535 || h > 65535)
    VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (dim % (2 * vec) || vdim % vec || ldq % vec || ldo % vec || r_ss % vec || r_sh % vec || (uintptr_t)q % 16 || (uintptr_t)out % 16 ||
      (uintptr_t)ring % 16 || ldq < (int64_t)h * dim || ldo < (int64_t)h * vdim)
    VY_FAIL(VY_ERR_ARG, "%s: widths and strides must be multiples of %d", who, vec);
  if (r_sh < (int64_t)R * (dim + vdim) || r_ss < hk * r_sh) VY_FAIL(VY_ERR_ARG, "%s: ring strides do not hold %d rows", who, R);
  if (diff->n_v < 1 || diff->n_v > vdim) VY_FAIL(VY_ERR_ARG, "%s: norm over %d of %d columns", who, diff->n_v, vdim);
  hipStream_t st = (hipStream_t)stream;
  const DiffArgs a{q, ldq, ring, r_ss, r_sh, slots, start, count, out, ldo, (int)B, (int)L, h, hk, dim / 2, vdim, diff->n_v,
                   scale, diff->lambda, diff->out_scale, diff->eps};
  const dim3 block(256);
  if (dtype == VY_BF16 && L > 1 && dim == vdim && (vdim == 64 || vdim == 128)) {
    const dim3 grid((unsigned)(h * B), (unsigned)((L + 127) / 128));
    if (vdim == 64) hipLaunchKernelGGL(diff_mfma_kernel<64>, grid, block, 0, st, a);
    else hipLaunchKernelGGL(diff_mfma_kernel<128>, grid, block, 0, st, a);
  } else if (dtype == VY_BF16 && L > 1 && a.dim <= 256 && vdim <= 256) {
    const dim3 grid((unsigned)(h * B), (unsigned)((L + 63) / 64));
    if (a.dim <= 32) gen_go<32>(a, grid, st);
    else if (a.dim <= 64) gen_go<64>(a, grid, st);
    else if (a.dim <= 128) gen_go<128>(a, grid, st);
    else gen_go<256>(a, grid, st);
  } else {
    if (a.dim > ROW_DIM || vdim > ROW_DIM) VY_FAIL(VY_ERR_UNSUPPORTED, "%s: heads of 2 x %d and %d columns", who, a.dim, vdim);
    const dim3 grid((unsigned)L, (unsigned)h, (unsigned)B);
    if (dtype == VY_BF16) hipLaunchKernelGGL(diff_row_kernel<bf16>, grid, block, 0, st, a);
    else hipLaunchKernelGGL(diff_row_kernel<float>, grid, block, 0, st, a);
  }
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}
