// Decode attention over a latent cache: one row c_j of R values per token serves every head as key AND value.
//
//   keys are W_uk,h c_j and values W_uv,h c_j, so the score of head h is q_h . (W_uk,h c_j) = (W_uk,h^T q_h) . c_j and the
//   output W_uv,h (sum_j p_j c_j): the query is taken into the latent space once, the cache is streamed once for all heads
//   (a multi-query problem whose keys and values are the same bytes), and the mean latent is expanded at the end.
//
// Three launches: latent_query_kernel (per-head W_uk^T q), latent_scan_kernel (flash attention over a slice of the keys,
// fp32 partial sums), latent_value_kernel (adds the slices, expands with W_uv, applies the sigmoid output gate).
// Precision: scores take the latent query as TWO bf16 numbers (hi + lo, ~16 bits of mantissa), so taking the query through
// W_uk costs no accuracy against expanding the keys; likewise the mean latent in front of W_uv.
//
// f32 (and bf16 latents wider than 512): the same three steps with plain fp32 FMAs.
#include "vy_common.h"
#include <float.h>

namespace {

constexpr float LOG2E = 1.4426950408889634f;
constexpr int MAX_SPLIT = 64;      // slices of the key range

struct LatentArgs {
  const void* q; int64_t ldq;
  const void* wukt; const void* wuv;
  const void* cache; int64_t c_ss, c_st;
  const int* slots; const int* start;
  void* out; int64_t ldo;
  const void* gate; int64_t ldg;
  int B, h, dh, dv, R, nsplit, seqs;
  int ring, gate_heads;            // rows of a slot's ring (0: rows are positions); one gate per head
  float c;                         // scale * log2(e)
  // workspace
  float* qf;                       // generic: latent queries [B][h][R]
  bf16* qhi; bf16* qlo;            // MFMA: the same as two bf16 halves
  float* part_o; float* part_ml;   // [B][h][nsplit][R], [B][h][nsplit][2]
};

__device__ __forceinline__ int row_keys(const LatentArgs& p, int b, int& slot) {
  slot = p.slots ? p.slots[b] : b;
  const int n = p.start[slot] + 1;
  return p.ring ? min(n, p.ring) : n;   // (every row of a ring is inside the window: order does not matter)
}
// combine over the four lane groups (lane >> 4) of a 16 x 16 MFMA layout
__device__ __forceinline__ float quad_max(float v) {
  v = fmaxf(v, __shfl_xor(v, 16, 64));
  return fmaxf(v, __shfl_xor(v, 32, 64));
}
__device__ __forceinline__ float quad_sum(float v) {
  v += __shfl_xor(v, 16, 64);
  return v + __shfl_xor(v, 32, 64);
}
__device__ __forceinline__ void split_bf16(float x, bf16& hi, bf16& lo) {
  const float h = vy_round_bf16(x);
  hi = (bf16)h;
  lo = (bf16)(x - h);
}

// ---- MFMA path ------------------------------------------------------------------------------
// q~[b][h][r] = sum_d W_uk^T[h][r][d] q[b][h][d]: workgroup = 64 latent columns of one head x 16 sequences
__global__ __launch_bounds__(256) void latent_query_kernel(LatentArgs p) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int r16 = lane & 15, kq = lane >> 4;
  const int head = blockIdx.y, b = (int)blockIdx.z * 16 + r16;
  const int r0 = (int)blockIdx.x * 64 + wave * 16;
  const bf16x8 zero8 = {};
  const bool wok = r0 + r16 < p.R, xok = b < p.B;
  const bf16* w = (const bf16*)p.wukt + ((int64_t)head * p.R + (wok ? r0 + r16 : 0)) * p.dh;
  const bf16* x = (const bf16*)p.q + (int64_t)(xok ? b : 0) * p.ldq + head * p.dh;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < p.dh; k0 += 128) {
    bf16x8 wf[4], xf[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int k = k0 + 32 * u + 8 * kq;
      const bool ok = k < p.dh;
      wf[u] = ok && wok ? *reinterpret_cast<const bf16x8*>(w + k) : zero8;
      xf[u] = ok && xok ? *reinterpret_cast<const bf16x8*>(x + k) : zero8;
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[u], xf[u], acc, 0, 0, 0);
  }
  const int r = r0 + 4 * kq;   // R is a multiple of 8: the quad is inside or outside as a whole
  if (xok && r < p.R) {
    bf16x4 hi, lo;
#pragma unroll
    for (int e = 0; e < 4; ++e) { bf16 a, c; split_bf16(acc[e], a, c); hi[e] = a; lo[e] = c; }
    const int64_t o = ((int64_t)b * p.h + head) * p.R + r;
    *reinterpret_cast<bf16x4*>(p.qhi + o) = hi;
    *reinterpret_cast<bf16x4*>(p.qlo + o) = lo;
  }
}

// asm forms of the score exchange: while LDS-DMA is in flight hipcc drains it (vmcnt(0)) in front of every LDS access it can
// see; these are retired by counted / explicit waits instead (vy_common.h)
__device__ __forceinline__ void lds_write4(unsigned addr, f32x4 v) {
  asm volatile("ds_write_b128 %0, %1" ::"v"(addr), "v"(v) : "memory");
}
__device__ __forceinline__ bf16x8 lds_read16(unsigned addr) { return vy_lds_read128_off<0>(addr); }

// grid (slices, head groups of 16, B); 4 waves share tiles of KT keys that LDS-DMA brings through a ring of NS buffers.
//   scores  S^T = c q~^T, swapped as in attn_fwd_gen_kernel: one head per lane column, four consecutive keys per lane
//           group.  A wave takes one block of 16 keys (KT = 64) or half of the contraction of one block (KT = 32); the
//           scores are exchanged through LDS, and every wave then holds the same running maximum and sum;
//   mean    U^T += c^T P^T: a wave owns RP / 4 of the latent columns, so nothing is combined across waves at the end.  The
//           same LDS tile serves both products: row reads for the scores, transposing reads for the mean.
// Rows are XOR-swizzled in 16-byte chunks with the low bits of the key index (applied to the DMA's source address).
template <int RP>
__global__ __launch_bounds__(256) void latent_scan_kernel(LatentArgs p) {
  constexpr int KT = RP >= 512 ? 32 : 64;     // keys per tile
  constexpr int NS = RP >= 512 ? 4 : RP >= 256 ? 2 : 3;
  constexpr int RB = RP * 2;                  // bytes per row
  constexpr int TILE = KT * RB;
  constexpr int NP = TILE / 1024 / 4;         // 1-KiB pieces per wave and tile
  constexpr int CPR = RP / 8;                 // 16-byte chunks per row
  constexpr int SWZ = CPR < 16 ? CPR - 1 : 15;
  constexpr int KH = KT == 32 ? 2 : 1;        // waves per key block
  constexpr int KS = RP / 32 / KH;            // k-steps of a wave
  constexpr int ND = RP / 64;                 // 16-wide latent blocks of a wave
  constexpr int SP = (KT + 4) * 4;            // bytes per score row (head)
  __shared__ __attribute__((aligned(16))) char smem[NS * TILE + KH * 16 * SP];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r16 = lane & 15, kq = lane >> 4;
  const int b = blockIdx.z, split = blockIdx.x;
  const int head = (int)blockIdx.y * 16 + r16;
  int slot;
  const int n = row_keys(p, b, slot);
  const int tiles = (n + KT - 1) / KT;
  const int tps = (tiles + p.nsplit - 1) / p.nsplit;
  const int t0 = split * tps, nt = max(0, min(tiles, t0 + tps) - t0);
  const bf16* Cs = (const bf16*)p.cache + (int64_t)slot * p.c_ss;

  int ld_row[NP], ld_col[NP];                 // row and source column (< 0: padding) of this lane's 16 bytes of a piece
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    const int P = (wave * NP + i) * 1024 + lane * 16;
    ld_row[i] = P / RB;
    const int ch = ((P % RB) >> 4) ^ (ld_row[i] & SWZ);
    ld_col[i] = ch * 8 < p.R ? ch * 8 : -1;
  }
  auto stage = [&](int t) {
    const int k0 = (t0 + t) * KT;
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int kj = min(k0 + ld_row[i], n - 1);
      const void* src = ld_col[i] < 0 ? (const void*)vy_zero16 : (const void*)(Cs + (int64_t)kj * p.c_st + ld_col[i]);
      __builtin_amdgcn_global_load_lds((const VY_GLOBAL void*)src,
                                       (VY_LDS void*)(smem + (t % NS) * TILE + (wave * NP + i) * 1024), 16, 0, 0);
    }
  };
  const int kblk = KH == 2 ? wave & 1 : wave, khalf = KH == 2 ? wave >> 1 : 0;
  bf16x8 qh[KS], ql[KS];
  const int64_t qo = ((int64_t)b * p.h + (head < p.h ? head : 0)) * p.R;
  const bf16x8 zero8 = {};
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) {
    const int k = 32 * (khalf * KS + ks) + 8 * kq;
    const bool ok = k < p.R && head < p.h;
    qh[ks] = ok ? *reinterpret_cast<const bf16x8*>(p.qhi + qo + k) : zero8;
    ql[ks] = ok ? *reinterpret_cast<const bf16x8*>(p.qlo + qo + k) : zero8;
  }
  // The ring is filled behind the query loads (without conditions, so that their wait can be counted: rows past the end are
  // clamped), and the queries are retired before the loop: a wait for them inside it would drain the ring.
#pragma unroll
  for (int t = 0; t < NS - 1; ++t) stage(t);
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) { asm volatile("" ::"v"(qh[ks])); asm volatile("" ::"v"(ql[ks])); }

  const unsigned base = vy_lds_addr(smem), sbase = base + NS * TILE;
  const int krow = 16 * kblk + r16;
  unsigned ka[KS];                            // score fragments: key row krow, chunk 4 ks + kq
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) ka[ks] = base + krow * RB + (((4 * (khalf * KS + ks) + kq) ^ (krow & SWZ)) << 4);
  const int vrow = 4 * kq + (r16 >> 2);       // mean fragments: rows vrow and vrow + 16 (same swizzle), 8 bytes per lane
  unsigned va[ND];
#pragma unroll
  for (int i = 0; i < ND; ++i) {
    const int ch = 2 * (wave * ND + i) + ((r16 & 3) >> 1);
    va[i] = base + vrow * RB + ((ch ^ (vrow & SWZ)) << 4) + (r16 & 1) * 8;
  }
  const unsigned sw_addr = sbase + khalf * 16 * SP + r16 * SP + (16 * kblk + 4 * kq) * 4;
  const unsigned sr_addr = sbase + r16 * SP + 4 * kq * 4;

  f32x4 o[ND];
#pragma unroll
  for (int i = 0; i < ND; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = -FLT_MAX, l_run = 0.f;

  for (int t = 0; t < nt; ++t) {
    const int younger = min(NS - 2, nt - 1 - t);      // tiles that may stay in flight
    if (NS >= 4 && younger >= 2) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(2 * NP) : "memory");
    else if (NS >= 3 && younger >= 1) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(NP) : "memory");
    else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    if (t + NS - 1 < nt) stage(t + NS - 1);           // into the buffer tile t - 1 was read from
    const unsigned buf = (t % NS) * TILE;
    f32x4 sh = {0.f, 0.f, 0.f, 0.f}, sl = {0.f, 0.f, 0.f, 0.f};
    bf16x8 kf[KS];
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) kf[ks] = lds_read16(ka[ks] + buf);
    vy_static_for<KS>([&](auto i_c) {
      constexpr int i = decltype(i_c)::value;
      constexpr int left = KS - 1 - i;
      if constexpr (left <= 15) asm volatile("s_waitcnt lgkmcnt(%0)" ::"n"(left) : "memory");
      vy_tie(kf[i]);
      sh = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[i], qh[i], sh, 0, 0, 0);
      sl = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[i], ql[i], sl, 0, 0, 0);
    });
    lds_write4(sw_addr, sh + sl);
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    // scores of every key of the tile for this lane's head, in the key order of the transposed fragments
    bf16x8 raw[KT / 16][KH];
#pragma unroll
    for (int g = 0; g < KT / 16; ++g)
#pragma unroll
      for (int hf = 0; hf < KH; ++hf) raw[g][hf] = lds_read16(sr_addr + hf * 16 * SP + g * 64);
    bf16x8 vf[KT / 32][ND];
    vy_static_for<KT / 32>([&](auto t_c) {
      constexpr int tt = decltype(t_c)::value;
#pragma unroll
      for (int i = 0; i < ND; ++i) vf[tt][i] = vy_lds_tr16_pair_off<32 * tt * RB, (32 * tt + 16) * RB>(va[i] + buf);
    });
    // (lgkmcnt has 4 bits: the scores are the oldest reads, the transposed fragments behind them may stay in flight)
    constexpr int behind = 2 * ND * (KT / 32);
    if constexpr (behind <= 15) asm volatile("s_waitcnt lgkmcnt(%0)" ::"n"(behind) : "memory");
    else asm volatile("s_waitcnt lgkmcnt(15)" ::: "memory");
    float sc[KT / 16][4];
    float tmax = -INFINITY;
    const int kbase = (t0 + t) * KT + 4 * kq;
#pragma unroll
    for (int g = 0; g < KT / 16; ++g) {
#pragma unroll
      for (int hf = 0; hf < KH; ++hf) vy_tie(raw[g][hf]);
      f32x4 v = __builtin_bit_cast(f32x4, raw[g][0]);
      if constexpr (KH == 2) v += __builtin_bit_cast(f32x4, raw[g][KH - 1]);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        sc[g][r] = kbase + 16 * g + r < n ? v[r] * p.c : -INFINITY;
        tmax = fmaxf(tmax, sc[g][r]);
      }
    }
    const float m_new = fmaxf(m_run, quad_max(tmax));
    if (__any(m_new > m_run)) {
      const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
      m_run = m_new;
      l_run *= alpha;
#pragma unroll
      for (int i = 0; i < ND; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[i][r] *= alpha;
    }
    bf16x8 pf[KT / 32];
#pragma unroll
    for (int g = 0; g < KT / 16; ++g)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float e = __builtin_amdgcn_exp2f(sc[g][r] - m_run);
        l_run += e;
        pf[g >> 1][4 * (g & 1) + r] = (bf16)e;
      }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
    for (int tt = 0; tt < KT / 32; ++tt)
#pragma unroll
      for (int i = 0; i < ND; ++i) {
        vy_tie(vf[tt][i]);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[tt][i], pf[tt], o[i], 0, 0, 0);
      }
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");   // tiles requested past the slice's end
  if (head < p.h) {
    const int64_t o_ = ((int64_t)b * p.h + head) * p.nsplit + split;
    const float l = quad_sum(l_run);
    if (wave == 0 && kq == 0) { p.part_ml[o_ * 2] = m_run; p.part_ml[o_ * 2 + 1] = l; }
#pragma unroll
    for (int i = 0; i < ND; ++i) {
      const int col = 16 * (wave * ND + i) + 4 * kq;
      if (col < p.R) *reinterpret_cast<f32x4*>(p.part_o + o_ * p.R + col) = o[i];
    }
  }
}

// weights of the slices of one (b, head): exp2(m_s - M) / L, 0 for an empty slice
__device__ __forceinline__ void slice_weights(const LatentArgs& p, int b, int head, float* w, int lane) {
  const float* ml = p.part_ml + ((int64_t)b * p.h + head) * p.nsplit * 2;
  const float m = lane < p.nsplit ? ml[2 * lane] : -FLT_MAX;
  const float l = lane < p.nsplit ? ml[2 * lane + 1] : 0.f;
  const float M = vy_wave_max(l > 0.f ? m : -FLT_MAX);
  const float e = l > 0.f ? __builtin_amdgcn_exp2f(m - M) : 0.f;
  const float L = vy_wave_sum(e * l);
  if (lane < p.nsplit) w[lane] = e / L;
}

// out[b][h][n] = (W_uv,h u_bh)_n * sigmoid(gate): workgroup = 64 value columns of one head x p.seqs (<= 16) sequences; the
// mean latents are added up from the slices into LDS first (few sequences: the slices are shared out over the threads)
// (RP: padded latent width.  The weights of the product are requested before anything else: one memory latency beside the
// slices', not one after another behind them.)
template <int RP>
__global__ __launch_bounds__(256) void latent_value_kernel(LatentArgs p) {
  extern __shared__ __attribute__((aligned(16))) char dyn[];
  constexpr int PITCH = (RP + 8) * 2, KS = RP / 32;
  float* sw = reinterpret_cast<float*>(dyn);                       // [seqs][MAX_SPLIT]
  f32x4* acc4 = reinterpret_cast<f32x4*>(dyn + p.seqs * MAX_SPLIT * 4);   // [256]
  char* xh = dyn + p.seqs * MAX_SPLIT * 4 + 4096;
  char* xl = xh + p.seqs * PITCH;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int r16 = lane & 15, kq = lane >> 4;
  const int head = blockIdx.y, b0 = (int)blockIdx.z * p.seqs;
  const int nb = min(p.seqs, p.B - b0);
  const bf16x8 zero8 = {};
  const int n0 = (int)blockIdx.x * 64 + wave * 16;
  const bool wok = n0 + r16 < p.dv;
  bf16x8 wf[KS];
  {
    const bf16* w = (const bf16*)p.wuv + ((int64_t)head * p.dv + (wok ? n0 + r16 : 0)) * p.R;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int k = 32 * ks + 8 * kq;
      wf[ks] = wok && k < p.R ? *reinterpret_cast<const bf16x8*>(w + k) : zero8;
    }
  }
  for (int i = wave; i < nb; i += 4) slice_weights(p, b0 + i, head, sw + i * MAX_SPLIT, lane);
  __syncthreads();
  constexpr int q4 = RP / 4;
  const int items = nb * q4;
  const int G = items >= 256 ? 1 : 256 / items;                    // groups of slices
  for (int base = 0; base < items; base += 256) {
    const int g = G > 1 ? (int)threadIdx.x / items : 0;
    const int idx = base + (int)threadIdx.x - g * items;
    const bool live = idx < items && g < G;
    const int i = live ? idx / q4 : 0, col = (idx - i * q4) * 4;
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
    if (live && col < p.R) {
      // batches of UB loads, all requested before the first is used (slices past the end: the last one, weight 0)
      const float* po = p.part_o + ((int64_t)(b0 + i) * p.h + head) * p.nsplit * p.R + col;
      constexpr int UB = 8;
      for (int k0 = g; k0 < p.nsplit; k0 += UB * G) {
        f32x4 v[UB];
        float wk[UB];
#pragma unroll
        for (int u = 0; u < UB; ++u) {
          const int k = k0 + u * G, kc = min(k, p.nsplit - 1);
          v[u] = *reinterpret_cast<const f32x4*>(po + (int64_t)kc * p.R);
          wk[u] = k < p.nsplit ? sw[i * MAX_SPLIT + kc] : 0.f;
        }
#pragma unroll
        for (int u = 0; u < UB; ++u) s += wk[u] * v[u];
      }
    }
    if (G > 1) {   // (workgroup-uniform; then one pass covers every item)
      acc4[threadIdx.x] = s;
      __syncthreads();
      if (live && g == 0)
        for (int k = 1; k < G; ++k) s += acc4[k * items + idx];
    }
    if (live && g == 0) {
      bf16x4 hi, lo;
#pragma unroll
      for (int e = 0; e < 4; ++e) { bf16 a, c; split_bf16(s[e], a, c); hi[e] = a; lo[e] = c; }
      *reinterpret_cast<bf16x4*>(xh + i * PITCH + col * 2) = hi;
      *reinterpret_cast<bf16x4*>(xl + i * PITCH + col * 2) = lo;
    }
  }
  __syncthreads();
  if (n0 >= p.dv) return;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f}, acl = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) {
    const int k = 32 * ks + 8 * kq;
    const bool ok = r16 < nb;
    const bf16x8 a = ok ? *reinterpret_cast<const bf16x8*>(xl + r16 * PITCH + k * 2) : zero8;
    const bf16x8 c = ok ? *reinterpret_cast<const bf16x8*>(xh + r16 * PITCH + k * 2) : zero8;
    acl = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[ks], a, acl, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[ks], c, acc, 0, 0, 0);
  }
  acc += acl;
  const int nn = n0 + 4 * kq;
  if (r16 < nb && nn < p.dv) {
    const int64_t b = b0 + r16;
    bf16x4 r;
    float g[4] = {1.f, 1.f, 1.f, 1.f};
    if (p.gate && p.gate_heads) {
      const float gh = vy_sigmoid((float)((const bf16*)p.gate)[b * p.ldg + head]);
#pragma unroll
      for (int e = 0; e < 4; ++e) g[e] = gh;
    } else if (p.gate) {
      const bf16x4 g4 = *reinterpret_cast<const bf16x4*>((const bf16*)p.gate + b * p.ldg + head * p.dv + nn);
#pragma unroll
      for (int e = 0; e < 4; ++e) g[e] = vy_sigmoid((float)g4[e]);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) r[e] = (bf16)(acc[e] * g[e]);
    *reinterpret_cast<bf16x4*>((bf16*)p.out + b * p.ldo + head * p.dv + nn) = r;
  }
}

// ---- generic path (fp32, or bf16 latents wider than 512): one wave per scalar product ------------
template <typename T>
__global__ __launch_bounds__(256) void latent_query_gen_kernel(LatentArgs p) {
  const int lane = threadIdx.x & 63;
  const int r = (int)blockIdx.x * 4 + (threadIdx.x >> 6), head = blockIdx.y, b = blockIdx.z;
  if (r >= p.R) return;
  const T* w = (const T*)p.wukt + ((int64_t)head * p.R + r) * p.dh;
  const T* x = (const T*)p.q + (int64_t)b * p.ldq + head * p.dh;
  float s = 0.f;
  for (int k = lane; k < p.dh; k += 64) s = fmaf(VyT<T>::ld(w + k), VyT<T>::ld(x + k), s);
  s = vy_wave_sum(s);
  if (lane == 0) p.qf[((int64_t)b * p.h + head) * p.R + r] = s;
}

template <typename T, int NR>
__global__ __launch_bounds__(256) void latent_scan_gen_kernel(LatentArgs p) {
  __shared__ float so[4][NR * 64];
  __shared__ float sm[4], sl[4];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int split = blockIdx.x, head = blockIdx.y, b = blockIdx.z;
  int slot;
  const int n = row_keys(p, b, slot);
  const int kps = (n + p.nsplit - 1) / p.nsplit;
  const int j1 = min(n, (split + 1) * kps);
  const T* C = (const T*)p.cache + (int64_t)slot * p.c_ss;
  const int64_t o_ = ((int64_t)b * p.h + head) * p.nsplit + split;
  float q[NR], acc[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int col = lane + 64 * i;
    q[i] = col < p.R ? p.qf[((int64_t)b * p.h + head) * p.R + col] : 0.f;
    acc[i] = 0.f;
  }
  float m = -FLT_MAX, l = 0.f;
  for (int j = split * kps + wave; j < j1; j += 4) {
    float c[NR], d = 0.f;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int col = lane + 64 * i;
      c[i] = col < p.R ? VyT<T>::ld(C + (int64_t)j * p.c_st + col) : 0.f;
      d = fmaf(q[i], c[i], d);
    }
    const float s = vy_wave_sum(d) * p.c;
    const float mn = fmaxf(m, s);
    const float a = exp2f(m - mn), e = exp2f(s - mn);
    m = mn;
    l = l * a + e;
#pragma unroll
    for (int i = 0; i < NR; ++i) acc[i] = acc[i] * a + e * c[i];
  }
#pragma unroll
  for (int i = 0; i < NR; ++i) so[wave][lane + 64 * i] = acc[i];
  if (lane == 0) { sm[wave] = m; sl[wave] = l; }
  __syncthreads();
  const float M = fmaxf(fmaxf(sm[0], sm[1]), fmaxf(sm[2], sm[3]));
  float w[4], L = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) { w[i] = exp2f(sm[i] - M); L += w[i] * sl[i]; }
  for (int col = threadIdx.x; col < p.R; col += 256)
    p.part_o[o_ * p.R + col] = w[0] * so[0][col] + w[1] * so[1][col] + w[2] * so[2][col] + w[3] * so[3][col];
  if (threadIdx.x == 0) { p.part_ml[o_ * 2] = M; p.part_ml[o_ * 2 + 1] = L; }
}

template <typename T>
__global__ __launch_bounds__(256) void latent_value_gen_kernel(LatentArgs p) {
  __shared__ float u[1024];
  __shared__ float sw[MAX_SPLIT];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int head = blockIdx.y, b = blockIdx.z;
  if (wave == 0) slice_weights(p, b, head, sw, lane);
  __syncthreads();
  const float* po = p.part_o + ((int64_t)b * p.h + head) * p.nsplit * p.R;
  for (int col = threadIdx.x; col < p.R; col += 256) {
    float s = 0.f;
    for (int k = 0; k < p.nsplit; ++k) s = fmaf(sw[k], po[(int64_t)k * p.R + col], s);
    u[col] = s;
  }
  __syncthreads();
  const int n1 = min(p.dv, ((int)blockIdx.x + 1) * 64);
  for (int n = (int)blockIdx.x * 64 + wave; n < n1; n += 4) {
    const T* w = (const T*)p.wuv + ((int64_t)head * p.dv + n) * p.R;
    float s = 0.f;
    for (int k = lane; k < p.R; k += 64) s = fmaf(VyT<T>::ld(w + k), u[k], s);
    s = vy_wave_sum(s);
    if (lane == 0) {
      if (p.gate) s *= vy_sigmoid(VyT<T>::ld((const T*)p.gate + (int64_t)b * p.ldg + (p.gate_heads ? head : head * p.dv + n)));
      VyT<T>::st((T*)p.out + (int64_t)b * p.ldo + head * p.dv + n, s);
    }
  }
}

int64_t up256(int64_t x) { return (x + 255) / 256 * 256; }
int64_t query_bytes(int B, int h, int R) { return up256((int64_t)B * h * R * 4); }

int scan_tile(int R) { return R > 256 ? 32 : 64; }
// slices of the key range: enough workgroups for the CUs' occupancy of the scan kernel, at least two tiles each
int pick_split(int B, int groups, int64_t max_keys, int R) {
  const int64_t tiles = vy_cdiv(max_keys, scan_tile(R));
  const int64_t want = vy_cdiv(R > 256 ? 256 : 512, (int64_t)B * groups);
  int64_t s = vy_cdiv(tiles, 2);
  if (s > want) s = want;
  if (s > MAX_SPLIT) s = MAX_SPLIT;
  return (int)(s < 1 ? 1 : s);
}

template <typename T>
int generic_go(LatentArgs& p, int64_t max_keys, hipStream_t st) {
  int64_t s = vy_cdiv(512, (int64_t)p.B * p.h);
  if (s > vy_cdiv(max_keys, 64)) s = vy_cdiv(max_keys, 64);
  p.nsplit = (int)(s > MAX_SPLIT ? MAX_SPLIT : s < 1 ? 1 : s);
  const dim3 block(256);
  hipLaunchKernelGGL(latent_query_gen_kernel<T>, dim3((unsigned)vy_cdiv(p.R, 4), p.h, p.B), block, 0, st, p);
  const dim3 grid(p.nsplit, p.h, p.B);
  if (p.R <= 128) hipLaunchKernelGGL((latent_scan_gen_kernel<T, 2>), grid, block, 0, st, p);
  else if (p.R <= 256) hipLaunchKernelGGL((latent_scan_gen_kernel<T, 4>), grid, block, 0, st, p);
  else if (p.R <= 512) hipLaunchKernelGGL((latent_scan_gen_kernel<T, 8>), grid, block, 0, st, p);
  else hipLaunchKernelGGL((latent_scan_gen_kernel<T, 16>), grid, block, 0, st, p);
  hipLaunchKernelGGL(latent_value_gen_kernel<T>, dim3((unsigned)vy_cdiv(p.dv, 64), p.h, p.B), block, 0, st, p);
  return 0;
}

}  // namespace

// latent queries and the partial sums of at most max(512 / (B groups), 1) <= MAX_SPLIT slices
extern "C" int64_t vy_latent_decode_ws_bytes(int32_t B, int32_t h, int32_t R) {
  int64_t s = vy_cdiv(512, (int64_t)B * ((h + 15) / 16));
  if (s > MAX_SPLIT) s = MAX_SPLIT;
  return query_bytes(B, h, R) + up256((int64_t)B * h * s * R * 4) + up256((int64_t)B * h * s * 8);
}

extern "C" int vy_latent_decode(const void* q, int64_t ldq, const void* wukt, const void* wuv, const void* cache, int64_t c_ss,
                                int64_t c_st, const int32_t* slots, const int32_t* start, int64_t max_keys, void* out,
                                int64_t ldo, const void* gate, int64_t ldg, int gate_heads, int32_t ring, int32_t B, int32_t h, int32_t dh, int32_t dv,
                                int32_t R, float scale, void* ws, int64_t ws_bytes, int dtype, void* stream) {
  const char* who = "vy_latent_decode";
  if (!q || !wukt || !wuv || !cache || !start || !out || !ws) VY_FAIL(VY_ERR_ARG, "%s: null pointer", who);
  if (B <= 0 || h <= 0 || dh <= 0 || dv <= 0 || R <= 0 || max_keys <= 0 || ring < 0) VY_FAIL(VY_ERR_ARG, "%s: empty problem", who);
  if (dh % 8 || dv % 8 || R % 8 || ldq % 8 || ldo % 8 || ldg % 8 || c_ss % 8 || c_st % 8)
    VY_FAIL(VY_ERR_ARG, "%s: widths and strides must be multiples of 8", who);
  if (R > 1024) VY_FAIL(VY_ERR_UNSUPPORTED, "%s: latent width %d > 1024", who, R);
  if (ws_bytes < vy_latent_decode_ws_bytes(B, h, R)) VY_FAIL(VY_ERR_ARG, "%s: workspace too small", who);
  hipStream_t st = (hipStream_t)stream;
  LatentArgs p{};
  p.q = q; p.ldq = ldq; p.wukt = wukt; p.wuv = wuv; p.cache = cache; p.c_ss = c_ss; p.c_st = c_st;
  p.slots = slots; p.start = start; p.out = out; p.ldo = ldo; p.gate = gate; p.ldg = ldg;
  p.B = B; p.h = h; p.dh = dh; p.dv = dv; p.R = R; p.c = scale * LOG2E; p.ring = ring; p.gate_heads = gate_heads;
  if (ring && max_keys > ring) max_keys = ring;
  char* w = (char*)ws;
  p.qf = (float*)w; p.qhi = (bf16*)w; p.qlo = p.qhi + (int64_t)B * h * R;
  int64_t s = vy_cdiv(512, (int64_t)B * ((h + 15) / 16));
  if (s > MAX_SPLIT) s = MAX_SPLIT;
  p.part_o = (float*)(w + query_bytes(B, h, R));
  p.part_ml = (float*)(w + query_bytes(B, h, R) + up256((int64_t)B * h * s * R * 4));
  if (dtype == VY_F32) generic_go<float>(p, max_keys, st);
  else if (dtype != VY_BF16) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  else if (R > 512) generic_go<bf16>(p, max_keys, st);
  else {
    const int groups = (h + 15) / 16, bt = (B + 15) / 16;
    p.nsplit = pick_split(B, groups, max_keys, R);
    const dim3 block(256);
    hipLaunchKernelGGL(latent_query_kernel, dim3((unsigned)vy_cdiv(R, 64), h, bt), block, 0, st, p);
    const dim3 grid(p.nsplit, groups, B);
    if (R <= 64) hipLaunchKernelGGL(latent_scan_kernel<64>, grid, block, 0, st, p);
    else if (R <= 128) hipLaunchKernelGGL(latent_scan_kernel<128>, grid, block, 0, st, p);
    else if (R <= 256) hipLaunchKernelGGL(latent_scan_kernel<256>, grid, block, 0, st, p);
    else hipLaunchKernelGGL(latent_scan_kernel<512>, grid, block, 0, st, p);
    const int nv = (int)vy_cdiv(dv, 64);
    const int64_t per = vy_cdiv((int64_t)B * h * nv, 256);         // sequences per workgroup: fill the CUs first
    p.seqs = (int)(per > 16 ? 16 : per);
    const dim3 vgrid(nv, h, (unsigned)vy_cdiv(B, p.seqs));
    auto lds = [&](int RP) { return p.seqs * MAX_SPLIT * 4 + 4096 + 2 * p.seqs * (RP + 8) * 2; };
    if (R <= 64) hipLaunchKernelGGL(latent_value_kernel<64>, vgrid, block, lds(64), st, p);
    else if (R <= 128) hipLaunchKernelGGL(latent_value_kernel<128>, vgrid, block, lds(128), st, p);
    else if (R <= 256) hipLaunchKernelGGL(latent_value_kernel<256>, vgrid, block, lds(256), st, p);
    else hipLaunchKernelGGL(latent_value_kernel<512>, vgrid, block, lds(512), st, p);
  }
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}
