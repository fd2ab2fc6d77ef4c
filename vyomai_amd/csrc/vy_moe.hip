// Mixture of experts: every token goes through `top` of E small feed-forward layers.
//
//   vy_moe_fwd   router logits (fp32), choice of experts, the experts, their outputs left as rows for
//                vy_residual_norm_routed (which adds them up, weighted, in fp32)
//   vy_clamped_act_fwd   the experts' activation on packed [gate | up] rows (a shared expert's)
//
// Expert e, gated and clamped: g = min(Wg h, limit), u = clamp(Wu h, -limit, limit), y = Wd (g sigmoid(alpha g) (u + 1)); or
// plain: y = Wd gelu(Wu h).  Wg and Wu are packed with their rows interleaved (row 2j: gate j, row 2j + 1: up j): in the accumulators' layout (a lane owns 4 consecutive
// output columns of one token) both halves of a pair sit in one lane and the activation is the product's epilogue.
//
// Few tokens (decode): expert_rows_kernel streams the weights of the experts in use straight into MFMA operands (vy_rows.h), one
// workgroup per 16 or 32 weight rows of an expert; which experts and tokens, every workgroup reads from the choice itself.
// Many tokens (prefill): tokens are sorted by expert (ranks from the choice kernel, offsets in the scatter kernel) and
// grouped_gemm_kernel runs 128 x 128 tiles over the experts' row ranges, gathering its rows of h on the way into LDS.
// fp32 takes the same way with a plain tile kernel.  A row's result does not depend on its place or on other rows.
#include "vy_moe.h"

namespace {

using namespace vy_moe_dev;

constexpr int COUNT_STRIDE = 32;   // the experts' counters, one per 128-byte line: adds to one line queue up

// ---- router -----------------------------------------------------------------------------------
// logits[m][e] = sum_k h[m][k] w[e][k], fp32 accumulation and result.  One workgroup: 16 ET experts x 16 MT tokens.
template <int ET, int MT, int NW>
__global__ __launch_bounds__(64 * NW) void router_logits_kernel(const bf16* __restrict__ h, int64_t ldh, const bf16* __restrict__ w,
                                                            float* __restrict__ logits, int64_t M, int K, int E) {
  __shared__ f32x4 red[vy_rows::RED<ET, MT, NW>];
  const int lane = threadIdx.x & 63, r16 = lane & 15, kq = lane >> 4;
  const int e0 = blockIdx.x * 16 * ET;
  const int64_t m0 = (int64_t)blockIdx.y * 16 * MT;
  const bf16* ws[ET];
  const bf16* hs[MT];
#pragma unroll
  for (int i = 0; i < ET; ++i) ws[i] = w + (int64_t)min(e0 + 16 * i + r16, E - 1) * K + 8 * kq;
#pragma unroll
  for (int j = 0; j < MT; ++j) hs[j] = h + (m0 + 16 * j + r16 < M ? m0 + 16 * j + r16 : M - 1) * ldh + 8 * kq;
  f32x4 acc[ET][MT];
  vy_rows::stream<ET, MT, false, NW>(ws, hs, K, acc, red);
  if (threadIdx.x >= 64) return;
#pragma unroll
  for (int i = 0; i < ET; ++i)
#pragma unroll
    for (int j = 0; j < MT; ++j) {
      const int64_t m = m0 + 16 * j + r16;
      const int e = e0 + 16 * i + 4 * kq;   // a lane: token r16, experts 4 kq .. + 3
      if (m < M)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (e + r < E) logits[m * E + e + r] = acc[i][j][r];
    }
}

__global__ __launch_bounds__(256) void router_logits_f32_kernel(const float* __restrict__ h, int64_t ldh, const float* __restrict__ w,
                                                                float* __restrict__ logits, int K, int E) {
  const int lane = threadIdx.x & 63, e = blockIdx.y * 4 + (threadIdx.x >> 6);
  const int64_t m = blockIdx.x;
  if (e >= E) return;
  float s = 0.f;
  for (int k = lane * 4; k < K; k += 256) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(h + m * ldh + k), b = *reinterpret_cast<const f32x4*>(w + (int64_t)e * K + k);
#pragma unroll
    for (int c = 0; c < 4; ++c) s = fmaf(a[c], b[c], s);
  }
  s = vy_wave_sum(s);
  if (lane == 0) logits[m * E + e] = s;
}

// ---- choice of experts ------------------------------------------------------------------------
// TPW tokens per wave; ranks: the workgroup's choices are counted in LDS, one global add per expert and workgroup
template <int EPL, int NW>
__global__ __launch_bounds__(64 * NW) void choose_kernel(ChooseArgs a, int tpw) {
  __shared__ float groups[NW][2 * 64 * EPL];
  __shared__ int hist[64 * EPL], base[64 * EPL];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int64_t m0 = ((int64_t)blockIdx.x * NW + wave) * tpw;
  if (a.counts) {
    for (int e = threadIdx.x; e < a.E; e += 64 * NW) hist[e] = 0;
    __syncthreads();
  }
  for (int t = 0; t < tpw; ++t) {
    const int64_t m = m0 + t;
    if (m >= a.M) break;
    int id;
    float w;
    choose_one<EPL>(a, m, a.logits + m * a.E, lane, groups[wave], id, w);
    if (lane < a.top) {
      a.ids[m * a.top + lane] = id;
      a.weight[m * a.top + lane] = w;
      if (a.pos) a.pos[m * a.top + lane] = id >= 0 ? (int)(m * a.top + lane) : -1;
      if (a.counts) a.rank[m * a.top + lane] = id >= 0 ? atomicAdd(&hist[id], 1) : 0;
    }
  }
  if (!a.counts) return;
  __syncthreads();
  for (int e = threadIdx.x; e < a.E; e += 64 * NW) base[e] = hist[e] ? atomicAdd(&a.counts[e * COUNT_STRIDE], hist[e]) : 0;
  __syncthreads();
  for (int t = 0; t < tpw; ++t) {
    const int64_t m = m0 + t;
    if (m >= a.M) break;
    if (lane < a.top) {   // (the lane that wrote them above)
      const int id = a.ids[m * a.top + lane];
      if (id >= 0) a.rank[m * a.top + lane] += base[id];
    }
  }
}

// ---- sorting by expert ------------------------------------------------------------------------
struct Tile { int expert, first, tiles, pad; };   // the expert of a tile, the expert's first tile and tile count
struct SortArgs {
  const int* ids; const int* rank; const int* counts;   // counts COUNT_STRIDE apart
  int64_t n; int top, E, bm;
  int* pos; int* token;                // choice -> sorted row, sorted row -> token
  int* offset; int* rows;              // [E] first sorted row and row count of an expert
  Tile* tiles; int* ntiles;
};

__global__ __launch_bounds__(256) void sort_kernel(SortArgs a) {
  __shared__ int off[MAX_E];
  __shared__ int wrow[4], wtile[4];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  // exclusive sums over the experts of rows and tiles; 4 experts per thread
  int c[4], rows = 0, tiles = 0;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int e = tid * 4 + i;
    c[i] = e < a.E ? a.counts[e * COUNT_STRIDE] : 0;
    rows += c[i];
    tiles += (c[i] + a.bm - 1) / a.bm;
  }
  int sr = rows, st = tiles;
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const int r = __shfl_up(sr, o, 64), t = __shfl_up(st, o, 64);
    if (lane >= o) { sr += r; st += t; }
  }
  if (lane == 63) { wrow[wave] = sr; wtile[wave] = st; }
  __syncthreads();
  int r0 = sr - rows, t0 = st - tiles;
  for (int w = 0; w < wave; ++w) { r0 += wrow[w]; t0 += wtile[w]; }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int e = tid * 4 + i, nt = (c[i] + a.bm - 1) / a.bm;
    if (e < a.E) {
      off[e] = r0;
      if (blockIdx.x == 0) {
        a.offset[e] = r0;
        a.rows[e] = c[i];
        for (int t = 0; t < nt; ++t) a.tiles[t0 + t] = Tile{e, t0, nt, 0};
      }
    }
    r0 += c[i];
    t0 += nt;
  }
  if (blockIdx.x == 0 && tid == 255) *a.ntiles = t0;
  __syncthreads();
  const int64_t i = (int64_t)blockIdx.x * 256 + tid;
  if (i < a.n) {
    const int id = a.ids[i];
    const int p = id >= 0 ? off[id] + a.rank[i] : -1;
    a.pos[i] = p;
    if (p >= 0) a.token[p] = (int)(i / a.top);
  }
}

// ---- the experts, many tokens -----------------------------------------------------------------
__device__ __forceinline__ int xcd_remap(int bid, int nwg) {
  const int xcd = bid & 7, q = nwg >> 3, r = nwg & 7;
  return (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + (bid >> 3);
}

struct GroupedArgs {
  const void* x; int64_t ldx;          // rows of h (gathered by `token`) or sorted activation rows (token NULL)
  const int* token; const int* offset; const int* count;
  const Tile* tiles; const int* ntiles;
  const void* w; int N, K;             // [E][N][K]
  void* y; int64_t ldy;                // sorted rows
  float limit, alpha;
};

// tile of this workgroup: expert by expert, an expert's row tiles innermost (they share the weight tile in L2)
__device__ __forceinline__ bool grouped_tile(const GroupedArgs& a, int tiles_n, int& e, int& mt, int& nt) {
  const int total = *a.ntiles * tiles_n;
  if ((int)blockIdx.x >= total) return false;
  const int id = xcd_remap(blockIdx.x, total);
  const Tile t = a.tiles[id / tiles_n];
  const int local = id - t.first * tiles_n;
  e = t.expert;
  nt = local / t.tiles;
  mt = local - nt * t.tiles;
  return true;
}

constexpr int BK = 64, ROWB = BK * 2;

// 128 x 128 x 64 tiles, two LDS stages, four waves of 64 x 64 on mfma_f32_16x16x32_bf16 (the structure of
// gemm_nt_bf16_m16_kernel).  GU: rows gathered, activation in the epilogue, half as many output columns.
template <int KIND>
__global__ __launch_bounds__(256) void grouped_gemm_kernel(GroupedArgs a) {
  constexpr int BM = 128, BN = 128, NW = 4, TM = 4, TN = 4, GX = BM / 8 / NW, GW = BN / 8 / NW;
  constexpr int STAGE = (BM + BN) * ROWB, ON = KIND == GATE_UP ? BN / 2 : BN, OROW = ON * 2 + 16;
  static_assert(BM * OROW <= 2 * STAGE, "the output tile fits");
  __shared__ __attribute__((aligned(16))) char smem[2 * STAGE];
  int e, mt, nt;
  if (!grouped_tile(a, (a.N + BN - 1) / BN, e, mt, nt)) return;
  const int rows = a.count[e] - mt * BM, row0 = a.offset[e] + mt * BM, n0 = nt * BN;
  const int N = a.N, K = a.K;
  const bf16* W = (const bf16*)a.w + (int64_t)e * N * K;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), wm = wave >> 1, wn = wave & 1;
  const int lrow = lane >> 3, slot = lane & 7;
  const bf16* xsrc[GX]; int xk[GX];
  const bf16* wsrc[GW]; int wk[GW];
#pragma unroll
  for (int t = 0; t < GX; ++t) {
    const int R = (wave + NW * t) * 8 + lrow, g = slot ^ ((R >> 1) & 7);
    const int r = row0 + (R < rows ? R : rows - 1);
    xsrc[t] = (const bf16*)a.x + (int64_t)(KIND != DOWN ? a.token[r] : r) * a.ldx + g * 8;
    xk[t] = g * 8;
  }
#pragma unroll
  for (int t = 0; t < GW; ++t) {
    const int R = (wave + NW * t) * 8 + lrow, g = slot ^ ((R >> 1) & 7);
    wsrc[t] = W + (int64_t)min(n0 + R, N - 1) * K + g * 8;
    wk[t] = g * 8;
  }
  const bf16* zero = reinterpret_cast<const bf16*>(vy_zero16);
  const bool ktail = (K % BK) != 0;
  const int KT = (K + BK - 1) / BK;
  auto stage = [&](int kt, int buf) {
    char* xb = smem + buf * STAGE;
    char* wb = xb + BM * ROWB;
    const int k0 = kt * BK;
#pragma unroll
    for (int t = 0; t < GX; ++t) {
      const bf16* s = xsrc[t] + k0;
      if (ktail && k0 + xk[t] >= K) s = zero;
      __builtin_amdgcn_global_load_lds((const VY_GLOBAL void*)s, (VY_LDS void*)(xb + (wave + NW * t) * 1024), 16, 0, 0);
    }
#pragma unroll
    for (int t = 0; t < GW; ++t) {
      const bf16* s = wsrc[t] + k0;
      if (ktail && k0 + wk[t] >= K) s = zero;
      __builtin_amdgcn_global_load_lds((const VY_GLOBAL void*)s, (VY_LDS void*)(wb + (wave + NW * t) * 1024), 16, 0, 0);
    }
  };
  f32x4 acc[TN][TM];
#pragma unroll
  for (int i = 0; i < TN; ++i)
#pragma unroll
    for (int j = 0; j < TM; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int r16 = lane & 15, kq = lane >> 4, fsw = (r16 >> 1) & 7;
  unsigned xa[2], wa[2];
#pragma unroll
  for (int ks = 0; ks < 2; ++ks) {
    const int coff = (((ks * 4 + kq) ^ fsw) << 4);
    xa[ks] = vy_lds_addr(smem) + (wm * 16 * TM + r16) * ROWB + coff;
    wa[ks] = vy_lds_addr(smem) + BM * ROWB + (wn * 16 * TN + r16) * ROWB + coff;
  }
  bf16x8 wf[2][TN], xf[2][TM];
  auto read_frags = [&](unsigned wbase, unsigned xbase, bf16x8 (&w_)[TN], bf16x8 (&x_)[TM]) {
    vy_static_for<TN>([&](auto i_c) { constexpr int i = decltype(i_c)::value; w_[i] = vy_lds_read128_off<i * 16 * ROWB>(wbase); });
    vy_static_for<TM>([&](auto j_c) { constexpr int j = decltype(j_c)::value; x_[j] = vy_lds_read128_off<j * 16 * ROWB>(xbase); });
  };
  auto tie_frags = [&](bf16x8 (&w_)[TN], bf16x8 (&x_)[TM]) {
#pragma unroll
    for (int i = 0; i < TN; ++i) vy_tie(w_[i]);
#pragma unroll
    for (int j = 0; j < TM; ++j) vy_tie(x_[j]);
  };
  auto mma = [&](bf16x8 (&w_)[TN], bf16x8 (&x_)[TM]) {
    __builtin_amdgcn_s_setprio(1);
#pragma unroll
    for (int i = 0; i < TN; ++i)
#pragma unroll
      for (int j = 0; j < TM; ++j)
        acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w_[i], x_[j], acc[i][j], 0, 0, 0);
    __builtin_amdgcn_s_setprio(0);
  };
  stage(0, 0);
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
  read_frags(wa[0], xa[0], wf[0], xf[0]);
  for (int kt = 0; kt < KT; ++kt) {
    const int cur = kt & 1;
    if (kt + 1 < KT) stage(kt + 1, cur ^ 1);
    const unsigned boff = cur * STAGE;
    read_frags(wa[1] + boff, xa[1] + boff, wf[1], xf[1]);
    asm volatile("s_waitcnt lgkmcnt(%0)" ::"n"(TN + TM) : "memory");
    tie_frags(wf[0], xf[0]);
    mma(wf[0], xf[0]);
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    tie_frags(wf[1], xf[1]);
    mma(wf[1], xf[1]);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    if (kt + 1 < KT) read_frags(wa[0] + (STAGE - boff), xa[0] + (STAGE - boff), wf[0], xf[0]);
  }
  // every wave is behind the loop's last barrier: the stages are free.  Lane: token r16 of block j, columns 4 kq .. of block i
#pragma unroll
  for (int i = 0; i < TN; ++i)
#pragma unroll
    for (int j = 0; j < TM; ++j) {
      char* at = smem + (wm * 16 * TM + 16 * j + r16) * OROW;
      const int n = wn * 16 * TN + 16 * i + 4 * kq;
      const f32x4 v = acc[i][j];
      if constexpr (KIND == GATE_UP) {
        bf16x2 w2;
        w2[0] = (bf16)clamped_act(v[0], v[1], a.limit, a.alpha);
        w2[1] = (bf16)clamped_act(v[2], v[3], a.limit, a.alpha);
        *reinterpret_cast<bf16x2*>(at + n) = w2;
      } else {
        bf16x4 w4;
#pragma unroll
        for (int r = 0; r < 4; ++r) w4[r] = (bf16)(KIND == UP ? vy_gelu_erf_fast(v[r]) : v[r]);
        *reinterpret_cast<bf16x4*>(at + 2 * n) = w4;
      }
    }
  __syncthreads();
  constexpr int CPR = ON / 8;
  const int NO = KIND == GATE_UP ? N / 2 : N, c0 = KIND == GATE_UP ? n0 / 2 : n0;
  for (int i = tid; i < BM * CPR; i += 256) {
    const int r = i / CPR, ch = (i % CPR) * 8;
    if (r < rows && c0 + ch < NO)
      *reinterpret_cast<bf16x8*>((bf16*)a.y + (int64_t)(row0 + r) * a.ldy + c0 + ch) = *reinterpret_cast<const bf16x8*>(smem + r * OROW + ch * 2);
  }
}

// fp32: 64 x 64 x 16 tiles, 4 x 4 outputs per thread, fused multiply-adds in order of k
template <int KIND>
__global__ __launch_bounds__(256) void grouped_gemm_f32_kernel(GroupedArgs a) {
  constexpr int T = 64, KB = 16;
  __shared__ float xs[KB][T + 4], ws[KB][T + 4];
  int e, mt, nt;
  if (!grouped_tile(a, (a.N + T - 1) / T, e, mt, nt)) return;
  const int rows = a.count[e] - mt * T, row0 = a.offset[e] + mt * T, n0 = nt * T;
  const float* W = (const float*)a.w + (int64_t)e * a.N * a.K;
  const int tid = threadIdx.x, lr = tid >> 2, lk = (tid & 3) * 4, ty = tid >> 4, tx = tid & 15;
  const int r = row0 + (lr < rows ? lr : rows - 1);
  const float* xr = (const float*)a.x + (int64_t)(KIND != DOWN ? a.token[r] : r) * a.ldx;
  const float* wr = W + (int64_t)min(n0 + lr, a.N - 1) * a.K;
  float acc[4][4] = {};
  for (int k0 = 0; k0 < a.K; k0 += KB) {
    f32x4 xv = {0.f, 0.f, 0.f, 0.f}, wv = xv;
    if (k0 + lk < a.K) {
      xv = *reinterpret_cast<const f32x4*>(xr + k0 + lk);
      wv = *reinterpret_cast<const f32x4*>(wr + k0 + lk);
    }
    __syncthreads();
#pragma unroll
    for (int c = 0; c < 4; ++c) { xs[lk + c][lr] = xv[c]; ws[lk + c][lr] = wv[c]; }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < KB; ++k)
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(xs[k][ty * 4 + i], ws[k][tx * 4 + j], acc[i][j]);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int m = ty * 4 + i, n = n0 + tx * 4;
    if (m >= rows || n >= a.N) continue;
    if constexpr (KIND == GATE_UP) {
      float* y = (float*)a.y + (int64_t)(row0 + m) * a.ldy + n / 2;
      y[0] = clamped_act(acc[i][0], acc[i][1], a.limit, a.alpha);
      y[1] = clamped_act(acc[i][2], acc[i][3], a.limit, a.alpha);
    } else {
      f32x4 v;
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = KIND == UP ? vy_gelu_erf(acc[i][j]) : acc[i][j];
      *reinterpret_cast<f32x4*>((float*)a.y + (int64_t)(row0 + m) * a.ldy + n) = v;
    }
  }
}

// ---- the experts, few tokens ------------------------------------------------------------------
template <int KIND, int NT>
__global__ __launch_bounds__(256) void expert_rows_kernel(ExpertRows a) {
  __shared__ ExpertLds<NT> lds;
  expert_rows<KIND, NT>(a, lds, blockIdx.x, blockIdx.y);
}
template <int KIND>
__global__ __launch_bounds__(256) void expert_rows1_kernel(ExpertRows a) {   // a single token
  expert_rows1<KIND>(a, blockIdx.x, blockIdx.y);
}

// ---- activation of packed [gate | up] rows ----------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void clamped_act_kernel(const T* __restrict__ gu, int64_t ldg, T* __restrict__ out, int64_t ldo,
                                                          int64_t M, int I, float limit, float alpha) {
  constexpr int VEC = VyChunk<T>::VEC;
  const int nch = I / VEC;
  const int64_t total = M * nch;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
    const int64_t m = i / nch;
    const int c = (int)(i - m * nch) * VEC;
    float g[VEC], u[VEC];
    VyChunk<T>::load(gu + m * ldg + c, g);
    VyChunk<T>::load(gu + m * ldg + I + c, u);
#pragma unroll
    for (int e = 0; e < VEC; ++e) g[e] = clamped_act(g[e], u[e], limit, alpha);
    VyChunk<T>::store(out + m * ldo + c, g);
  }
}

// ---- launchers --------------------------------------------------------------------------------
int64_t up(int64_t x) { return (x + 255) / 256 * 256; }

bool few(const vy_moe* d, int64_t M, int dtype) {
  const int64_t n = M * d->top;
  return dtype == VY_BF16 && n <= MAX_ENTRIES && (M <= 64 || n <= 24 * (int64_t)d->experts);
}
int tile_rows(int dtype) { return dtype == VY_BF16 ? 128 : 64; }
int64_t max_tiles(const vy_moe* d, int64_t M, int dtype) {   // every expert in use may end with a partial tile
  const int64_t n = M * d->top, e = n < d->experts ? n : d->experts;
  return n / tile_rows(dtype) + e;
}

struct Parts { float* logits; char* act; int* counts; int* rank; int* token; int* offset; int* rows; int* ntiles; Tile* tiles; };

int64_t lay_out(const vy_moe* d, int64_t M, int dtype, char* ws, Parts& p) {
  const int64_t n = M * d->top, e = dtype == VY_BF16 ? 2 : 4;
  char* at = ws;
  auto take = [&](int64_t bytes) { char* r = at; at += up(bytes); return r; };
  p.logits = (float*)take(M * d->experts * 4);
  p.act = take(n * d->ff * e);
  p.counts = (int*)take((int64_t)d->experts * COUNT_STRIDE * 4);
  p.rank = (int*)take(n * 4);
  p.token = (int*)take(n * 4);
  p.offset = (int*)take(d->experts * 4);
  p.rows = (int*)take(d->experts * 4);
  p.ntiles = (int*)take(4);
  p.tiles = (Tile*)take(max_tiles(d, M, dtype) * (int64_t)sizeof(Tile));
  return at - ws;
}

int check_moe(const char* who, const vy_moe* d, int dtype) {
  if (!d || !d->w_router || !d->w_gu || !d->w_down) VY_FAIL(VY_ERR_ARG, "%s: null weights", who);
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  if (d->experts < 1 || d->experts > MAX_E || d->top < 1 || d->top > 64 || d->groups < 1 || d->experts % d->groups ||
      d->keep < 1 || d->keep > d->groups || d->top > d->keep * (d->experts / d->groups))
    VY_FAIL(VY_ERR_UNSUPPORTED, "%s: %d of %d experts, %d of %d groups", who, d->top, d->experts, d->keep, d->groups);
  if ((d->act != VY_MOE_CLAMPED && d->act != VY_MOE_GELU) || (d->score != VY_SCORE_SOFTMAX && d->score != VY_SCORE_SIGMOID) ||
      d->group_best < 1 || d->group_best > 2)
    VY_FAIL(VY_ERR_ARG, "%s: activation %d, score %d, groups by %d scores", who, d->act, d->score, d->group_best);
  if (d->width < 8 || d->ff < 8 || d->width % 8 || d->ff % 8) VY_FAIL(VY_ERR_ARG, "%s: widths %d / %d must be multiples of 8", who, d->width, d->ff);
  return VY_OK;
}

// the experts of few tokens whose choice is made; rows by choice
void few_experts(const vy_moe* d, const void* h, int64_t ldh, int64_t M, const int* ids, void* act, void* rows, int64_t ldr, hipStream_t st) {
  const bool gated = d->act == VY_MOE_CLAMPED;
  const int K = d->width, n = (int)(M * d->top);
  const unsigned active = (unsigned)(n < d->experts ? n : d->experts);
  ExpertRows g{(const bf16*)h, ldh, ids, n, d->top, (const bf16*)d->w_gu, gated ? 2 * d->ff : d->ff, K, (bf16*)act, d->ff, d->limit, d->alpha};
  ExpertRows o{(const bf16*)act, d->ff, ids, n, d->top, (const bf16*)d->w_down, K, d->ff, (bf16*)rows, ldr, 0.f, 0.f};
  auto go = [&](auto kind, ExpertRows& a) {
    constexpr int KIND = decltype(kind)::value;
    const dim3 block(256);
    if (M == 1) hipLaunchKernelGGL((expert_rows1_kernel<KIND>), dim3((unsigned)vy_cdiv(a.N, 8), active), block, 0, st, a);
    else if (vy_cdiv(a.N, 16) * active > 1536) hipLaunchKernelGGL((expert_rows_kernel<KIND, 2>), dim3((unsigned)vy_cdiv(a.N, 32), active), block, 0, st, a);
    else hipLaunchKernelGGL((expert_rows_kernel<KIND, 1>), dim3((unsigned)vy_cdiv(a.N, 16), active), block, 0, st, a);
  };
  if (gated) go(std::integral_constant<int, GATE_UP>{}, g);
  else go(std::integral_constant<int, UP>{}, g);
  go(std::integral_constant<int, DOWN>{}, o);
}

__global__ void zero_kernel(int* p, int n) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < n) p[i] = 0;
}

}  // namespace

extern "C" int64_t vy_moe_ws_bytes(const vy_moe* d, int64_t M, int dtype) {
  if (!d || M < 1 || d->experts < 1 || d->top < 1) return -1;
  Parts p;
  return lay_out(d, M, dtype, nullptr, p);
}

extern "C" int vy_moe_fwd(const vy_moe* d, const void* h, int64_t ldh, int64_t M, const int32_t* count, int64_t L, void* rows,
                          int64_t ldr, int32_t* ids, int32_t* pos, float* weight, void* ws, int64_t ws_bytes, int dtype,
                          void* stream) {
  const char* who = "vy_moe_fwd";
  if (int rc = check_moe(who, d, dtype)) return rc;
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!h || !rows || !ids || !pos || !weight || !ws || M < 1 || L < 1 || M * d->top > INT32_MAX / 2) VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (ldh % vec || ldr % vec || ldh < d->width || ldr < d->width || (uintptr_t)ws % 16) VY_FAIL(VY_ERR_ARG, "%s: bad row strides or alignment", who);
  Parts p;
  if (ws_bytes < lay_out(d, M, dtype, (char*)ws, p)) VY_FAIL(VY_ERR_ARG, "%s: workspace too small", who);
  hipStream_t st = (hipStream_t)stream;
  const int E = d->experts, K = d->width;
  const int64_t n = M * d->top;
  const bool small = few(d, M, dtype), gated = d->act == VY_MOE_CLAMPED;
  const int up_rows = gated ? 2 * d->ff : d->ff;
  if (!small) hipLaunchKernelGGL(zero_kernel, dim3((unsigned)vy_cdiv((int64_t)E * COUNT_STRIDE, 256)), dim3(256), 0, st, p.counts, E * COUNT_STRIDE);
  if (dtype == VY_F32) {
    hipLaunchKernelGGL(router_logits_f32_kernel, dim3((unsigned)M, (unsigned)vy_cdiv(E, 4)), dim3(256), 0, st, (const float*)h, ldh,
                       (const float*)d->w_router, p.logits, K, E);
  } else if (M <= 256) {
    hipLaunchKernelGGL((router_logits_kernel<1, 1, 4>), dim3((unsigned)vy_cdiv(E, 16), (unsigned)vy_cdiv(M, 16)), dim3(256), 0, st,
                       (const bf16*)h, ldh, (const bf16*)d->w_router, p.logits, M, K, E);
  } else {
    hipLaunchKernelGGL((router_logits_kernel<4, 2, 8>), dim3((unsigned)vy_cdiv(E, 64), (unsigned)vy_cdiv(M, 32)), dim3(512), 0, st,
                       (const bf16*)h, ldh, (const bf16*)d->w_router, p.logits, M, K, E);
  }
  ChooseArgs c{p.logits, M, E, d->top, d->groups, d->keep, d->score == VY_SCORE_SIGMOID, d->group_best, d->normalize, d->scale, count, (int)L, ids, weight, small ? pos : nullptr, small ? nullptr : p.counts, p.rank};
  // few tokens: a wave each, spread over the CUs; many: several per workgroup, so that few global adds count them
  const dim3 block(256);
#define CHOOSE(EPL, NW, TPW) hipLaunchKernelGGL((choose_kernel<EPL, NW>), dim3((unsigned)vy_cdiv(M, NW * TPW)), dim3(64 * NW), 0, st, c, TPW)
  if (small || E > 256) {
    if (E <= 64) CHOOSE(1, 4, 1);
    else if (E <= 128) CHOOSE(2, 4, 1);
    else if (E <= 256) CHOOSE(4, 4, 1);
    else CHOOSE(16, 4, 2);
  } else if (E <= 64) CHOOSE(1, 16, 2);
  else if (E <= 128) CHOOSE(2, 16, 2);
  else CHOOSE(4, 16, 2);
#undef CHOOSE
  if (small) {
    few_experts(d, h, ldh, M, ids, p.act, rows, ldr, st);
    VY_CHECK_LAUNCH(who);
    return VY_OK;
  }
  const int bm = tile_rows(dtype);
  SortArgs s{ids, p.rank, p.counts, n, d->top, E, bm, pos, p.token, p.offset, p.rows, p.tiles, p.ntiles};
  hipLaunchKernelGGL(sort_kernel, dim3((unsigned)vy_cdiv(n, 256)), block, 0, st, s);
  GroupedArgs g{h, ldh, p.token, p.offset, p.rows, p.tiles, p.ntiles, d->w_gu, up_rows, K, p.act, d->ff, d->limit, d->alpha};
  GroupedArgs o{p.act, d->ff, nullptr, p.offset, p.rows, p.tiles, p.ntiles, d->w_down, K, d->ff, rows, ldr, 0.f, 0.f};
  const int64_t tiles = max_tiles(d, M, dtype);
  const dim3 ggrid((unsigned)(tiles * vy_cdiv(g.N, bm))), ogrid((unsigned)(tiles * vy_cdiv(o.N, bm)));
  if (dtype == VY_BF16) {
    if (gated) hipLaunchKernelGGL((grouped_gemm_kernel<GATE_UP>), ggrid, block, 0, st, g);
    else hipLaunchKernelGGL((grouped_gemm_kernel<UP>), ggrid, block, 0, st, g);
    hipLaunchKernelGGL((grouped_gemm_kernel<DOWN>), ogrid, block, 0, st, o);
  } else {
    if (gated) hipLaunchKernelGGL((grouped_gemm_f32_kernel<GATE_UP>), ggrid, block, 0, st, g);
    else hipLaunchKernelGGL((grouped_gemm_f32_kernel<UP>), ggrid, block, 0, st, g);
    hipLaunchKernelGGL((grouped_gemm_f32_kernel<DOWN>), ogrid, block, 0, st, o);
  }
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}

// internal (vy_hybrid.hip): the experts alone, behind a choice made elsewhere (no padding tokens); rows by choice.
// VY_ERR_UNSUPPORTED: too many tokens for that
int vy_moe_few(const vy_moe* d, const void* h, int64_t ldh, int64_t M, const int32_t* ids, void* rows, int64_t ldr, void* ws,
               int64_t ws_bytes, int dtype, void* stream) {
  const char* who = "vy_moe_fwd";
  if (int rc = check_moe(who, d, dtype)) return rc;
  if (!few(d, M, dtype)) return VY_ERR_UNSUPPORTED;
  if (!h) return VY_OK;   // (asked whether it would)
  Parts p;
  if (!ids || !rows || !ws || ws_bytes < lay_out(d, M, dtype, (char*)ws, p)) VY_FAIL(VY_ERR_ARG, "%s: workspace too small", who);
  few_experts(d, h, ldh, M, ids, p.act, rows, ldr, (hipStream_t)stream);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}

extern "C" int vy_clamped_act_fwd(const void* gate_up, int64_t ldg, void* out, int64_t ldo, int64_t M, int64_t I, float limit,
                                  float alpha, int dtype, void* stream) {
  const char* who = "vy_clamped_act_fwd";
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!gate_up || !out || M <= 0 || I <= 0 || I % vec || ldg % vec || ldo % vec) VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  const int64_t want = vy_cdiv(M * (I / vec), 256);
  const dim3 grid((unsigned)(want < 8192 ? want : 8192)), block(256);
  hipStream_t st = (hipStream_t)stream;
  if (dtype == VY_BF16) hipLaunchKernelGGL((clamped_act_kernel<bf16>), grid, block, 0, st, (const bf16*)gate_up, ldg, (bf16*)out, ldo, M, (int)I, limit, alpha);
  else hipLaunchKernelGGL((clamped_act_kernel<float>), grid, block, 0, st, (const float*)gate_up, ldg, (float*)out, ldo, M, (int)I, limit, alpha);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}
