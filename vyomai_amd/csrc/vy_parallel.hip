// Decode step of a parallel layer (windowed attention beside a feed-forward, both reading one norm), bf16, up to 64 sequences: the
// layer's independent pieces share launches, so that what depends on each other is all that waits.
//
//   parallel_in       in = w_in h (q | k | v | gate | shared gate | shared up)          router logits
//   parallel_mix      window attention over the ring                                    choice of experts, shared activation
//   parallel_experts  attention's slices put together (few sequences only)              experts: gate and up, activation
//   parallel_out      y = w_o [heads | shared activation]                               experts: down
//
// (the residual sum, the experts' weighted sum and the next norm are vy_residual_norm's).  The blocks of a launch are cut into
// ranges, one per piece; every piece is device code that also runs alone (vy_rows.h, vy_window.h, vy_moe.h).
#include "vy_moe.h"
#include "vy_window.h"

namespace {

using namespace vy_moe_dev;
using namespace vy_window;
using vy_rows::Dense;

// MB: blocks of 16 sequences; 0: one sequence (8 weight rows per workgroup instead of 16)
template <int MB>
__global__ __launch_bounds__(256) void parallel_in_kernel(Dense in, Dense router, int n_in) {
  const bool first = (int)blockIdx.x < n_in;
  const int tile = first ? blockIdx.x : blockIdx.x - n_in;
  if constexpr (MB == 0) {
    vy_rows::dense1(first ? in : router, tile);
  } else {
    __shared__ f32x4 red[vy_rows::RED<1, MB>];
    vy_rows::dense<MB>(first ? in : router, red, tile);
  }
}

struct MixArgs {
  DecodeArgs win; int n_win;           // blocks of the attention: slices innermost, then heads, then sequences
  ChooseArgs choose; int n_choose;     // blocks of four tokens
  const bf16* gu; int64_t ldg; bf16* act; int64_t lda; int B, ff;   // shared feed-forward: packed [gate | up] rows
  float limit, alpha;
};

template <int DHP, int DVP>
__global__ __launch_bounds__(256) void parallel_mix_kernel(MixArgs a) {
  constexpr int LDS = WindowDecode<DHP, DVP>::LDS;
  static_assert(LDS >= 4 * 2 * 256 * 4, "the choice's LDS fits");
  __shared__ __attribute__((aligned(16))) char smem[LDS];
  int id = blockIdx.x;
  if (id < a.n_win) {
    const int rows = a.win.hk * a.win.passes, slice = id % a.win.ns, r = id / a.win.ns;
    WindowDecode<DHP, DVP>::run(a.win, smem, slice, r % rows, r / rows);
    return;
  }
  id -= a.n_win;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  if (id < a.n_choose) {
    const int64_t m = (int64_t)id * 4 + wave;
    if (m >= a.choose.M) return;
    int e;
    float w;
    float* lds = reinterpret_cast<float*>(smem) + wave * 512;
    const float* z = a.choose.logits + m * a.choose.E;
    if (a.choose.E <= 64) choose_one<1>(a.choose, m, z, lane, lds, e, w);
    else if (a.choose.E <= 128) choose_one<2>(a.choose, m, z, lane, lds, e, w);
    else choose_one<4>(a.choose, m, z, lane, lds, e, w);
    if (lane < a.choose.top) {
      a.choose.ids[m * a.choose.top + lane] = e;
      a.choose.weight[m * a.choose.top + lane] = w;
    }
    return;
  }
  id -= a.n_choose;
  const int nch = a.ff / 8, i = id * 256 + (int)threadIdx.x, b = i / nch, c = (i - b * nch) * 8;
  if (b >= a.B) return;
  float g[8], u[8];
  VyChunk<bf16>::load(a.gu + (int64_t)b * a.ldg + c, g);
  VyChunk<bf16>::load(a.gu + (int64_t)b * a.ldg + a.ff + c, u);
#pragma unroll
  for (int e = 0; e < 8; ++e) g[e] = clamped_act(g[e], u[e], a.limit, a.alpha);
  VyChunk<bf16>::store(a.act + (int64_t)b * a.lda + c, g);
}

template <int NT>
__global__ __launch_bounds__(256) void parallel_experts_kernel(DecodeArgs win, int n_finish, ExpertRows ex, int tiles) {
  const int id = blockIdx.x;
  if constexpr (NT == 0) {   // one sequence
    __shared__ __attribute__((aligned(16))) float red[FINISH_LDS / 4];
    if (id < n_finish) window_finish(win, red, id % win.h, id / win.h);
    else expert_rows1<GATE_UP>(ex, (id - n_finish) % tiles, (id - n_finish) / tiles);
  } else {
    __shared__ union { ExpertLds<NT> ex; float red[FINISH_LDS / 4]; } lds;
    if (id < n_finish) window_finish(win, lds.red, id % win.h, id / win.h);
    else expert_rows<GATE_UP, NT>(ex, lds.ex, (id - n_finish) % tiles, (id - n_finish) / tiles);
  }
}

template <int MB, int NT>
__global__ __launch_bounds__(256) void parallel_out_kernel(Dense out, int n_out, ExpertRows ex, int tiles) {
  const int id = blockIdx.x;
  if constexpr (MB == 0) {   // one sequence
    if (id < n_out) vy_rows::dense1(out, id);
    else expert_rows1<DOWN>(ex, (id - n_out) % tiles, (id - n_out) / tiles);
  } else {
    __shared__ union { ExpertLds<NT> ex; f32x4 red[vy_rows::RED<1, MB>]; } lds;
    if (id < n_out) vy_rows::dense<MB>(out, lds.red, id);
    else expert_rows<DOWN, NT>(ex, lds.ex, (id - n_out) % tiles, (id - n_out) / tiles);
  }
}

template <int DHP>
void mix_go(const MixArgs& a, int blocks, hipStream_t st) {
  const dim3 grid((unsigned)blocks), block(256);
  if (a.win.vdim <= 64) hipLaunchKernelGGL((parallel_mix_kernel<DHP, 64>), grid, block, 0, st, a);
  else if (a.win.vdim <= 128) hipLaunchKernelGGL((parallel_mix_kernel<DHP, 128>), grid, block, 0, st, a);
  else hipLaunchKernelGGL((parallel_mix_kernel<DHP, 256>), grid, block, 0, st, a);
}

template <int NT>
void out_go(int B, const Dense& d, int n_out, const ExpertRows& ex, int tiles, int blocks, hipStream_t st) {
  const dim3 grid((unsigned)blocks), block(256);
  if (B <= 16) hipLaunchKernelGGL((parallel_out_kernel<1, NT>), grid, block, 0, st, d, n_out, ex, tiles);
  else if (B <= 32) hipLaunchKernelGGL((parallel_out_kernel<2, NT>), grid, block, 0, st, d, n_out, ex, tiles);
  else hipLaunchKernelGGL((parallel_out_kernel<4, NT>), grid, block, 0, st, d, n_out, ex, tiles);
}

}  // namespace

// internal (vy_hybrid.hip): y and the experts' rows (by choice: row b * top + k, weights ew) of one VY_FORM_PARALLEL layer with
// VY_MIX_WINDOW.  VY_ERR_UNSUPPORTED: the driver's separate launches take the layer.
int vy_parallel_decode(const vy_hybrid_plan* p, const vy_hybrid_layer* L, const void* h, void* in, void* ao, void* y, void* erows,
                       int32_t* eids, float* ew, void* moe_ws, int64_t moe_ws_bytes, const int32_t* slots, const int32_t* lengths,
                       int64_t max_keys, void* mix_ws, int64_t mix_ws_bytes, void* stream) {
  const char* who = "vy_hybrid_decoder_step";
  const vy_moe* d = L->moe;
  const int B = p->B;
  const int64_t n = d ? (int64_t)B * d->top : 0;
  if (p->dtype != VY_BF16 || L->form != VY_FORM_PARALLEL || L->mixer != VY_MIX_WINDOW || B > 64 || L->dim > 256 || L->vdim > 256 ||
      (L->ff && !L->clamped) || n > MAX_ENTRIES || (d && (d->experts > 256 || d->act != VY_MOE_CLAMPED)) || !L->gate || L->prep || L->diff || L->b_in)
    return VY_ERR_UNSUPPORTED;
  const int64_t nk = (int64_t)L->heads * L->dim, gk = (int64_t)L->kv_heads * L->dim, gv = (int64_t)L->kv_heads * L->vdim,
                nv = (int64_t)L->heads * L->vdim, na = nv + L->ff, n_in = nk + gk + gv + nv + 2 * (int64_t)L->ff;
  if (L->heads < 1 || L->kv_heads < 1 || L->heads % L->kv_heads || L->dim < 8 || L->vdim < 8 || L->dim % 8 || L->vdim % 8 ||
      L->ff % 8 || p->dp % 8 || L->n_in != n_in || !(L->scale > 0.f) || L->cap < 1 || !L->cache || !L->w_in || !L->w_o ||
      L->c_sh < (int64_t)L->cap * (L->dim + L->vdim) || L->c_ss < L->kv_heads * L->c_sh || L->c_sh % 8 || L->c_ss % 8)
    VY_FAIL(VY_ERR_ARG, "%s: bad window layer", who);
  if (L->rope_dims < 0 || L->rope_dims % 2 || L->rope_dims > L->dim || (L->rope_dims && (!L->rope || max_keys > L->rope_len)))
    VY_FAIL(VY_ERR_ARG, "%s: %ld positions, rotary table of %d", who, (long)max_keys, L->rope_len);
  if (d && (!d->w_router || !d->w_gu || !d->w_down || d->experts < 1 || d->top < 1 || d->top > 64 || d->groups < 1 || d->keep < 1 ||
            d->experts % d->groups || d->keep > d->groups || d->top > d->keep * (d->experts / d->groups) || d->width != p->dp ||
            d->group_best < 1 || d->group_best > 2 || d->ff < 8 || d->ff % 8 || moe_ws_bytes < vy_moe_ws_bytes(d, B, p->dtype)))
    VY_FAIL(VY_ERR_ARG, "%s: bad mixture", who);
  hipStream_t st = (hipStream_t)stream;
  const dim3 block(256);
  auto tiles_of = [&](int64_t rows) { return (int)(B == 1 ? (rows + 7) / 8 : (rows + 15) / 16); };

  // input products and router logits
  float* logits = (float*)moe_ws;
  bf16* act = d ? (bf16*)((char*)moe_ws + ((int64_t)B * d->experts * 4 + 255) / 256 * 256) : nullptr;
  const Dense din{(const bf16*)h, p->dp, B, (const bf16*)L->w_in, (int)n_in, p->dp, in, n_in, 0};
  const Dense drouter{(const bf16*)h, p->dp, B, d ? (const bf16*)d->w_router : nullptr, d ? d->experts : 0, p->dp, logits,
                      d ? d->experts : 0, 1};
  const int t_in = tiles_of(n_in);
  const dim3 g_in((unsigned)(t_in + (d ? tiles_of(d->experts) : 0)));
  if (B == 1) hipLaunchKernelGGL(parallel_in_kernel<0>, g_in, block, 0, st, din, drouter, t_in);
  else if (B <= 16) hipLaunchKernelGGL(parallel_in_kernel<1>, g_in, block, 0, st, din, drouter, t_in);
  else if (B <= 32) hipLaunchKernelGGL(parallel_in_kernel<2>, g_in, block, 0, st, din, drouter, t_in);
  else hipLaunchKernelGGL(parallel_in_kernel<4>, g_in, block, 0, st, din, drouter, t_in);

  // attention, choice, shared activation
  MixArgs m{};
  DecodeArgs& w = m.win;
  w.p = (const bf16*)in; w.ldp = n_in; w.oq = 0; w.ok = nk; w.ov = nk + gk; w.og = nk + gk + gv;
  w.ring = (bf16*)L->cache; w.r_ss = L->c_ss; w.r_sh = L->c_sh; w.R = L->cap; w.keep = L->keep;
  w.rope = (const float2*)L->rope; w.half = L->rope_dims / 2; w.rope_len = L->rope_len > 0 ? L->rope_len : 1;
  w.slots = slots; w.start = lengths; w.out = (bf16*)ao; w.ldo = na;
  w.h = L->heads; w.hk = L->kv_heads; w.dim = L->dim; w.vdim = L->vdim; w.scale = L->scale; w.sink = L->sink;
  w.passes = (L->heads / L->kv_heads + 15) / 16;
  w.ns = slices_of((int64_t)B * w.hk * w.passes, max_keys < L->cap ? max_keys : L->cap);
  if (w.ns > 1) {
    if (!mix_ws || mix_ws_bytes < (int64_t)B * w.h * w.ns * (w.vdim + 2) * 4) VY_FAIL(VY_ERR_ARG, "%s: workspace too small", who);
    w.part_o = (float*)mix_ws;
    w.part_ml = w.part_o + (int64_t)B * w.h * w.ns * w.vdim;
  }
  m.n_win = w.ns * w.hk * w.passes * B;
  if (d) {
    m.choose = ChooseArgs{logits, B, d->experts, d->top, d->groups, d->keep, d->score == VY_SCORE_SIGMOID, d->group_best, d->normalize, d->scale, nullptr, 1, eids, ew, nullptr, nullptr, nullptr};
    m.n_choose = (B + 3) / 4;
  }
  m.gu = (const bf16*)in + (n_in - 2 * (int64_t)L->ff); m.ldg = n_in; m.act = (bf16*)ao + nv; m.lda = na; m.B = B; m.ff = L->ff;
  m.limit = L->limit; m.alpha = L->alpha;
  const int blocks = m.n_win + m.n_choose + (L->ff ? (int)vy_cdiv((int64_t)B * (L->ff / 8), 256) : 0);
  if (L->dim <= 64) mix_go<64>(m, blocks, st);
  else if (L->dim <= 128) mix_go<128>(m, blocks, st);
  else mix_go<256>(m, blocks, st);

  // experts in, attention's slices
  const int active = d ? (int)(n < d->experts ? n : d->experts) : 0, n_finish = w.ns > 1 ? w.h * B : 0;
  ExpertRows up{}, down{};
  if (d) {
    up = ExpertRows{(const bf16*)h, p->dp, eids, (int)n, d->top, (const bf16*)d->w_gu, 2 * d->ff, p->dp, act, d->ff, d->limit, d->alpha};
    down = ExpertRows{act, d->ff, eids, (int)n, d->top, (const bf16*)d->w_down, p->dp, d->ff, (bf16*)erows, p->dp, 0.f, 0.f};
  }
  // 16 weight rows per workgroup, 32 where there are plenty (one sequence: 8)
  auto wide = [&](const ExpertRows& e) { return B > 1 && (int64_t)tiles_of(e.N) * active > 1536; };
  auto ex_tiles = [&](const ExpertRows& e) { return wide(e) ? (e.N + 31) / 32 : tiles_of(e.N); };
  if (n_finish + active) {
    const dim3 grid((unsigned)(n_finish + ex_tiles(up) * active));
    if (B == 1) hipLaunchKernelGGL(parallel_experts_kernel<0>, grid, block, 0, st, w, n_finish, up, ex_tiles(up));
    else if (wide(up)) hipLaunchKernelGGL(parallel_experts_kernel<2>, grid, block, 0, st, w, n_finish, up, ex_tiles(up));
    else hipLaunchKernelGGL(parallel_experts_kernel<1>, grid, block, 0, st, w, n_finish, up, ex_tiles(up));
  }

  // output products
  const Dense dout{(const bf16*)ao, na, B, (const bf16*)L->w_o, p->dp, (int)na, y, p->dp, 0};
  const int n_out = tiles_of(p->dp), t_down = ex_tiles(down), blocks_out = n_out + t_down * active;
  if (B == 1) hipLaunchKernelGGL((parallel_out_kernel<0, 0>), dim3((unsigned)blocks_out), block, 0, st, dout, n_out, down, t_down);
  else if (wide(down)) out_go<2>(B, dout, n_out, down, t_down, blocks_out, st);
  else out_go<1>(B, dout, n_out, down, t_down, blocks_out, st);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}
