/*
 * vyom_hip.h -- C ABI of libvyom_hip.so, the MI355X (gfx950 / CDNA4) kernel library
 * behind vyomai_amd's mirror of the VyomAI layer API.
 *
 * The reference (Ajax0564/VyomAI) has no FFI: its hot path is the Python class API of
 * VyomAI/layers consumed by VyomAI/models.  Each entry point
 * below replaces the torch ops that one reference call site issues; the citation after
 * "replaces:" is path:line in the reference checkout.
 *
 * Conventions (every function):
 *   - plain device pointers + explicit sizes/strides (in ELEMENTS unless noted), no torch types;
 *   - `dtype`: VY_F32 or VY_BF16 -- the storage type of activations/weights; accumulation,
 *     softmax and norm statistics are always fp32;
 *   - `stream` is a hipStream_t passed as void*; work is enqueued, never synchronised;
 *   - no device allocation inside; callers pass workspaces;
 *   - returns 0 on success, a negative vy_status otherwise; vy_last_error() describes it.
 */
#ifndef VYOM_HIP_H
#define VYOM_HIP_H

#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

typedef enum { VY_F32 = 0, VY_BF16 = 1 } vy_dtype;

typedef enum {
  VY_OK = 0,
  VY_ERR_ARG = -1,       /* bad shape / alignment / null pointer */
  VY_ERR_UNSUPPORTED = -2,
  VY_ERR_LAUNCH = -3     /* hipGetLastError() after the launch */
} vy_status;

typedef enum { VY_ACT_NONE = 0, VY_ACT_GELU_ERF = 1, VY_ACT_GELU_TANH = 2,
               VY_ACT_SILU = 3, /* gated products only (vy_gated_act_fwd, the decode steps) */
               VY_ACT_RELU2 = 4, /* max(x, 0)^2; products only */
               VY_ACT_SOFTCAP = 5 /* vy_linear_softcap_fwd */ } vy_act;
/* OR-ed into `act` of vy_linear_fwd / vy_linear_dgrad (training): the tensor saved for backward is act'(x W^T + b)
 * instead of the pre-activation -- the forward epilogue has Phi and the Gaussian of the erf GELU at hand anyway, and
 * the dgrad epilogue (dX = (dY W) * act') becomes one multiply per element instead of an erf + exp evaluation.
 * vy_linear_fwd: pre_out receives act' (rounded to the storage type); vy_linear_dgrad: `pre` holds act'. */
#define VY_ACT_SAVE_DERIV 0x100

/* attention mask descriptor bits (vy_attn_fwd / vy_attn_bwd) */
enum {
  VY_MASK_NONE = 0,
  VY_MASK_CAUSAL = 1,   /* key j visible to query i iff j <= i + start_pos              */
  VY_MASK_KEYPAD = 2,   /* uint8 keep[B][S]; 0 = masked with finfo.min like the reference */
  VY_MASK_ADDITIVE = 4  /* generic fp32 additive mask (B,1,Lm,S), Lm in {1, L}            */
};

const char* vy_last_error(void);
int vy_abi_version(void);

/* Launch-sizing hint: the caller is about to run `n` independent launch chains side by side on `n` streams (the
 * training forward as two batch halves, vyomai_amd/ops.py `lanes`), so each launch should size its grid for 1/n of
 * the 256 CUs: a 128-tile launch of 256 x 192 tiles is then a full share, not a half-empty chip.  n = 1 (the default)
 * restores whole-chip sizing.  Process-global, read on the host when a launch is sized; results never depend on it. */
int vy_set_concurrent_chains(int n);

/* Scratch for the launches on `stream` (the library never allocates device memory): mid-size GEMMs (32 < M <= ~2304 rows,
 * fewer than 300 tiles of 128 x 128) split K over workgroups and keep fp32 partial tiles here between their two launches
 * -- 64 KiB per (tile, slice), the widest launch (16 slices of 16 tiles of 320 x 128) needs 42 MiB; the host layer registers 64 MiB.  One workspace per stream (launches on one stream are
 * ordered, so they can share it); ws = NULL or bytes = 0 removes the entry.  Without a workspace such GEMMs run unsplit:
 * results are the same up to the fp32 summation order over K. */
int vy_workspace_set(void* stream, void* ws, int64_t bytes);

/* ------------------------------------------------------------------------------------------
 * vy_linear_fwd:  Y[M,N] = act(X[M,K] . W[N,K]^T + bias[N]) + residual[M,N]
 * replaces: nn.Linear call sites -- AttentionSelfOutput.dense + residual add
 *   (VyomAI/layers/attention.py:69-71), FeedForward.intermediate + GELU and FeedForward.out +
 *   residual (VyomAI/layers/ffn.py:35-39), LMHead.dense/decoder (VyomAI/models/decoder.py:267-275).
 * `pre_out` (nullable, [M,ldy]) receives X.W^T+bias before the activation (saved for backward).
 * bias/residual/pre_out may be NULL.  K % 8 == 0 (bf16) / K % 4 == 0 (f32); rows 16-byte aligned.
 * ------------------------------------------------------------------------------------------ */
int vy_linear_fwd(const void* x, int64_t ldx, const void* w, int64_t ldw, const void* bias,
                  const void* residual, int64_t ldr, void* y, int64_t ldy, void* pre_out,
                  int64_t M, int64_t N, int64_t K, int act, int dtype, void* stream);
/* vy_linear_softcap_fwd: Y = cap * tanh(X . W^T / cap), a vocabulary product whose logits stay within +-cap. */
int vy_linear_softcap_fwd(const void* x, int64_t ldx, const void* w, int64_t ldw, void* y, int64_t ldy, int64_t M, int64_t N,
                          int64_t K, float cap, int dtype, void* stream);

/* ------------------------------------------------------------------------------------------
 * vy_qkv_rope_fwd: fused Q/K/V projection + bias + rotary embedding + head split.
 * replaces: self.query/key/value (or self.qkv + chunk), rearrange 'b l (h d) -> b h l d',
 *   apply_rotary_pos_emb and the KV-cache slice write
 *   (VyomAI/layers/attention.py:114-126, 607-617; VyomAI/models/decoder.py:91-105;
 *    VyomAI/layers/positional_embeddings.py:155-182; VyomAI/layers/kv_cache.py:355-356).
 * w: packed [(h + 2*hk)*dh, K] rows = [Wq; Wk; Wv]; bias likewise or NULL.
 * cos/sin: fp32 tables [>= pos0+L][dh/2] (angles' cos/sin, half width) or NULL for no RoPE;
 *          row (pos0 + l) is used for token l.
 * q/k/v outputs are (B, heads, *, dh) with element strides {batch, head, token}; writing K/V
 * straight into a static cache is done by pointing k/v at cache[:, :, start_pos] with the
 * cache's strides.
 * ------------------------------------------------------------------------------------------ */
int vy_qkv_rope_fwd(const void* x, int64_t ldx, const void* w, int64_t ldw, const void* bias,
                    const float* cos_tab, const float* sin_tab, int64_t pos0,
                    void* q, int64_t q_sb, int64_t q_sh, int64_t q_sl,
                    void* k, int64_t k_sb, int64_t k_sh, int64_t k_sl,
                    void* v, int64_t v_sb, int64_t v_sh, int64_t v_sl,
                    int64_t B, int64_t L, int64_t K, int h, int hk, int dh, int dtype,
                    void* stream);

/* ------------------------------------------------------------------------------------------
 * vy_attn_fwd: softmax(Q K^T / sqrt(dh) + mask) V, flash style, heads merged on output.
 * replaces: repeat_kv + F.scaled_dot_product_attention + rearrange 'b h l d -> b l (h d)'
 *   (VyomAI/layers/attention.py:8-19, 128-132, 205-213, 283-287, 368-377, 619-623;
 *    VyomAI/models/decoder.py:107-111, 190-199).
 * q (B,h,L,dh), k/v (B,hk,S,dh) with element strides {batch, head, token}; kv head of query
 * head i is i / (h/hk).  out is (B, L, h*dh) with strides {o_sb, o_sl}.
 * mask_kind: OR of VY_MASK_*; keypad uint8 [B][S] (stride kp_sb); additive fp32 with strides
 * {am_sb, am_sl} (am_sl = 0 broadcasts one row).  Masked scores take finfo(fp32).min exactly as
 * the reference's (1-mask)*finfo.min does, so a fully masked row averages V.
 * lse (nullable) fp32 [B,h,L]: natural-log sum-exp of the scaled, masked scores (for backward).
 * ------------------------------------------------------------------------------------------ */
int vy_attn_fwd(const void* q, int64_t q_sb, int64_t q_sh, int64_t q_sl,
                const void* k, int64_t k_sb, int64_t k_sh, int64_t k_sl,
                const void* v, int64_t v_sb, int64_t v_sh, int64_t v_sl,
                void* out, int64_t o_sb, int64_t o_sl, float* lse,
                int mask_kind, int64_t start_pos, const uint8_t* keypad, int64_t kp_sb,
                const float* addmask, int64_t am_sb, int64_t am_sl,
                int64_t B, int h, int hk, int64_t L, int64_t S, int dh, float scale, int dtype,
                void* stream);

/* ------------------------------------------------------------------------------------------
 * vy_attn_decode: one query token per sequence against a KV cache (L == 1, no mask).
 * replaces: the L==1 branch of DecoderAttention*.forward (mask=None, VyomAI/models/decoder.py:
 *   355-356, 105-111) reading StaticCacheOne/DynamicCacheOne prefixes (VyomAI/layers/kv_cache.py:
 *   229-236, 358-361).  q (B,h,1,dh) strides {q_sb,q_sh}; k/v cache strides {batch, head, token};
 *   S = start_pos + 1 keys are attended.  out (B,1,h*dh) row stride o_sb.
 * ------------------------------------------------------------------------------------------ */
int vy_attn_decode(const void* q, int64_t q_sb, int64_t q_sh,
                   const void* k, int64_t k_sb, int64_t k_sh, int64_t k_sl,
                   const void* v, int64_t v_sb, int64_t v_sh, int64_t v_sl,
                   void* out, int64_t o_sb, int64_t B, int h, int hk, int64_t S, int dh,
                   float scale, int dtype, void* stream);

/* ------------------------------------------------------------------------------------------
 * vy_layernorm_fwd: y = (x - mean) * rstd * gamma + beta over the last dim (biased variance).
 * replaces: nn.LayerNorm in AttentionSelfOutput / FeedForward / LMHead
 *   (VyomAI/layers/attention.py:71, VyomAI/layers/ffn.py:39, VyomAI/models/decoder.py:270).
 * mean/rstd (nullable) fp32 [M] are saved for backward.
 * ------------------------------------------------------------------------------------------ */
int vy_layernorm_fwd(const void* x, int64_t ldx, const void* gamma, const void* beta, void* y,
                     int64_t ldy, float* mean, float* rstd, int64_t M, int64_t N, float eps,
                     int dtype, void* stream);

/* vy_rmsnorm_fwd: y = x * rsqrt(mean(x^2) + eps) * (w_offset + w); Gemma uses w_offset = 1
 * (Examples/paligemma.ipynb cell 11, GemmaRMSNorm).  Statistics in fp32. */
int vy_rmsnorm_fwd(const void* x, int64_t ldx, const void* w, void* y, int64_t ldy, int64_t M,
                   int64_t N, float eps, float w_offset, int dtype, void* stream);

/* vy_gated_act_fwd: out[m, i] = act(gate_up[m, i]) * gate_up[m, I + i] -- the GeGLU of GemmaMLP
 * (Examples/paligemma.ipynb cell 11: gelu_tanh(gate_proj(x)) * up_proj(x)) after one packed
 * [gate; up] projection. */
int vy_gated_act_fwd(const void* gate_up, int64_t ldg, void* out, int64_t ldo, int64_t M, int64_t I,
                     int act, int dtype, void* stream);

/* vy_clamped_act_fwd: with g = min(gate_up[m, i], limit), u = clamp(gate_up[m, I + i], -limit, limit):
 * out[m, i] = g * sigmoid(alpha * g) * (u + 1). */
int vy_clamped_act_fwd(const void* gate_up, int64_t ldg, void* out, int64_t ldo, int64_t M, int64_t I, float limit, float alpha,
                       int dtype, void* stream);

/* ------------------------------------------------------------------------------------------
 * Decoders with an fp32 residual stream (norm before and after every sublayer), latent attention and decayed linear
 * attention.  Conventions shared by this group:
 *   - rows may be padded: N columns are used of NP (NP a multiple of 8), and the padding is zero in weights and operands;
 *   - norm weights are fp32;
 *   - the batch of a launch is B sequences of L tokens; sequence b owns cache / state slot slots[b] (slots NULL: slot b) and
 *     already holds start[slot] tokens; count[b] <= L of its tokens are real (NULL: all L), the rest is padding behind them.
 *
 * vy_residual_norm: x (fp32) += norm(y) * w_post ; h = norm(x) * w_pre.  ids given: x = table[ids] instead (an id outside
 *   [0, V) gives zeros and sets *err_flag); w_post NULL: plain add; y and ids NULL: x is only read; h NULL: no second norm;
 *   h without w_pre: h = x, rounded to h's type.
 *   rms = 0: (v - mean) / sqrt(var + eps), rms = 1: v / sqrt(mean(v^2) + eps).
 * vy_residual_norm_routed: the same with y += sum_k weight[row][k] * rows[pos[row][k]] ahead of the post norm (routed
 *   nullable; weight fp32 and pos int32 are [M][top], pos NULL: row * top + k, pos < 0: left out; y NULL: the sum alone) and
 *   x = table_scale * table[ids].
 * vy_latent_norm: p = packed rows [query latent (npq) | key/value latent (npc) | ...]: q_out = RMSNorm(latent) * w_q,
 *   c_out (nullable) = RMSNorm(latent) * w_c, also written to cache[slot][start + l] (strides c_ss / c_st, cap rows per slot).
 *   w_q NULL: the first npq columns are no latent and left alone.  ring != 0: the cap rows are a ring, position p lives in row
 *   p % cap, and only the last cap tokens are written.
 * vy_rmsnorm_gate: y = RMSNorm(x) * w * sigmoid(gate).
 * ------------------------------------------------------------------------------------------ */
int vy_residual_norm(float* x, int64_t ldx, const void* y, int64_t ldy, const void* table, int64_t ldt, const int64_t* ids,
                     int64_t V, int32_t* err_flag, const float* w_post, float eps_post, const float* w_pre, float eps_pre,
                     void* h, int64_t ldh, int64_t M, int64_t N, int64_t NP, int rms, int dtype, void* stream);
typedef struct vy_routed_rows {
  const void* rows; int64_t ld;
  const int32_t* pos; const float* weight; int32_t top;
} vy_routed_rows;
int vy_residual_norm_routed(float* x, int64_t ldx, const void* y, int64_t ldy, const void* table, int64_t ldt,
                            const int64_t* ids, int64_t V, int32_t* err_flag, float table_scale, const vy_routed_rows* routed,
                            const float* w_post, float eps_post, const float* w_pre, float eps_pre, void* h, int64_t ldh,
                            int64_t M, int64_t N, int64_t NP, int rms, int dtype, void* stream);
int vy_latent_norm(const void* p, int64_t ldp, const float* w_q, void* q_out, int64_t ldq, int32_t nq, int32_t npq,
                   const float* w_c, void* c_out, int64_t ldc, int32_t nc, int32_t npc, void* cache, int64_t c_ss,
                   int64_t c_st, int32_t cap, int ring, const int32_t* slots, const int32_t* start, const int32_t* count, int64_t B,
                   int64_t L, float eps, int dtype, void* stream);
int vy_rmsnorm_gate(const void* x, int64_t ldx, const float* w, const void* gate, int64_t ldg, void* y, int64_t ldy, int64_t M,
                    int64_t N, int64_t NP, float eps, int dtype, void* stream);
/* vy_head_norm_gate: every head of a row by itself: y = x / rms(x) * w * silu(gate); heads of NP columns, N used; w (nullable): NP
 * factors shared by the heads, zero in the padding; gate nullable. */
int vy_head_norm_gate(const void* x, int64_t ldx, const float* w, const void* gate, int64_t ldg, void* y, int64_t ldy, int64_t M,
                      int32_t heads, int64_t N, int64_t NP, float eps, int dtype, void* stream);

/* vy_attn_fwd_ex: causal attention whose values may have a width of their own (dv), with a start position per sequence
 * (key j is visible to query i of sequence b iff j <= start[slot] + i; start NULL: 0) and an optional output gate:
 * out *= sigmoid(gate), gate laid out as out (strides g_sb, g_sl).
 * win (nullable) adds, with s_b = min(start[slot], start_cap) in the place of start[slot]:
 *   window     query i sees only the keys j > s_b + i - window (0: every earlier key) ...
 *   keep       ... and, whatever the window, the keys j < keep up to its own;
 *   sink       one more term exp(0) in every softmax denominator, without a value;
 *   rope       rotary positions of the queries: (cos, sin) pairs [rope_len][rope_dims / 2], fp32; columns 2c and 2c + 1 of the
 *              first rope_dims turn by the angle of position start[slot] + i (the keys are rotated already);
 *   kv_by_slot k and v are indexed by slots[b] instead of b (row-wise kernel);
 *   gate_heads the gate is one number per head, gate rows [h]. */
typedef struct vy_attn_window {
  int32_t window, sink, kv_by_slot, start_cap;
  const float* rope; int32_t rope_dims, rope_len;
  int32_t keep, gate_heads;
} vy_attn_window;
int vy_attn_fwd_ex(const void* q, int64_t q_sb, int64_t q_sh, int64_t q_sl, const void* k, int64_t k_sb, int64_t k_sh,
                   int64_t k_sl, const void* v, int64_t v_sb, int64_t v_sh, int64_t v_sl, void* out, int64_t o_sb,
                   int64_t o_sl, const void* gate, int64_t g_sb, int64_t g_sl, const int32_t* start, const int32_t* slots,
                   int64_t B, int h, int hk, int64_t L, int64_t S, int dh, int dv, float scale, const vy_attn_window* win,
                   int dtype, void* stream);

/* vy_moe_fwd: mixture of experts on rows h [M][width].  z = w_router h (fp32), scores softmax(z) or sigmoid(z); experts form
 * `groups` equal groups of neighbours, and only those of the `keep` best groups can be chosen (a group's score: the sum of its
 * group_best largest scores, 1 or 2); the `top` best of them are, with weight = scale * score, divided by (sum of the chosen
 * scores + 1e-20) if normalize.  Expert e, by `act`: VY_MOE_CLAMPED vy_clamped_act_fwd's activation between w_gu[e] (rows
 * interleaved: 2j gate j, 2j + 1 up j) and w_down[e]; VY_MOE_GELU the exact GELU between w_gu[e] (the up rows alone) and
 * w_down[e].  Nothing is added up here:
 *   rows   the experts' outputs, row stride ldr, M * top of them in an order of its own,
 *   pos    [M][top] a choice's row, weight [M][top] its weight (vy_residual_norm_routed takes the three), ids [M][top] its expert
 *          (-1, 0 and -1 for padding tokens: those with l >= count[b], m = b L + l; count nullable).
 * width and ff are padded to multiples of 8.  experts <= 1024, top <= 64. */
enum { VY_MOE_CLAMPED = 0, VY_MOE_GELU = 1 };
enum { VY_SCORE_SOFTMAX = 0, VY_SCORE_SIGMOID = 1 };
typedef struct vy_moe {
  int32_t experts, top, groups, keep, width, ff;
  int32_t act, score, group_best, normalize;
  float scale, limit, alpha;
  const void *w_router, *w_gu, *w_down;   /* [experts][width], [experts][2 ff or ff][width], [experts][width][ff] */
} vy_moe;
int64_t vy_moe_ws_bytes(const vy_moe* d, int64_t M, int dtype);
int vy_moe_fwd(const vy_moe* d, const void* h, int64_t ldh, int64_t M, const int32_t* count, int64_t L, void* rows, int64_t ldr,
               int32_t* ids, int32_t* pos, float* weight, void* ws, int64_t ws_bytes, int dtype, void* stream);

/* Sliding-window attention over a ring of keys and values.  Per slot and key/value head the ring holds R rows [key (dim) |
 * value (vdim)] (strides r_ss per slot, r_sh per head).  The first `keep` tokens of a sequence stay visible for good: position p
 * lives in row p while p < R, later ones in row keep + (p - keep) % (R - keep); R is keep + the window, or less while no sequence
 * is longer than R.  Packed projection rows p (stride ldp): queries at column oq ([h][dim]), keys ok ([hk][dim]), values ov
 * ([hk][vdim]), output gate og ([h][vdim], og < 0: none).  rope / rope_dims / rope_len as in vy_attn_window.
 *
 * (vdim 0: rows of one part, the keys', for vy_window_rows and vy_window_context.)
 *
 * vy_window_rows: rotate != 0: rotary positions on the new keys, in place; store != 0: those of the count[b] new rows of every
 *   sequence that its ring still holds behind them, to the ring.
 * vy_window_context: ctx [B][hk][S][dim + vdim] = min(start, past) rows of the ring in order of position (the kept ones, then the
 *   last of the others), then the L new rows (rotated already), then zeros: what vy_attn_fwd_ex takes with start_cap = past.
 * vy_qkv_rows: what a vy_qkv_prep asks for, in place on the packed rows: RMS norms of the whole query and of the whole key
 *   projection or of groups of their columns, rotary positions on both, a temperature on the queries, values mixed; store != 0:
 *   as vy_window_rows.
 * vy_window_decode: one new token per sequence (L = 1): its key and value to the ring, then attention of its queries over the
 *   ring with sink and gate, prep (nullable) as in vy_qkv_rows; diff (nullable): differential attention, without sink, gate and
 *   rope; max_keys >= every start + 1; ws: vy_window_decode_ws_bytes(...).  scale > 0.
 * vy_diff_attn_fwd: causal differential attention of packed queries (B sequences of L rows, row stride ldq, heads of dim columns)
 *   over keys and values that lie in a ring which has not wrapped (row = position): the new tokens' rows are in it already.
 *   out rows [h][vdim]; rows behind count[b] hold finite numbers. */
typedef struct vy_qkv_prep {
  const float *q_norm, *k_norm;     /* [h][dim], [hk][dim] factors (NULL: no norms), zero in padded columns */
  int32_t n_q, n_k;                 /* columns the norms divide by */
  float eps, lambda;
  const void* v_mix; int64_t ldm;   /* nullable: v <- (1 - lambda) v + lambda v_mix, both as flat rows of their used columns */
  int32_t n_v, m_v, m_vp;           /* used columns of a value head; of v_mix's heads, and those with their padding (m_v 0: as v's) */
  void* v_out; int64_t ldo;         /* nullable: receives the values as they were before mixing */
  int32_t group;                    /* 0: norms over whole projections; else over every `group` neighbouring columns by themselves
                                       (n_q = n_k of them used; dim a multiple of group); no v_mix / v_out then */
  int32_t temp_every; float temp_coef;  /* temp_every > 0 (with group): the query of position p times
                                       1 + temp_coef * ln(floor((p + 1) / temp_every) + 1) */
} vy_qkv_prep;
/* Differential attention: a head's dim columns of queries and keys are [map 1 | map 2], two attentions over the same values.  With
 * their outputs a1, a2: o = a1 - lambda a2, out = o / rms(o) * out_scale over a head's n_v used value columns. */
typedef struct vy_diff {
  float lambda, out_scale, eps;
  int32_t n_v;
} vy_diff;
int vy_qkv_rows(void* p, int64_t ldp, int64_t oq, int64_t ok, int64_t ov, const vy_qkv_prep* prep, void* ring, int64_t r_ss,
                int64_t r_sh, int32_t R, int32_t keep, const float* rope, int32_t rope_dims, int32_t rope_len, int store,
                const int32_t* slots, const int32_t* start, const int32_t* count, int64_t B, int64_t L, int32_t h, int32_t hk,
                int32_t dim, int32_t vdim, int dtype, void* stream);
int vy_window_rows(void* p, int64_t ldp, int64_t ok, int64_t ov, void* ring, int64_t r_ss, int64_t r_sh, int32_t R, int32_t keep,
                   const float* rope, int32_t rope_dims, int32_t rope_len, int rotate, int store, const int32_t* slots,
                   const int32_t* start, const int32_t* count, int64_t B, int64_t L, int32_t hk, int32_t dim, int32_t vdim,
                   int dtype, void* stream);
int vy_window_context(const void* p, int64_t ldp, int64_t ok, int64_t ov, const void* ring, int64_t r_ss, int64_t r_sh,
                      int32_t R, int32_t keep, void* ctx, int32_t S, int32_t past, const int32_t* slots, const int32_t* start, int64_t B,
                      int64_t L, int32_t hk, int32_t dim, int32_t vdim, int dtype, void* stream);
int64_t vy_window_decode_ws_bytes(int32_t B, int32_t h, int32_t hk, int32_t vdim, int32_t R, int diff);
int vy_window_decode(void* p, int64_t ldp, int64_t oq, int64_t ok, int64_t ov, int64_t og, void* ring, int64_t r_ss, int64_t r_sh,
                     int32_t R, int32_t keep, const float* rope, int32_t rope_dims, int32_t rope_len, const vy_qkv_prep* prep,
                     const vy_diff* diff, const int32_t* slots, const int32_t* start, int64_t max_keys, void* out, int64_t ldo, int64_t B, int32_t h, int32_t hk,
                     int32_t dim, int32_t vdim, float scale, int32_t sink, void* ws, int64_t ws_bytes, int dtype, void* stream);

int vy_diff_attn_fwd(const void* q, int64_t ldq, const void* ring, int64_t r_ss, int64_t r_sh, int32_t R, const vy_diff* diff,
                     const int32_t* slots, const int32_t* start, const int32_t* count, void* out, int64_t ldo, int64_t B, int64_t L,
                     int32_t h, int32_t hk, int32_t dim, int32_t vdim, float scale, int dtype, void* stream);

/* vy_latent_decode: one query token per sequence against a cache of latents c (one row of R per token, shared by all
 * heads).  Keys and values are never expanded:  q~_h = Wuk_h^T q_h,  s_j = scale * q~_h . c_j over j <= start[slot],
 * u_h = sum_j softmax(s)_j c_j,  out_h = (Wuv_h u_h) * sigmoid(gate_h)  (gate nullable).
 *   q [B][h*dh] (row stride ldq), wukt [h][R][dh] (= Wuk_h transposed), wuv [h][dv][R], out / gate rows [h*dv];
 *   cache rows cache[slot][j] with strides c_ss / c_st; max_keys >= every start + 1 (sizes the grid, cap rows per slot);
 *   ring > 0: a slot's rows are a ring of that many (vy_latent_norm), all of whose tokens are seen; gate_heads != 0: gate rows [h],
 *   one number per head.  ws: vy_latent_decode_ws_bytes(...) of scratch.  dh, dv, R multiples of 8, R <= 1024. */
int64_t vy_latent_decode_ws_bytes(int32_t B, int32_t h, int32_t R);
int vy_latent_decode(const void* q, int64_t ldq, const void* wukt, const void* wuv, const void* cache, int64_t c_ss,
                     int64_t c_st, const int32_t* slots, const int32_t* start, int64_t max_keys, void* out, int64_t ldo,
                     const void* gate, int64_t ldg, int gate_heads, int32_t ring, int32_t B, int32_t h, int32_t dh, int32_t dv,
                     int32_t R, float scale, void* ws, int64_t ws_bytes, int dtype, void* stream);

/* vy_decay_attn: linear attention with a per-head decay on packed rows p (row stride ldp; q / k / v of head a at columns
 * oq + a*dk, ok + a*dk, ov + a*dv):  S_t = decay_a S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t  with q, k, v = silu of the
 * projections (silu = 0: taken as they are).  rope (nullable; as in vy_attn_window): rotary positions on q and k, in fp32 and
 * not rounded before the recurrence; k is multiplied by k_scale behind it.  state: fp32 [slot][h][dk][dv], taken as zero where start[slot] == 0 and left as
 * S after the sequence's last real token.  decay_pow: fp32 [h][VY_DECAY_CHUNK + 1], decay_a^0 .. decay_a^CHUNK.
 * out rows [h*dv].  ws: vy_decay_attn_ws_bytes(...) of scratch (chunked prefill: bf16, L > 1, dk <= 128; otherwise the
 * token-by-token recurrence runs and ws may be NULL).  dk, dv multiples of 8, dk <= 512. */
#define VY_DECAY_CHUNK 64
int64_t vy_decay_attn_ws_bytes(int64_t B, int64_t L, int32_t h, int32_t dk, int32_t dv, int dtype);
int vy_decay_attn(const void* p, int64_t ldp, int64_t oq, int64_t ok, int64_t ov, float* state, const float* decay_pow,
                  const int32_t* slots, const int32_t* start, const int32_t* count, void* out, int64_t ldo, int64_t B,
                  int64_t L, int32_t h, int32_t dk, int32_t dv, int silu, const float* rope, int32_t rope_dims, int32_t rope_len,
                  float k_scale, void* ws, int64_t ws_bytes, int dtype, void* stream);

/* vy_gated_attn: linear attention with a forget gate f per key channel, tied to the input gate 1 - f, on packed rows p (q, gate
 * logits z and v of head a at columns oq + a*dk, of + a*dk, ov + a*dv):
 *   f = lower + (1 - lower) * sigmoid(z + bias),   S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T,   o_t = S_t^T q_t
 * with q = silu of its projection (silu = 0: taken as it is); bias (nullable) and lower fp32 [h][dk] (lower 1 in padded channels).
 * Everything else as in vy_decay_attn; ws: vy_gated_attn_ws_bytes(...). */
int64_t vy_gated_attn_ws_bytes(int64_t B, int64_t L, int32_t h, int32_t dk, int32_t dv, int dtype);
int vy_gated_attn(const void* p, int64_t ldp, int64_t oq, int64_t of, int64_t ov, float* state, const float* bias,
                  const float* lower, const int32_t* slots, const int32_t* start, const int32_t* count, void* out, int64_t ldo,
                  int64_t B, int64_t L, int32_t h, int32_t dk, int32_t dv, int silu, void* ws, int64_t ws_bytes, int dtype,
                  void* stream);

/* vy_rope_fwd: in-place rotary embedding on a (B,heads,L,dh) tensor (strides as above);
 * used when the fused epilogue does not apply.  `inverse` != 0 applies the transpose rotation
 * (the backward of RoPE).  replaces: VyomAI/layers/positional_embeddings.py:155-182. */
int vy_rope_fwd(void* x, int64_t sb, int64_t sh, int64_t sl, const float* cos_tab,
                const float* sin_tab, int64_t pos0, int64_t B, int heads, int64_t L, int dh,
                int inverse, int dtype, void* stream);

/* ------------------------------------------------------------------------------------------
 * Backward / training entry points (bf16 storage, fp32 accumulation).
 * They mirror what autograd derives for the reference modules; the fusion groups follow the
 * author's own fused notebook (Examples/vyom-ai-decoder-fused.ipynb cells 2-7, 11).
 * ------------------------------------------------------------------------------------------ */

/* dX[M,K] = dY[M,N] . W[N,K]  (+ add_to[M,K] + add_to2[M,K]); optional GELU backward: when `pre` is
 * given the result is multiplied by gelu'(pre[M,K]) (pre = saved pre-activation of the consumer of
 * dX).  wt is W transposed, i.e. stored [K,N] row-major (the trainer keeps both copies).  The two
 * addends are the residual-path gradients a layer input collects besides the QKV projection's
 * (add_to2 needs add_to). */
int vy_linear_dgrad(const void* dy, int64_t lddy, const void* wt, int64_t ldwt, const void* pre,
                    int64_t ldpre, int act, const void* add_to, int64_t ldadd, const void* add_to2,
                    int64_t ldadd2, void* dx, int64_t lddx, int64_t M, int64_t N, int64_t K, int dtype,
                    void* stream);

/* dW[N,K] (fp32, accumulate when beta != 0) = alpha * dY[M,N]^T . X[M,K];  db[N] (fp32) likewise
 * alpha * colsum(dY).  alpha_dev: optional DEVICE fp32 scalar (NULL = 1), e.g. the upstream
 * gradient of a loss whose unit gradient is already stored in dY -- no host sync to read it.
 * dtype VY_BF16: MFMA kernels (K, lddy, ldx multiples of 8).  VY_F32: the parity path, plain FMAs
 * (any K; the reference's autograd of nn.Linear in full precision). */
int vy_linear_wgrad(const void* dy, int64_t lddy, const void* x, int64_t ldx, float* dw,
                    int64_t lddw, float* db, float beta, const float* alpha_dev, int64_t M, int64_t N,
                    int64_t K, int dtype, void* stream);

/* Several weight gradients in one launch: dW_i += dY_i^T X_i and db_i += column sums of dY_i (db_i may be NULL)
 * for 1..8 GEMMs, accumulating (the beta = 1 form of vy_linear_wgrad).  The four projections of a
 * transformer layer (reference: the autograd of the nn.Linear layers at layers/attention.py:87-95, :57-72,
 * layers/ffn.py:19-40) are small as wgrad problems -- 9 to 36 output tiles of 256 x 256 -- and filling the
 * chip one at a time costs M-splits, i.e. fp32 atomic traffic; together they need a quarter of it. */
typedef struct vy_wgrad_desc {
  const void* dy; int64_t lddy;
  const void* x; int64_t ldx;
  float* dw; int64_t lddw;
  float* db;
  int64_t M, N, K;
} vy_wgrad_desc;
int vy_linear_wgrad_grouped(const vy_wgrad_desc* descs, int32_t n, int dtype, void* stream);

/* LayerNorm backward: dx = rstd*(g - mean(g) - xhat*mean(g*xhat)), g = dy*gamma;
 * dgamma/dbeta fp32 [N] accumulated (beta) from per-block partials in `ws`
 * (ws: fp32, at least 2 * ws_rows * N elements; ws_rows = vy_layernorm_bwd_ws_rows(M)). */
int64_t vy_layernorm_bwd_ws_rows(int64_t M);
int vy_layernorm_bwd(const void* dy, int64_t lddy, const void* x, int64_t ldx, const void* gamma,
                     const float* mean, const float* rstd, void* dx, int64_t lddx, float* dgamma,
                     float* dbeta, float beta, float* ws, int64_t M, int64_t N, int dtype,
                     void* stream);

/* Flash attention backward.  dO/O are (B,L,h*dh) (strides {sb,sl}); dq/dk/dv use q/k/v layouts.
 * delta_ws: fp32 [B,h,L] scratch.  dk/dv are (B,hk,S,dh): the n_rep query heads of one kv head
 * are summed in-kernel.  Same mask descriptor as the forward.  cos_tab/sin_tab (nullable): when
 * q/k were rotated by RoPE (row rope_pos0 + token of the tables), the inverse rotation is applied
 * to dq and dk (in the epilogues at dh = 64 bf16, by rotation launches otherwise), so they are
 * gradients w.r.t. the un-rotated projections.
 * bf16: dh = 64 (tuned kernels) or any multiple of 8 up to 256 (general MFMA kernels; SigLIP's 72 runs
 * as 96 columns).  fp32: the parity path (plain FMAs, expf), dh a multiple of 8 up to 256 -- there a
 * row without a visible key is differentiated as the uniform softmax the forward returned for it
 * (reference layers/attention.py:133-137 under autograd); the bf16 kernels give such rows no gradient. */
int vy_attn_bwd(const void* q, int64_t q_sb, int64_t q_sh, int64_t q_sl,
                const void* k, int64_t k_sb, int64_t k_sh, int64_t k_sl,
                const void* v, int64_t v_sb, int64_t v_sh, int64_t v_sl,
                const void* out, const void* dout, int64_t o_sb, int64_t o_sl, const float* lse,
                float* delta_ws,
                void* dq, int64_t dq_sb, int64_t dq_sh, int64_t dq_sl,
                void* dk, int64_t dk_sb, int64_t dk_sh, int64_t dk_sl,
                void* dv, int64_t dv_sb, int64_t dv_sh, int64_t dv_sl,
                int mask_kind, int64_t start_pos, const uint8_t* keypad, int64_t kp_sb,
                const float* cos_tab, const float* sin_tab, int64_t rope_pos0,
                int64_t B, int h, int hk, int64_t L, int64_t S, int dh, float scale, int dtype,
                void* stream);

/* ---- data-parallel gradient exchange (RCCL) --------------------------------------------------------------------
 * Replaces what the reference gets from accelerate / torch DDP (Examples/vyom-ai-decoder_clm.ipynb cell 31,
 * Examples/vyom-ai-accelerate-multimodel-2t4.ipynb cells 1-2): one process per GPU, one communicator per process.
 *   vy_ddp_unique_id   rank 0 fills 128 bytes; the host hands them to every rank (any side channel: torch.distributed's
 *                      store, MPI, a file)
 *   vy_ddp_init        collective; binds the communicator to the calling thread's current HIP device
 *   vy_ddp_all_reduce_async  in-place SUM of `count` elements (VY_F32 | VY_BF16) enqueued on `stream`: the caller orders
 *                      it behind the kernels that wrote the bucket and ahead of its consumers with events / stream waits
 *                      (there is no separate wait call: completion is stream order)
 * RCCL is bound at run time (the copy already in the process, e.g. torch's, else librccl.so): where it is absent these
 * return VY_ERR_UNSUPPORTED.  The number of CUs RCCL's channel kernels occupy beside the backward GEMMs is RCCL's own
 * knob (NCCL_MAX_NCHANNELS / NCCL_MIN_NCHANNELS in the environment of the process), read at vy_ddp_init. */
int vy_ddp_unique_id(void* id128);
int vy_ddp_init(const void* id128, int rank, int world);
int vy_ddp_world(void);   /* 0 before vy_ddp_init */
int vy_ddp_rank(void);    /* -1 before vy_ddp_init */
int vy_ddp_all_reduce_async(void* buf, int64_t count, int dtype, void* stream);
int vy_ddp_destroy(void);

/* Fused AdamW over a flat fp32 parameter arena; also refreshes the bf16 working copy.
 * p, m, v fp32 [n]; g fp32 [n]; p_bf16 (nullable) bf16 [n].  Matches torch.optim.AdamW. */
int vy_adamw_step(float* p, const float* g, float* m, float* v, void* p_bf16, int64_t n, float lr,
                  float beta1, float beta2, float eps, float weight_decay, int64_t step,
                  float grad_scale, const float* grad_scale_dev, void* stream);
/* The same with a gate (nullable): one fp32 on the device; when it reads 0 the launch changes nothing.  Data-parallel
 * training with parameters that some ranks' batches do not reach (the reference's multimodal model under
 * find_unused_parameters=True, Examples/vyom-ai-accelerate-multimodel-2t4.ipynb cell 1): whether such a parameter is
 * updated is decided by a flag all-reduced over the ranks, read here on the device. */
int vy_adamw_step_gated(float* p, const float* g, float* m, float* v, void* p_bf16, int64_t n, float lr,
                        float beta1, float beta2, float eps, float weight_decay, int64_t step,
                        float grad_scale, const float* grad_scale_dev, const float* gate, void* stream);
/* grad_scale_dev (nullable): one fp32 on the device multiplied into grad_scale by the kernel -- the
 * clip_grad_norm_ coefficient min(1, max_norm / (norm + 1e-6)) of the reference's training loops
 * (Examples/vyomai-fused-kernals-2t4.ipynb cell 0) without a host round trip. */

/* out[0] = sum_i x[i]^2 over an fp32 arena (global gradient norm, same loops).  ws: >= 1024 floats of
 * scratch.  Two launches, fixed summation order (run-to-run identical). */
int vy_sumsq(const float* x, int64_t n, float* out, float* ws, void* stream);

/* ------------------------------------------------------------------------------------------
 * Dropout of the two hidden-state sites of a block.
 * replaces: self.dropout(hidden_states) between dense and the residual add in AttentionSelfOutput
 *   (VyomAI/layers/attention.py:55,69-71) and FeedForward (VyomAI/layers/ffn.py:24,37-39), p =
 *   config.hidden_dropout_prob (VyomAI/utils.py:96, default 0.1), active in train().
 * The keep mask is a pure function of (seed, offset, row, column) -- Philox4x32-7 on the counter
 * {column / 8, row, offset}, sixteen bits per element, drop when below round(p * 65536) -- so the forward
 * epilogue, the backward pass and a test all regenerate it; nothing is stored.
 * vy_linear_dropout_fwd: Y = dropout(X . W^T + bias) / (1 - p) + residual   (vy_linear_fwd with the
 *   mask applied in the epilogue, before the residual add).
 * vy_dropout: y = x * keep / (1 - p) as its own pass over an [M, N] view (backward: the same mask on the
 *   incoming gradient; x = ones gives the mask).
 * ------------------------------------------------------------------------------------------ */
int vy_linear_dropout_fwd(const void* x, int64_t ldx, const void* w, int64_t ldw, const void* bias,
                          const void* residual, int64_t ldr, void* y, int64_t ldy, int64_t M, int64_t N,
                          int64_t K, float p_drop, uint64_t seed, uint64_t offset, int dtype, void* stream);
int vy_dropout(const void* x, int64_t ldx, void* y, int64_t ldy, int64_t M, int64_t N, float p_drop,
               uint64_t seed, uint64_t offset, int dtype, void* stream);

/* dx = dy * act'(pre), elementwise over [M,N] row-major views (GELU backward outside a GEMM). */
int vy_act_bwd(const void* dy, int64_t lddy, const void* pre, int64_t ldpre, void* dx, int64_t lddx,
               int64_t M, int64_t N, int act, int dtype, void* stream);

/* Softmax cross-entropy over the vocabulary, ignore_index aware (the CLM loss of
 * Examples/vyom-ai-decoder_clm.ipynb cell 29 after the label shift).
 * fwd: lse[m] = logsumexp(logits[m,:V]); loss_sum += sum_m (lse[m] - logits[m,label]) and
 *      count += #(label != ignore) -- both fp32 scalars on the device, accumulated atomically
 *      (zero them first).
 * bwd: logits[m,:] <- (softmax(logits[m,:]) - onehot(label)) * (*gscale) / (*count), in place
 *      (rows with label == ignore become 0); gscale/count are device pointers: no host sync. */
int vy_xent_fwd(const void* logits, int64_t ld, const int64_t* labels, int64_t ignore_index, float* lse,
                float* loss_sum, float* count, int64_t M, int64_t V, int32_t* err_flag, int dtype, void* stream);
int vy_xent_bwd(void* logits, int64_t ld, const int64_t* labels, int64_t ignore_index, const float* lse,
                const float* gscale, const float* count, int64_t M, int64_t V, int dtype, void* stream);
/* Both in ONE pass over the logits (bf16, V <= 65536): `count` (device scalar: the number of rows
 * with label != ignore) is an INPUT here; lse and loss_sum as in vy_xent_fwd, then the row is
 * overwritten in place as in vy_xent_bwd.  The logits cross HBM once in each direction. */
int vy_xent_fused(void* logits, int64_t ld, const int64_t* labels, int64_t ignore_index, float* lse,
                  float* loss_sum, const float* count, const float* gscale, int64_t M, int64_t V,
                  int32_t* err_flag, int dtype, void* stream);
/* A label that is neither ignore_index nor inside [0, V) (torch.cross_entropy device-asserts on it) is
 * never dereferenced: the row counts as ignored (zero loss, zero gradient) and *err_flag (nullable,
 * device int32) is set to 1 for the host to report. */

/* Token embedding (nn.Embedding: VyomAI/models/decoder.py:287, encoder.py:41, multimodel.py):
 * fwd: out[m,:] = table[ids[m],:] (bf16 or fp32).  Ids outside [0,V) give a zero row and set the
 *      optional device flag *err_flag to 1 (the host cannot check ids without a sync).
 * bwd: dW[ids[m],:] += dOut[m,:] in fp32 (atomics), except for id == padding_idx (pass -1 for none). */
int vy_embedding_fwd(const void* table, int64_t ldt, const int64_t* ids, void* out, int64_t ldo,
                     int64_t M, int64_t d, int64_t V, int32_t* err_flag, int dtype, void* stream);
int vy_embedding_bwd(const void* dout, int64_t lddo, const int64_t* ids, float* dw, int64_t lddw,
                     int64_t padding_idx, int64_t M, int64_t d, int64_t V, int dtype, void* stream);

/* out[c, r] = in[r, c] for a [R,C] matrix (bf16 or f32): keeps W^T copies for dgrad. */
int vy_transpose(const void* in, int64_t ldin, void* out, int64_t ldout, int64_t R, int64_t C,
                 int dtype, void* stream);

/* Many transposes in one launch: descs_dev is a DEVICE array of n descriptors; tile0 is the running
 * sum of ceil(R/64)*ceil(C/64) over the preceding descriptors, tiles_c = ceil(C/64), total_tiles the
 * sum over all.  Used once per training step for every W^T the dgrad GEMMs read. */
typedef struct vy_transpose_desc {
  const void* in; void* out;      /* in: [R,C] row-major (ldin); out: [C,R] (ldout) */
  int64_t ldin, ldout;
  int32_t R, C, tile0, tiles_c;
} vy_transpose_desc;              /* 48 bytes */
int vy_transpose_batched(const vy_transpose_desc* descs_dev, int32_t n, int32_t total_tiles, int dtype,
                         void* stream);

/* Sampling front end of the generate loops.
 * vy_greedy_step replaces reference models/decoder.py:478-507 (topk(k=1), the where() that forces prompt
 *   tokens, the token write, the isin()/or of the EOS bookkeeping and the all() reduction) for one
 *   generated position: for row b, next = argmax_v logits[b,v] (lowest index among equal maxima) unless
 *   text_mask[b,cur_pos] != 0 (the row is still inside its prompt), then next = tokens[b,cur_pos];
 *   tokens[b,cur_pos] = next; eos_reached[b] |= !forced && next in eos_ids[0..n_eos); *not_done (may be
 *   NULL; zeroed by the caller) += number of rows with eos_reached[b] == 0 afterwards.
 * vy_sampling_probs replaces reference logits_processors.py LogitsProcessor.__call__ for the five
 *   processors: probs = softmax(mask(logits) / temperature) in fp32.  top_k > 0 keeps the values >= the
 *   k-th largest (:59-63); 0 < top_p < 1 keeps the descending-sorted prefix up to and including the first
 *   element whose cumulative softmax of the unscaled, top-k-masked logits exceeds top_p (:73-81, :92-102);
 *   masked entries get probability exactly 0 (the reference writes -1e20 into them).  Equal logits at
 *   the nucleus cut are all kept (the reference keeps an implementation-defined subset of a tie). */
int vy_greedy_step(const void* logits, int64_t ldl, int64_t B, int64_t V, int dtype, int64_t* tokens,
                   int64_t ldt, int64_t cur_pos, const uint8_t* text_mask, int64_t ldm,
                   const int64_t* eos_ids, int32_t n_eos, uint8_t* eos_reached, int32_t* not_done, void* stream);
int vy_sampling_probs(const void* logits, int64_t ldl, int64_t B, int64_t V, int dtype, float temperature,
                      int32_t top_k, float top_p, float* probs, int64_t ldp, void* stream);

/* y = x converted between fp32 and bf16 (n elements). src_dtype -> dst_dtype. */
int vy_cast(const void* src, void* dst, int64_t n, int src_dtype, int dst_dtype, void* stream);

/* ------------------------------------------------------------------------------------------
 * Native decode driver: one call runs a whole single-token step (L == 1) of the GPT-style
 * decoder -- every layer's QKV+RoPE (K/V appended to the static cache in place), cached
 * attention, out-projection + residual + LayerNorm, FFN + residual + LayerNorm, then the LM head
 * -- as ~8 launches per layer with no host work in between.
 * replaces: the per-token body of DecoderModel.generate / DecoderModel.forward for seqlen == 1
 *   (VyomAI/models/decoder.py:343-374, 477-488) and DecoderLayer.forward (:222-250).
 * All pointers are device pointers; weights are `dtype` (bf16 or f32) in nn.Linear layout.
 * ------------------------------------------------------------------------------------------ */
typedef struct {
  const void *wqkv, *bqkv;          /* packed [(h+2hk)*dh, d], [(h+2hk)*dh] (bias may be NULL) */
  const void *wo, *bo, *ln1_w, *ln1_b;
  const void *w1, *b1, *w2, *b2, *ln2_w, *ln2_b;
  void *kcache, *vcache;            /* (B, hk, cap, dh) */
  int64_t c_sb, c_sh, c_sl;         /* cache element strides {batch, head, token} */
} vy_decode_layer;

typedef struct {
  int32_t num_layers, B, d, h, hk, dh, ffn, vocab, act, dtype;
  float eps_attn, eps_ffn, eps_head;
  const float *cos_tab, *sin_tab;   /* NULL: no RoPE (additive position encodings) */
  const vy_decode_layer* layers;    /* host array [num_layers] */
  const void *head_wd, *head_bd, *head_ln_w, *head_ln_b, *head_wv, *head_bias;
  void* ws; int64_t ws_bytes;       /* device workspace, >= vy_decode_ws_bytes(...) */
} vy_decode_plan;

int64_t vy_decode_ws_bytes(int32_t B, int32_t d, int32_t h, int32_t hk, int32_t dh, int32_t ffn,
                           int32_t dtype);
/* x: (B, d) input embeddings (+ position info); pos: index of this token (keys 0..pos are
 * attended); hidden_out (nullable): (B, d) last hidden state; logits (nullable): (B, ldv).
 * pos_dev (nullable): device int32 holding the position -- when given, every kernel reads the
 * position on the device and `pos` is ignored, so one captured hipGraph of this call can be
 * replayed for every token (bf16, head_dim 64 models). */
int vy_decoder_step(const vy_decode_plan* plan, const void* x, int64_t pos, const int32_t* pos_dev,
                    void* hidden_out, void* logits, int64_t ldv, void* stream);

/* ------------------------------------------------------------------------------------------
 * vy_gemma_decoder_step: one single-token step of a Gemma-style decoder stack (the
 * PaliGemma-shape language model; Examples/paligemma.ipynb cells 11-13): per layer
 *   n = RMSNorm(x) ; q,k,v = n Wqkv^T (+b) with RoPE, k/v written into the cache at `pos` ;
 *   x = x + attn(q, K[0..pos], V[0..pos]) Wo^T ; n = RMSNorm(x) ; x = x + (gelu_tanh(n Wg^T) * n Wu^T) Wd^T
 * then the final RMSNorm and the (tied) vocabulary projection.  Same launches as the Python layer
 * (models/paligemma.py GemmaDecoderLayer), one C call per generated token instead of ~150.
 * -------------------------------------------------------------------------------------------- */
typedef struct vy_gemma_layer {
  const void* wqkv; const void* bqkv;      /* packed [q;k;v] projection, bias may be NULL */
  const void* wo; const void* bo;
  const void* ln_in; const void* ln_post;  /* RMSNorm weights (applied as 1 + w) */
  const void* wgu;                         /* packed [gate; up], [2*ffn, d] */
  const void* wdown;                       /* [d, ffn] */
  void* kcache; void* vcache;              /* (B, hk, cap, dh) */
  int64_t c_sb, c_sh, c_sl;
} vy_gemma_layer;
typedef struct vy_gemma_plan {
  int32_t num_layers, B, d, h, hk, dh, ffn, vocab, dtype;
  float eps;
  const float* cos_tab; const float* sin_tab;
  const vy_gemma_layer* layers;
  const void* norm_w; const void* head_w;  /* final RMSNorm, [vocab, d] projection */
  void* ws; int64_t ws_bytes;              /* >= vy_gemma_ws_bytes(...) */
  int32_t flags;                           /* VY_GEMMA_PRESCALED: every layer's wqkv / wgu is already multiplied by
                                              (1 + ln_in) / (1 + ln_post) along K (bf16, B <= 4): the step skips the
                                              RMSNorm launches and scales each product by rsqrt(mean x^2 + eps) */
} vy_gemma_plan;
#define VY_GEMMA_PRESCALED 1
int64_t vy_gemma_ws_bytes(int32_t B, int32_t d, int32_t h, int32_t dh, int32_t ffn, int32_t dtype);
/* x: (B, d) embeddings of the current token (already scaled by sqrt(d)); keys 0..pos are attended;
 * logits: (B, ldv). */
int vy_gemma_decoder_step(const vy_gemma_plan* plan, const void* x, int64_t pos, void* logits, int64_t ldv,
                          void* stream);

/* ------------------------------------------------------------------------------------------
 * vy_hybrid_decoder_step: one new token for each of B sequences of a decoder that mixes layer kinds over an fp32 residual
 * stream.  Forms of a layer:
 *   VY_FORM_SANDWICH  h = norm(x) * norm1; y = w_o mixer(h); x += norm(y) * norm1b;
 *                     h = norm(x) * norm2; x += norm(ff(h)) * norm2b                       (ff = 0 and no moe: no second half)
 *                     norm1 / norm2 NULL: the sublayers read x itself
 *   VY_FORM_PARALLEL  h = norm(x) * norm1; x += w_o [mixer(h) | act(h)] + routed(h): one packed product w_in of h also gives the
 *                     [gate; up] rows of a dense feed-forward of width ff (its last 2 ff rows), one product w_o takes both back
 * w_up instead of w_gu: a feed-forward without a gate, w_down act(w_up h) with the plan's act (VY_FORM_SANDWICH).
 * norm1b / norm2b NULL: no norm on a sublayer's output.  moe (nullable): routed experts, added to the feed-forward's output.
 * clamped: the feed-forward's activation is vy_clamped_act_fwd's (limit, alpha), else the plan's act.
 * Mixers, all from ONE packed input projection w_in of h:
 *   VY_MIX_LATENT  rows [query latent | key/value latent | output gate]: vy_latent_norm, q = w_uq latent, vy_latent_decode;
 *                  w_uq NULL: rows [q | key/value latent | output gate]; ring: the cache is a ring of cap rows; gate 0: none;
 *                  gate_heads: one gate per head
 *   VY_MIX_DECAY   rows [q | k | v | output gate]: vy_decay_attn (silu, rope, k_scale), then vy_rmsnorm_gate, or without
 *                  mix_norm vy_head_norm_gate (mix_n: columns of a head)
 *   VY_MIX_GATED   rows [q | gate logits | v]: vy_gated_attn (f_bias, f_lower, silu), then vy_head_norm_gate with mix_norm
 *   VY_MIX_WINDOW  rows [q | k | v | output gate if gate]: vy_window_decode on the ring `cache` (strides c_ss per slot, c_sh per
 *                  head); prep (nullable): its norms, and lambda; values: VY_VALUES_FIRST keeps this layer's values,
 *                  VY_VALUES_MIX mixes them in (the step's own buffer is prep's v_out / v_mix); diff (nullable): differential
 *                  attention (dim: both maps' columns of a head)
 * b_in (nullable): bias of w_in.  softcap > 0: logits <- softcap tanh(logits / softcap).
 * Sequence b (ids[b]) lives in slot slots[b] (NULL: b) and holds lengths[slot] tokens, which the step advances by one on the
 * device; max_keys >= every lengths[slot] + 1.  Widths with _p, dim, vdim, ff and dp are padded to multiples of 8; d, q_rank,
 * kv_rank and mix_n are the true counts the norms divide by.  logits: (B, ldv).
 * -------------------------------------------------------------------------------------------- */
enum { VY_MIX_LATENT = 0, VY_MIX_DECAY = 1, VY_MIX_WINDOW = 2, VY_MIX_GATED = 3 };
enum { VY_FORM_SANDWICH = 0, VY_FORM_PARALLEL = 1 };
enum { VY_VALUES_OWN = 0, VY_VALUES_FIRST = 1, VY_VALUES_MIX = 2 };
typedef struct vy_hybrid_layer {
  int32_t mixer, heads, dim, vdim, n_in, ff;
  int32_t q_rank, q_rank_p, kv_rank, kv_rank_p;   /* VY_MIX_LATENT */
  int32_t cap, mix_n;                             /* cache rows per slot; VY_MIX_DECAY: width of mix_norm */
  int32_t form, clamped;
  int32_t kv_heads, rope_dims, rope_len, sink;    /* VY_MIX_WINDOW (rope_*: VY_MIX_DECAY too) */
  int32_t keep, gate, values, silu;               /* VY_MIX_WINDOW, the last one VY_MIX_DECAY and VY_MIX_GATED */
  int32_t ring, gate_heads;                       /* VY_MIX_LATENT */
  float scale, limit, alpha, k_scale;
  const float *norm1, *norm1b, *norm2, *norm2b;
  const void *w_in, *b_in, *w_o, *w_gu, *w_up, *w_down;   /* w_gu: packed [gate; up] (VY_FORM_SANDWICH) */
  const float *q_norm, *c_norm;
  const void *w_uq, *w_ukt, *w_uv;
  void* cache; int64_t c_ss, c_sh, c_st;
  float* state; const float *decay_pow, *mix_norm, *f_bias, *f_lower;
  const float* rope;
  const vy_qkv_prep* prep;
  const vy_diff* diff;
  const vy_moe* moe;
} vy_hybrid_layer;
typedef struct vy_hybrid_plan {
  int32_t num_layers, B, d, dp, vocab, dtype, rms, act;
  float eps, embed_scale, softcap;
  const vy_hybrid_layer* layers;                  /* host array [num_layers] */
  const void *embed, *head; const float* final_norm;
  int32_t* err;                                   /* nullable: set when an id is outside the vocabulary */
  void* ws; int64_t ws_bytes;                     /* >= vy_hybrid_ws_bytes(plan) */
} vy_hybrid_plan;
int64_t vy_hybrid_ws_bytes(const vy_hybrid_plan* plan);
int vy_hybrid_decoder_step(const vy_hybrid_plan* plan, const int64_t* ids, const int32_t* slots, int32_t* lengths,
                           int64_t max_keys, void* logits, int64_t ldv, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* VYOM_HIP_H */
