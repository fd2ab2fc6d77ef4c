// Native decode driver (host code) of decoders that mix layer kinds: one call runs a whole single-token step of a batch of
// sequences of different lengths -- embedding, every layer (latent attention over its latent cache or ring, decayed or gated
// linear attention over its fp32 state, or windowed or differential attention over its ring), dense or routed feed-forward behind
// or beside the mixer, final norm and vocabulary product.  See include/vyom_hip.h (vy_hybrid_decoder_step).
#include "vy_common.h"

int vy_residual_norm_ex(float* x, int64_t ldx, const void* y, int64_t ldy, const void* table, int64_t ldt, const int64_t* ids,
                        int64_t V, int32_t* err, float table_scale, const vy_routed_rows* routed, const float* w_post,
                        float eps_post, const float* w_pre, float eps_pre, void* h, int64_t ldh, int64_t M, int64_t N, int64_t NP,
                        int rms, int* advance, const int* slots, int n_adv, int dtype, void* stream);
int vy_residual_route(float* x, int64_t ldx, const void* y, int64_t ldy, const float* w_post, const float* w_pre, float eps, void* h,
                      int64_t ldh, int64_t M, int64_t N, int64_t NP, int rms, const vy_moe* d, int32_t* ids, float* weight, int dtype,
                      void* stream);
int vy_moe_few(const vy_moe* d, const void* h, int64_t ldh, int64_t M, const int32_t* ids, void* rows, int64_t ldr, void* ws,
               int64_t ws_bytes, int dtype, void* stream);
int vy_parallel_decode(const vy_hybrid_plan* p, const vy_hybrid_layer* L, const void* h, void* in, void* ao, void* y, void* erows,
                       int32_t* eids, float* ew, void* moe_ws, int64_t moe_ws_bytes, const int32_t* slots, const int32_t* lengths,
                       int64_t max_keys, void* mix_ws, int64_t mix_ws_bytes, void* stream);
int vy_dec_gemv1_act(const void* x, const void* w, const void* bias, int act, float act_arg, void* y, int N, int K, hipStream_t st);
int vy_rows_linear(const void* x, const void* w, const void* bias, int act, float act_arg, void* y, int64_t ldy, int64_t M, int64_t N,
                   int64_t K, hipStream_t st);
int vy_dec_gemv1_gated(const void* x, const void* wgu, void* y, int I, int K, int act, int prescaled, float eps, hipStream_t st);
int vy_gemv_gated(const void* x, int64_t ldx, const void* w, int64_t ldw, const void* norm_w, float eps, void* y, int64_t ldy,
                  int64_t M, int64_t I, int64_t K, int act, void* stream);

namespace {

int64_t up(int64_t x) { return (x + 255) / 256 * 256; }

struct Sizes { int64_t in, q, cq, ao, o, gu, ff, mix_ws, top, moe_ws, values; };   // widest of each over the layers

Sizes sizes_of(const vy_hybrid_plan* p) {
  Sizes s{};
  auto mx = [](int64_t& a, int64_t b) { if (b > a) a = b; };
  for (int l = 0; l < p->num_layers; ++l) {
    const vy_hybrid_layer& L = p->layers[l];
    mx(s.in, L.n_in);
    const bool parallel = L.form == VY_FORM_PARALLEL;
    mx(s.ao, (int64_t)L.heads * L.vdim + (parallel ? L.ff : 0));
    if (L.mixer == VY_MIX_LATENT) {
      if (L.w_uq) mx(s.q, (int64_t)L.heads * L.dim);
      if (L.w_uq) mx(s.cq, L.q_rank_p);
      mx(s.mix_ws, vy_latent_decode_ws_bytes(p->B, L.heads, L.kv_rank_p));
    } else if (L.mixer == VY_MIX_WINDOW) {
      mx(s.mix_ws, vy_window_decode_ws_bytes(p->B, L.heads, L.kv_heads, L.vdim, L.cap, L.diff != nullptr));
      if (L.values != VY_VALUES_OWN) mx(s.values, (int64_t)L.kv_heads * L.vdim);
    } else {
      mx(s.o, (int64_t)L.heads * L.vdim);
    }
    if (!parallel) {
      mx(s.gu, 2 * (int64_t)L.ff);
      mx(s.ff, L.ff);
    }
    if (L.moe) {
      mx(s.top, L.moe->top);
      mx(s.moe_ws, vy_moe_ws_bytes(L.moe, p->B, p->dtype));
    }
  }
  return s;
}

// y[B, N] = act(x[B, K] W^T + bias); cap: of VY_ACT_SOFTCAP
int product(const vy_hybrid_plan* p, const void* x, const void* w, void* y, int64_t ldy, int64_t N, int64_t K, void* stream,
            const void* bias = nullptr, int act = VY_ACT_NONE, float cap = 0.f) {
  if (p->dtype == VY_BF16 && p->B == 1 && N <= INT32_MAX) {
    const int rc = vy_dec_gemv1_act(x, w, bias, act, cap, y, (int)N, (int)K, (hipStream_t)stream);
    if (rc != VY_ERR_UNSUPPORTED) return rc;
  }
  if (p->dtype == VY_BF16) {
    const int rc = vy_rows_linear(x, w, bias, act, cap, y, ldy, p->B, N, K, (hipStream_t)stream);
    if (rc != VY_ERR_UNSUPPORTED) return rc;
  }
  if (act == VY_ACT_SOFTCAP) return vy_linear_softcap_fwd(x, K, w, K, y, ldy, p->B, N, K, cap, p->dtype, stream);
  return vy_linear_fwd(x, K, w, K, bias, nullptr, 0, y, ldy, nullptr, p->B, N, K, act, p->dtype, stream);
}

// packed [gate | up] rows -> activation rows
int activation(const vy_hybrid_plan* p, const vy_hybrid_layer& L, const void* gu, int64_t ldg, void* act, int64_t lda, void* stream) {
  if (L.clamped) return vy_clamped_act_fwd(gu, ldg, act, lda, p->B, L.ff, L.limit, L.alpha, p->dtype, stream);
  return vy_gated_act_fwd(gu, ldg, act, lda, p->B, L.ff, p->act, p->dtype, stream);
}

int gated(const vy_hybrid_plan* p, const vy_hybrid_layer& L, const void* x, void* gu, void* act, void* stream) {
  if (!L.clamped && p->dtype == VY_BF16 && p->B == 1) {
    const int rc = vy_dec_gemv1_gated(x, L.w_gu, act, L.ff, p->dp, p->act, 0, 0.f, (hipStream_t)stream);
    if (rc != VY_ERR_UNSUPPORTED) return rc;
  }
  if (!L.clamped && p->dtype == VY_BF16 && p->B <= 4)
    return vy_gemv_gated(x, p->dp, L.w_gu, p->dp, nullptr, 0.f, act, L.ff, p->B, L.ff, p->dp, p->act, stream);
  const int rc = product(p, x, L.w_gu, gu, 2 * (int64_t)L.ff, 2 * (int64_t)L.ff, p->dp, stream);
  return rc ? rc : activation(p, L, gu, 2 * (int64_t)L.ff, act, L.ff, stream);
}

}  // namespace

extern "C" int64_t vy_hybrid_ws_bytes(const vy_hybrid_plan* p) {
  if (!p || !p->layers) return -1;
  const Sizes s = sizes_of(p);
  const int64_t e = p->dtype == VY_BF16 ? 2 : 4, B = p->B;
  return up(B * p->dp * 4) + 2 * up(B * p->dp * e) + up(B * s.in * e) + up(B * s.q * e) + up(B * s.cq * e) +
         up(B * s.ao * e) + up(B * s.o * e) + up(B * s.gu * e) + up(B * s.ff * e) + up(s.mix_ws) + up(B * s.top * p->dp * e) +
         3 * up(B * s.top * 4) + up(s.moe_ws) + up(B * s.values * e);
}

extern "C" int vy_hybrid_decoder_step(const vy_hybrid_plan* p, const int64_t* ids, const int32_t* slots, int32_t* lengths,
                                      int64_t max_keys, void* logits, int64_t ldv, void* stream) {
  const char* who = "vy_hybrid_decoder_step";
  if (!p || !p->layers || !p->ws || !ids || !lengths || !logits) VY_FAIL(VY_ERR_ARG, "%s: null plan/input/workspace/output", who);
  if (p->ws_bytes < vy_hybrid_ws_bytes(p)) VY_FAIL(VY_ERR_ARG, "%s: workspace too small", who);
  if (max_keys < 1) VY_FAIL(VY_ERR_ARG, "%s: max_keys %ld", who, (long)max_keys);
  const Sizes s = sizes_of(p);
  const int64_t e = p->dtype == VY_BF16 ? 2 : 4, B = p->B, dp = p->dp;
  char* w = (char*)p->ws;
  auto take = [&](int64_t bytes) { char* r = w; w += up(bytes); return r; };
  float* x = (float*)take(B * dp * 4);
  void* h = take(B * dp * e);
  void* y = take(B * dp * e);
  void* in = take(B * s.in * e);
  void* q = take(B * s.q * e);
  void* cq = take(B * s.cq * e);
  void* ao = take(B * s.ao * e);
  void* o = take(B * s.o * e);
  void* gu = take(B * s.gu * e);
  void* act = take(B * s.ff * e);
  void* mws = take(s.mix_ws);
  void* erows = take(B * s.top * dp * e);
  int32_t* eids = (int32_t*)take(B * s.top * 4);
  int32_t* epos = (int32_t*)take(B * s.top * 4);
  float* ew = (float*)take(B * s.top * 4);
  void* ews = take(s.moe_ws);
  void* values = take(B * s.values * e);
  const vy_hybrid_layer* values_of = nullptr;   // the layer that filled them
  int rc;
  auto norm = [&](const void* yy, const vy_routed_rows* routed, const float* post, const float* pre, bool last) {
    return vy_residual_norm_ex(x, dp, yy, dp, p->embed, dp, yy || routed ? nullptr : ids, p->vocab, p->err, p->embed_scale, routed,
                               post, p->eps, pre, p->eps, h, dp, B, p->d, dp, p->rms, last ? lengths : nullptr, slots,
                               last ? (int)B : 0, p->dtype, stream);
  };
  if ((rc = norm(nullptr, nullptr, nullptr, p->layers[0].norm1, false))) return rc;
  for (int l = 0; l < p->num_layers; ++l) {
    const vy_hybrid_layer& L = p->layers[l];
    const bool last = l + 1 == p->num_layers, parallel = L.form == VY_FORM_PARALLEL;
    const float* next = last ? p->final_norm : p->layers[l + 1].norm1;
    const int64_t nv = (int64_t)L.heads * L.vdim, nk = (int64_t)L.heads * L.dim, na = nv + (parallel ? L.ff : 0);
    if (parallel) {   // windowed attention beside clamped feed-forwards: the pieces of the layer share launches
      rc = vy_parallel_decode(p, &L, h, in, ao, y, erows, eids, ew, ews, s.moe_ws, slots, lengths, max_keys, mws, s.mix_ws, stream);
      if (rc == VY_OK) {
        const vy_routed_rows rows{erows, dp, nullptr, ew, L.moe ? L.moe->top : 0};
        if ((rc = norm(y, L.moe ? &rows : nullptr, L.norm1b, next, last))) return rc;
        continue;
      }
      if (rc != VY_ERR_UNSUPPORTED) return rc;
    }
    if ((rc = product(p, h, L.w_in, in, L.n_in, L.n_in, dp, stream, L.b_in))) return rc;
    if (L.mixer == VY_MIX_LATENT) {
      if (!L.ring && max_keys > L.cap) VY_FAIL(VY_ERR_ARG, "%s: %ld keys exceed the cache capacity %d", who, (long)max_keys, L.cap);
      const int64_t nq = L.w_uq ? L.q_rank_p : nk;   // columns ahead of the key/value latent: the queries' latent, or the queries
      if ((rc = vy_latent_norm(in, L.n_in, L.w_uq ? L.q_norm : nullptr, cq, L.q_rank_p, L.q_rank, (int)nq, L.c_norm, nullptr, 0, L.kv_rank,
                               L.kv_rank_p, L.cache, L.c_ss, L.c_st, L.cap, L.ring, slots, lengths, nullptr, B, 1, p->eps, p->dtype,
                               stream))) return rc;
      if (L.w_uq && (rc = product(p, cq, L.w_uq, q, nk, nk, L.q_rank_p, stream))) return rc;
      const char* gate = L.gate ? (const char*)in + (nq + L.kv_rank_p) * e : nullptr;
      if ((rc = vy_latent_decode(L.w_uq ? q : in, L.w_uq ? nk : L.n_in, L.w_ukt, L.w_uv, L.cache, L.c_ss, L.c_st, slots, lengths, max_keys, ao,
                                 na, gate, L.n_in, L.gate_heads, L.ring ? L.cap : 0, (int)B, L.heads, L.dim, L.vdim, L.kv_rank_p,
                                 L.scale, mws, s.mix_ws, p->dtype, stream)))
        return rc;
    } else if (L.mixer == VY_MIX_WINDOW) {
      const int64_t gk = (int64_t)L.kv_heads * L.dim, gv = (int64_t)L.kv_heads * L.vdim;
      vy_qkv_prep prep{};
      if (L.prep) prep = *L.prep;
      if (L.values == VY_VALUES_FIRST) {
        prep.v_out = values;
        prep.ldo = gv;
        values_of = &L;
      } else if (L.values == VY_VALUES_MIX) {
        const vy_hybrid_layer* F = values_of;
        if (!F || !F->prep || F->kv_heads * F->prep->n_v != L.kv_heads * prep.n_v)
          VY_FAIL(VY_ERR_ARG, "%s: layer %d has no values to mix in", who, l);
        prep.v_mix = values;
        prep.ldm = (int64_t)F->kv_heads * F->vdim;
        prep.m_v = F->prep->n_v;
        prep.m_vp = F->vdim;
      }
      if ((rc = vy_window_decode(in, L.n_in, 0, nk, nk + gk, L.gate ? nk + gk + gv : -1, L.cache, L.c_ss, L.c_sh, L.cap, L.keep, L.rope,
                                 L.rope_dims, L.rope_len, L.prep || L.values != VY_VALUES_OWN ? &prep : nullptr, L.diff, slots, lengths, max_keys, ao, na, B, L.heads, L.kv_heads, L.dim, L.vdim, L.scale,
                                 L.sink, mws, s.mix_ws, p->dtype, stream))) return rc;
    } else if (L.mixer == VY_MIX_GATED) {
      if ((rc = vy_gated_attn(in, L.n_in, 0, nk, 2 * nk, L.state, L.f_bias, L.f_lower, slots, lengths, nullptr, o, nv, B, 1, L.heads, L.dim,
                              L.vdim, L.silu, nullptr, 0, p->dtype, stream))) return rc;
      if ((rc = vy_head_norm_gate(o, nv, L.mix_norm, nullptr, 0, ao, na, B, L.heads, L.mix_n, L.vdim, p->eps, p->dtype, stream))) return rc;
    } else {
      if ((rc = vy_decay_attn(in, L.n_in, 0, nk, 2 * nk, L.state, L.decay_pow, slots, lengths, nullptr, o, nv, B, 1, L.heads, L.dim,
                              L.vdim, L.silu, L.rope, L.rope_dims, L.rope_len, L.k_scale, nullptr, 0, p->dtype, stream))) return rc;
      const char* gate = (const char*)in + (2 * nk + nv) * e;
      if (!L.mix_norm) {
        if ((rc = vy_head_norm_gate(o, nv, nullptr, gate, L.n_in, ao, na, B, L.heads, L.mix_n, L.vdim, p->eps, p->dtype, stream))) return rc;
      } else if ((rc = vy_rmsnorm_gate(o, nv, L.mix_norm, gate, L.n_in, ao, na, B, L.mix_n, nv, p->eps, p->dtype, stream))) return rc;
    }
    vy_routed_rows rows{erows, dp, epos, ew, L.moe ? L.moe->top : 0};
    const vy_routed_rows* routed = L.moe ? &rows : nullptr;
    auto experts = [&]() {
      return L.moe ? vy_moe_fwd(L.moe, h, dp, B, nullptr, 1, erows, dp, eids, epos, ew, ews, s.moe_ws, p->dtype, stream) : VY_OK;
    };
    if (parallel) {
      if (L.ff && (rc = activation(p, L, (const char*)in + (L.n_in - 2 * (int64_t)L.ff) * e, L.n_in, (char*)ao + nv * e, na, stream)))
        return rc;
      if ((rc = experts())) return rc;
      if ((rc = product(p, ao, L.w_o, y, dp, dp, na, stream))) return rc;
      if ((rc = norm(y, routed, L.norm1b, next, last))) return rc;
      continue;
    }
    if ((rc = product(p, ao, L.w_o, y, dp, dp, nv, stream))) return rc;
    if (!L.ff && !L.moe) {
      if ((rc = norm(y, nullptr, L.norm1b, next, last))) return rc;
      continue;
    }
    // few tokens: the choice of experts comes with the residual sum
    bool chosen = false;
    if (L.moe) {
      rc = vy_moe_few(L.moe, nullptr, 0, B, nullptr, nullptr, 0, nullptr, 0, p->dtype, stream);
      if (rc == VY_OK)
        rc = vy_residual_route(x, dp, y, dp, L.norm1b, L.norm2, p->eps, h, dp, B, p->d, dp, p->rms, L.moe, eids, ew, p->dtype, stream);
      if (rc && rc != VY_ERR_UNSUPPORTED) return rc;
      chosen = rc == VY_OK;
    }
    if (!chosen && (rc = norm(y, nullptr, L.norm1b, L.norm2, false))) return rc;
    if (L.ff) {
      if (L.w_up) rc = product(p, h, L.w_up, act, L.ff, L.ff, dp, stream, nullptr, p->act);
      else rc = gated(p, L, h, gu, act, stream);
      if (rc) return rc;
      if ((rc = product(p, act, L.w_down, y, dp, dp, L.ff, stream))) return rc;
    }
    if (chosen) {
      rows.pos = nullptr;
      rc = vy_moe_few(L.moe, h, dp, B, eids, erows, dp, ews, s.moe_ws, p->dtype, stream);
    } else {
      rc = experts();
    }
    if (rc) return rc;
    if ((rc = norm(L.ff ? y : nullptr, routed, L.norm2b, next, last))) return rc;
  }
  return product(p, h, p->head, logits, ldv, p->vocab, dp, stream, nullptr, p->softcap > 0.f ? VY_ACT_SOFTCAP : VY_ACT_NONE, p->softcap);
}
