// Sliding-window attention over a ring of keys and values, for decoders whose queries see only the last `window` tokens.
//
// Memory: per sequence (slot) and key/value head a ring of R rows [key (dim) | value (vdim)], R = keep + the window (or less while
// sequences are shorter): the first `keep` positions stay in their rows, later ones go round the others, so a sequence never
// holds more than its window and its kept tokens.
//
//   vy_window_rows     prefill: rotary positions on the new keys (in place in the packed projection rows) and the last new
//                      rows to the ring
//   vy_qkv_rows        the same for designs that norm their queries and keys (over the whole projection, or over heads or other
//                      groups of columns by themselves), scale their queries by position and mix their values: in place
//   vy_window_context  prefill behind a past: the ring's rows and the new ones as one contiguous context for vy_attn_fwd_ex
//   vy_window_decode   one query token per sequence: rotation of query and key, the new row to the ring, attention over the
//                      ring, sink, output gate.  Every row of the ring that holds a token is inside the window, so decode
//                      needs no mask but the row count -- and no order: softmax does not care where a row lies.  Also
//                      differential attention (vy_diff.hip has its prompts).
#include "vy_window.h"

namespace {

using namespace vy_window;

struct RowsArgs {
  const void* p; int64_t ldp, ok, ov;       // packed rows; key / value columns
  void* ring; int64_t r_ss, r_sh; int R, keep;   // ring rows of dim + vdim elements
  const float2* rope; int half, rope_len;
  const int* slots; const int* start; const int* count;
  int64_t M; int L, hk, dim, vdim, rotate, store;
};

// whether the ring still holds a token once its sequence's n new tokens are in (position first + l)
__device__ __forceinline__ bool stays(int first, int l, int n, int R, int keep) {
  return l < n && (first + l < keep || l + (R - keep) >= n);
}

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
    const bool keep = a.store && stays(first, l, n, a.R, a.keep);
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
    if (keep) VyChunk<T>::store((T*)a.ring + (int64_t)slot * a.r_ss + (int64_t)g * a.r_sh + (int64_t)ring_row(pos, a.R, a.keep) * (a.dim + a.vdim) + c * VEC, v);
  }
}

struct QkvArgs {
  RowsArgs r;
  int64_t oq; int h;
  const float* q_norm; const float* k_norm; int n_q, n_k; float eps, lambda;
  const void* vm; int64_t ldm; int n_v, m_v, m_vp;
  void* vo; int64_t ldvo;
};

// WPR waves per token: sums of squares of its query and key projections, then every chunk once more (from cache) to be scaled,
// rotated, rounded once and written back.  CH chunks per lane are held between the two (more are read again).
template <typename T, int WPR, int CH>
__global__ __launch_bounds__(256) void qkv_rows_kernel(QkvArgs a) {
  constexpr int VEC = VyChunk<T>::VEC, LPR = 64 * WPR;
  __shared__ float red[8];
  const RowsArgs& r = a.r;
  const int t = threadIdx.x % LPR;
  const int64_t m0 = (int64_t)blockIdx.x * (4 / WPR) + threadIdx.x / LPR, row = m0 < r.M ? m0 : r.M - 1;
  T* p = (T*)r.p + row * r.ldp;
  const int b = (int)(row / r.L), l = (int)(row - (int64_t)b * r.L);
  const int slot = r.slots ? r.slots[b] : b;
  const int first = r.start ? r.start[slot] : 0, n = r.count ? r.count[b] : r.L, pos = first + l;
  const int nq = a.h * r.dim / VEC, nk = r.hk * r.dim / VEC, nv = r.hk * r.vdim / VEC;
  float held[CH][VEC];
  float sq = 0.f, sk = 0.f;
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = t + LPR * c;
    if (i < nq + nk) {
      VyChunk<T>::load(i < nq ? p + a.oq + i * VEC : p + r.ok + (i - nq) * VEC, held[c]);
      float s = 0.f;
#pragma unroll
      for (int e = 0; e < VEC; ++e) s = fmaf(held[c][e], held[c][e], s);
      if (i < nq) sq += s;
      else sk += s;
    }
  }
  for (int i = t + LPR * CH; i < nq + nk; i += LPR) {
    float v[VEC], s = 0.f;
    VyChunk<T>::load(i < nq ? p + a.oq + i * VEC : p + r.ok + (i - nq) * VEC, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) s = fmaf(v[e], v[e], s);
    if (i < nq) sq += s;
    else sk += s;
  }
  sq = vy_wave_sum(sq);
  sk = vy_wave_sum(sk);
  if constexpr (WPR == 4) {
    const int wave = threadIdx.x >> 6;
    if ((threadIdx.x & 63) == 0) { red[wave] = sq; red[4 + wave] = sk; }
    __syncthreads();
    sq = red[0] + red[1] + red[2] + red[3];
    sk = red[4] + red[5] + red[6] + red[7];
  }
  if (m0 >= r.M) return;
  const float rq = a.q_norm ? rms_factor(sq, a.n_q, a.eps) : 1.f, rk = a.k_norm ? rms_factor(sk, a.n_k, a.eps) : 1.f;
  const float2* trig = r.rope + (int64_t)(pos < r.rope_len ? pos : r.rope_len - 1) * r.half;   // (clamped: padding rows only)
  const bool keep = r.store && stays(first, l, n, r.R, r.keep);
  T* ring = keep ? (T*)r.ring + (int64_t)slot * r.r_ss + (int64_t)ring_row(pos, r.R, r.keep) * (r.dim + r.vdim) : nullptr;
  auto finish = [&](int i, float (&v)[VEC]) {   // chunk i of [queries | keys]
    const bool key = i >= nq;
    const int col = (key ? i - nq : i) * VEC, g = col / r.dim, d = col - g * r.dim;
    const float* w = key ? a.k_norm : a.q_norm;
    if (w) {
      const float f = key ? rk : rq;
#pragma unroll
      for (int e = 0; e < VEC; e += 4) {
        float w4[4];
        VyChunk<float>::load(w + col + e, w4);
#pragma unroll
        for (int c = 0; c < 4; ++c) v[e + c] *= f * w4[c];
      }
    }
    if (d < 2 * r.half) {
#pragma unroll
      for (int e = 0; e < VEC; e += 2) {
        const int j = (d + e) >> 1;
        if (j < r.half) {
          const float2 cs = trig[j];
          const float x = v[e], y = v[e + 1];
          v[e] = x * cs.x - y * cs.y;
          v[e + 1] = y * cs.x + x * cs.y;
        }
      }
    }
    VyChunk<T>::store(p + (key ? r.ok : a.oq) + col, v);
    if (key && keep) VyChunk<T>::store(ring + (int64_t)g * r.r_sh + d, v);
  };
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = t + LPR * c;
    if (i < nq + nk) finish(i, held[c]);
  }
  for (int i = t + LPR * CH; i < nq + nk; i += LPR) {
    float v[VEC];
    VyChunk<T>::load(i < nq ? p + a.oq + i * VEC : p + r.ok + (i - nq) * VEC, v);
    finish(i, v);
  }
  if (!a.vm && !a.vo && !keep) return;
  for (int i = t; i < nv; i += LPR) {
    const int col = i * VEC, g = col / r.vdim, d = col - g * r.vdim;
    float v[VEC];
    VyChunk<T>::load(p + r.ov + col, v);
    if (a.vo) VyChunk<T>::store((T*)a.vo + row * a.ldvo + col, v);
    if (a.vm) {
      mix_values(v, (const T*)a.vm + row * a.ldm, a.lambda, g, d, r.vdim, a.n_v, a.m_v, a.m_vp);
      VyChunk<T>::store(p + r.ov + col, v);
    }
    if (keep) VyChunk<T>::store(ring + (int64_t)g * r.r_sh + r.dim + d, v);
  }
}

// norms over groups of columns: LPG lanes per unit, a unit being a group of a token's queries or keys, or a head of its values
// (which are only copied to the ring)
template <typename T, int LPG>
__global__ __launch_bounds__(256) void group_rows_kernel(QkvArgs a, int group, int temp_every, float temp_coef) {
  constexpr int VEC = VyChunk<T>::VEC;
  const RowsArgs& r = a.r;
  const int sub = threadIdx.x % LPG;
  const int gq = a.h * r.dim / group, gk = r.hk * r.dim / group, per_row = gq + gk + (r.store ? r.hk : 0);
  const int64_t units = r.M * per_row, u0 = (int64_t)blockIdx.x * (256 / LPG) + threadIdx.x / LPG, u = u0 < units ? u0 : units - 1;
  const int64_t row = u / per_row;
  const int x = (int)(u - row * per_row);
  const int b = (int)(row / r.L), l = (int)(row - (int64_t)b * r.L);
  const int slot = r.slots ? r.slots[b] : b;
  const int first = r.start ? r.start[slot] : 0, n = r.count ? r.count[b] : r.L, pos = first + l;
  const bool keep = r.store && stays(first, l, n, r.R, r.keep);
  T* p = (T*)r.p + row * r.ldp;
  T* ring = keep ? (T*)r.ring + (int64_t)slot * r.r_ss + (int64_t)ring_row(pos, r.R, r.keep) * (r.dim + r.vdim) : nullptr;
  const bool value = x >= gq + gk, key = !value && x >= gq;
  const int col = key ? (x - gq) * group : x * group;              // of the group, in its projection
  T* src = value ? p + r.ov + (int64_t)(x - gq - gk) * r.vdim : p + (key ? r.ok : a.oq) + col;
  const int width = value ? r.vdim : group;
  float v[VEC], s = 0.f;
  for (int c = sub * VEC; c < width; c += LPG * VEC) {
    VyChunk<T>::load(src + c, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) s = fmaf(v[e], v[e], s);
  }
#pragma unroll
  for (int o = LPG / 2; o > 0; o >>= 1) s += __shfl_xor(s, o, 64);
  if (u0 >= units || (value && !keep)) return;
  const float f = value ? 1.f : rms_factor(s, key ? a.n_k : a.n_q, a.eps) * (key ? 1.f : query_temperature(pos, temp_every, temp_coef));
  const float* w = key ? a.k_norm : a.q_norm;
  const float2* trig = r.rope + (int64_t)(pos < r.rope_len ? pos : r.rope_len - 1) * r.half;   // (clamped: padding rows only)
  const int head = value ? x - gq - gk : col / r.dim, d0 = value ? r.dim : col - head * r.dim;
  for (int c = sub * VEC; c < width; c += LPG * VEC) {
    if (LPG * VEC < width) VyChunk<T>::load(src + c, v);           // (several passes: read again, from cache)
    if (!value) {
      if (w) {
#pragma unroll
        for (int e = 0; e < VEC; e += 4) {
          float w4[4];
          VyChunk<float>::load(w + col + c + e, w4);
#pragma unroll
          for (int i = 0; i < 4; ++i) v[e + i] *= f * w4[i];
        }
      }
#pragma unroll
      for (int e = 0; e < VEC; e += 2) {
        const int j = (d0 + c + e) >> 1;
        if (j < r.half) {
          const float2 cs = trig[j];
          const float y = v[e], z = v[e + 1];
          v[e] = y * cs.x - z * cs.y;
          v[e + 1] = z * cs.x + y * cs.y;
        }
      }
      VyChunk<T>::store(src + c, v);
    }
    if (keep && (key || value)) VyChunk<T>::store(ring + (int64_t)head * r.r_sh + d0 + c, v);
  }
}

template <typename T>
void group_rows_go(const QkvArgs& a, int group, int temp_every, float temp_coef, hipStream_t st) {
  const int nch = group / VyChunk<T>::VEC;   // (wider values take more passes)
  const int64_t units = a.r.M * ((int64_t)(a.h + a.r.hk) * a.r.dim / group + (a.r.store ? a.r.hk : 0));
#define GR_GO(LPG) hipLaunchKernelGGL((group_rows_kernel<T, LPG>), dim3((unsigned)vy_cdiv(units, 256 / LPG)), dim3(256), 0, st, a, group, temp_every, temp_coef)
  if (nch <= 4) GR_GO(4);
  else if (nch <= 8) GR_GO(8);
  else if (nch <= 16) GR_GO(16);
  else if (nch <= 32) GR_GO(32);
  else GR_GO(64);
#undef GR_GO
}

struct ContextArgs {
  const void* p; int64_t ldp, ok, ov;
  const void* ring; int64_t r_ss, r_sh; int R, keep;
  void* ctx; int S, past;                   // ctx [B][hk][S][dim + vdim]; past rows of the ring at most
  const int* slots; const int* start;
  int B, L, hk, dim, vdim;
};

// row s of sequence b, k = min(start, past): the first k rows come from the ring, positions 0 .. keep - 1, then the k - keep last;
// the new tokens follow
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
      VyChunk<T>::load((const T*)a.ring + (int64_t)slot * a.r_ss + (int64_t)g * a.r_sh + (int64_t)ring_row(s < a.keep ? s : first - k + s, a.R, a.keep) * W + c, v);
    } else if (s - k < a.L) {
      const T* row = (const T*)a.p + ((int64_t)b * a.L + s - k) * a.ldp;
      VyChunk<T>::load(c < a.dim ? row + a.ok + (int64_t)g * a.dim + c : row + a.ov + (int64_t)g * a.vdim + (c - a.dim), v);
    }
    VyChunk<T>::store((T*)a.ctx + (((int64_t)b * a.hk + g) * a.S + s) * W + c, v);
  }
}

// ---- decode ---------------------------------------------------------------------------------
template <int DHP, int DVP, int MAPS>
__global__ __launch_bounds__(256) void window_decode_kernel(DecodeArgs a) {
  __shared__ __attribute__((aligned(16))) char smem[WindowDecode<DHP, DVP, MAPS>::LDS];
  WindowDecode<DHP, DVP, MAPS>::run(a, smem, blockIdx.x, blockIdx.y, blockIdx.z);
}

__global__ __launch_bounds__(256) void window_finish_kernel(DecodeArgs a) {
  __shared__ __attribute__((aligned(16))) float red[FINISH_LDS / 4];
  window_finish(a, red, blockIdx.x, blockIdx.y);
}

__global__ __launch_bounds__(256) void window_finish_diff_kernel(DecodeArgs a) {
  __shared__ __attribute__((aligned(16))) float red[FINISH_DIFF_LDS / 4];
  window_finish_diff(a, red, blockIdx.x, blockIdx.y);
}

template <int DHP, int MAPS = 1>
void decode_go(const DecodeArgs& a, dim3 grid, hipStream_t st) {
  const dim3 block(256);
  if (a.vdim <= 64) hipLaunchKernelGGL((window_decode_kernel<DHP, 64, MAPS>), grid, block, 0, st, a);
  else if (a.vdim <= 128) hipLaunchKernelGGL((window_decode_kernel<DHP, 128, MAPS>), grid, block, 0, st, a);
  else hipLaunchKernelGGL((window_decode_kernel<DHP, 256, MAPS>), grid, block, 0, st, a);
}

int check_ring(const char* who, const void* ring, int64_t r_ss, int64_t r_sh, int32_t R, int32_t keep, int32_t hk, int32_t dim,
               int32_t vdim, int vec) {
  if (!ring || R < 1 || hk < 1 || dim < 1 || vdim < 0) VY_FAIL(VY_ERR_ARG, "%s: bad ring", who);
  if (keep < 0 || keep >= R) VY_FAIL(VY_ERR_ARG, "%s: %d kept of %d rows", who, keep, R);
  if (dim % vec || vdim % vec || r_ss % vec || r_sh % vec) VY_FAIL(VY_ERR_ARG, "%s: widths and strides must be multiples of %d", who, vec);
  if (r_sh < (int64_t)R * (dim + vdim) || r_ss < hk * r_sh) VY_FAIL(VY_ERR_ARG, "%s: ring strides do not hold %d rows", who, R);
  return VY_OK;
}

int check_prep(const char* who, const vy_qkv_prep* q, int32_t h, int32_t hk, int32_t dim, int32_t vdim, int vec) {
  if (!q) return VY_OK;
  if (q->group) {
    if (q->group < 1 || q->group % vec || dim % q->group || !q->q_norm || !q->k_norm || q->n_q < 1 || q->n_q > q->group || q->n_k != q->n_q ||
        q->temp_every < 0 || q->v_mix || q->v_out)
      VY_FAIL(VY_ERR_ARG, "%s: norms over %d of %d columns of heads of %d", who, q->n_q, q->group, dim);
    return VY_OK;
  }
  if (q->temp_every) VY_FAIL(VY_ERR_ARG, "%s: a temperature without norms over groups", who);
  if (!q->q_norm != !q->k_norm || (q->q_norm && (q->n_q < 1 || q->n_k < 1 || q->n_q > h * dim || q->n_k > hk * dim)))
    VY_FAIL(VY_ERR_ARG, "%s: bad query / key norms", who);
  const int m_v = q->m_v ? q->m_v : q->n_v, m_vp = q->m_v ? q->m_vp : vdim;
  if (q->v_mix && (q->n_v < 1 || q->n_v > vdim || m_v < 1 || m_v > m_vp || hk * q->n_v % m_v || (m_v == q->n_v && m_vp != vdim) ||
                   q->ldm < (int64_t)(hk * q->n_v / m_v) * m_vp))
    VY_FAIL(VY_ERR_ARG, "%s: bad value rows", who);
  if ((q->v_mix && q->ldm % vec) || (q->v_out && (q->ldo % vec || q->ldo < (int64_t)hk * vdim)))
    VY_FAIL(VY_ERR_ARG, "%s: bad value rows", who);
  return VY_OK;
}

int check_rope(const char* who, const float* rope, int32_t rope_dims, int32_t rope_len, int32_t dim) {
  if (rope_dims < 0 || rope_dims % 2 || rope_dims > dim || (rope_dims && (!rope || rope_len < 1)))
    VY_FAIL(VY_ERR_ARG, "%s: rotary table of %d columns, %d positions for heads of %d", who, rope_dims, rope_len, dim);
  return VY_OK;
}

}  // namespace

extern "C" int vy_window_rows(void* p, int64_t ldp, int64_t ok, int64_t ov, void* ring, int64_t r_ss, int64_t r_sh, int32_t R,
                              int32_t keep, const float* rope, int32_t rope_dims, int32_t rope_len, int rotate, int store,
                              const int32_t* slots, const int32_t* start, const int32_t* count, int64_t B, int64_t L, int32_t hk,
                              int32_t dim, int32_t vdim, int dtype, void* stream) {
  const char* who = "vy_window_rows";
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!p || B <= 0 || L <= 0 || hk <= 0 || dim <= 0 || vdim < 0 || dim % vec || vdim % vec || ldp % vec || ok % vec || ov % vec)
    VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (store) {
    if (!start) VY_FAIL(VY_ERR_ARG, "%s: ring without start positions", who);
    if (int rc = check_ring(who, ring, r_ss, r_sh, R, keep, hk, dim, vdim, vec)) return rc;
  }
  if (rotate)
    if (int rc = check_rope(who, rope, rope_dims, rope_len, dim)) return rc;
  if (!rotate && !store) return VY_OK;
  RowsArgs a{p, ldp, ok, ov, ring, r_ss, r_sh, store ? R : 1, store ? keep : 0, (const float2*)rope, rope_dims / 2, rope_len, slots, start, count,
             B * L, (int)L, hk, dim, vdim, rotate && rope_dims > 0, store};
  const int64_t want = vy_cdiv(a.M * hk * ((dim + vdim) / vec), 256);
  const dim3 grid((unsigned)(want < 16384 ? want : 16384)), block(256);
  if (dtype == VY_BF16) hipLaunchKernelGGL((window_rows_kernel<bf16>), grid, block, 0, (hipStream_t)stream, a);
  else hipLaunchKernelGGL((window_rows_kernel<float>), grid, block, 0, (hipStream_t)stream, a);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}

extern "C" int vy_qkv_rows(void* p, int64_t ldp, int64_t oq, int64_t ok, int64_t ov, const vy_qkv_prep* prep, void* ring, int64_t r_ss,
                           int64_t r_sh, int32_t R, int32_t keep, const float* rope, int32_t rope_dims, int32_t rope_len, int store,
                           const int32_t* slots, const int32_t* start, const int32_t* count, int64_t B, int64_t L, int32_t h,
                           int32_t hk, int32_t dim, int32_t vdim, int dtype, void* stream) {
  const char* who = "vy_qkv_rows";
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!p || !prep || B <= 0 || L <= 0 || h <= 0 || hk <= 0 || dim <= 0 || vdim <= 0 || dim % vec || vdim % vec || ldp % vec || oq % vec ||
      ok % vec || ov % vec || L > INT32_MAX || (int64_t)(h + hk) * dim > 1 << 24)
    VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (int rc = check_prep(who, prep, h, hk, dim, vdim, vec)) return rc;
  if (int rc = check_rope(who, rope, rope_dims, rope_len, dim)) return rc;
  if (store) {
    if (!start) VY_FAIL(VY_ERR_ARG, "%s: ring without start positions", who);
    if (int rc = check_ring(who, ring, r_ss, r_sh, R, keep, hk, dim, vdim, vec)) return rc;
  }
  QkvArgs a{};
  a.r = RowsArgs{p, ldp, ok, ov, ring, r_ss, r_sh, store ? R : 1, store ? keep : 0, (const float2*)rope, rope_dims / 2,
                 rope_len > 0 ? rope_len : 1, slots, start, count, B * L, (int)L, hk, dim, vdim, rope_dims > 0, store};
  a.oq = oq; a.h = h; a.q_norm = prep->q_norm; a.k_norm = prep->k_norm; a.n_q = prep->n_q; a.n_k = prep->n_k;
  a.eps = prep->eps; a.lambda = prep->lambda; a.vm = prep->v_mix; a.ldm = prep->ldm;
  a.n_v = prep->n_v; a.m_v = prep->m_v ? prep->m_v : prep->n_v; a.m_vp = prep->m_v ? prep->m_vp : vdim; a.vo = prep->v_out; a.ldvo = prep->ldo;
  hipStream_t st = (hipStream_t)stream;
  const int chunks = (h + hk) * dim / vec;
  if (prep->group) {
    if (a.r.M * ((int64_t)(h + hk) * dim / prep->group + hk) > INT32_MAX) VY_FAIL(VY_ERR_UNSUPPORTED, "%s: %ld rows", who, (long)a.r.M);
    if (dtype == VY_BF16) group_rows_go<bf16>(a, prep->group, prep->temp_every, prep->temp_coef, st);
    else group_rows_go<float>(a, prep->group, prep->temp_every, prep->temp_coef, st);
    VY_CHECK_LAUNCH(who);
    return VY_OK;
  }
  // narrow rows: a wave each
  const bool narrow = chunks <= 64 * 8 && B * L >= 1024;
  const dim3 grid((unsigned)(narrow ? vy_cdiv(B * L, 4) : B * L)), block(256);
#define QKV_GO(T)                                                                              \
  do {                                                                                         \
    if (narrow && chunks <= 256) hipLaunchKernelGGL((qkv_rows_kernel<T, 1, 4>), grid, block, 0, st, a); \
    else if (narrow) hipLaunchKernelGGL((qkv_rows_kernel<T, 1, 8>), grid, block, 0, st, a);    \
    else if (chunks <= 512) hipLaunchKernelGGL((qkv_rows_kernel<T, 4, 2>), grid, block, 0, st, a); \
    else hipLaunchKernelGGL((qkv_rows_kernel<T, 4, 4>), grid, block, 0, st, a);                \
  } while (0)
  if (dtype == VY_BF16) QKV_GO(bf16);
  else QKV_GO(float);
#undef QKV_GO
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}

extern "C" int vy_window_context(const void* p, int64_t ldp, int64_t ok, int64_t ov, const void* ring, int64_t r_ss, int64_t r_sh,
                                 int32_t R, int32_t keep, void* ctx, int32_t S, int32_t past, const int32_t* slots, const int32_t* start,
                                 int64_t B, int64_t L, int32_t hk, int32_t dim, int32_t vdim, int dtype, void* stream) {
  const char* who = "vy_window_context";
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!p || !ctx || !start || B <= 0 || L <= 0 || S < L || past < 0 || past > R || ldp % vec || ok % vec || ov % vec)
    VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (int rc = check_ring(who, ring, r_ss, r_sh, R, keep, hk, dim, vdim, vec)) return rc;
  ContextArgs a{p, ldp, ok, ov, ring, r_ss, r_sh, R, keep, ctx, S, past, slots, start, (int)B, (int)L, hk, dim, vdim};
  const int64_t want = vy_cdiv(B * hk * S * ((dim + vdim) / vec), 256);
  const dim3 grid((unsigned)(want < 16384 ? want : 16384)), block(256);
  if (dtype == VY_BF16) hipLaunchKernelGGL((window_context_kernel<bf16>), grid, block, 0, (hipStream_t)stream, a);
  else hipLaunchKernelGGL((window_context_kernel<float>), grid, block, 0, (hipStream_t)stream, a);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}

extern "C" int64_t vy_window_decode_ws_bytes(int32_t B, int32_t h, int32_t hk, int32_t vdim, int32_t R, int diff) {
  if (B < 1 || h < 1 || hk < 1 || vdim < 1 || R < 1) return 0;
  const int ns = slices_of((int64_t)B * hk * ((h / hk + 15) / 16), R);
  return ns == 1 && !diff ? 0 : (int64_t)B * h * (diff ? 2 : 1) * ns * (vdim + 2) * 4 + 256;
}

extern "C" int vy_window_decode(void* p, int64_t ldp, int64_t oq, int64_t ok, int64_t ov, int64_t og, void* ring, int64_t r_ss,
                                int64_t r_sh, int32_t R, int32_t keep, const float* rope, int32_t rope_dims, int32_t rope_len,
                                const vy_qkv_prep* prep, const vy_diff* diff, const int32_t* slots, const int32_t* start, int64_t max_keys, void* out,
                                int64_t ldo, int64_t B,
                                int32_t h, int32_t hk, int32_t dim, int32_t vdim, float scale, int32_t sink, void* ws,
                                int64_t ws_bytes, int dtype, void* stream) {
  const char* who = "vy_window_decode";
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!p || !out || !start || B <= 0 || h <= 0 || hk <= 0 || h % hk || max_keys < 1 || !(scale > 0.f))
    VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (ldp % vec || oq % vec || ok % vec || ov % vec || ldo % vec || (og >= 0 && og % vec))
    VY_FAIL(VY_ERR_ARG, "%s: columns and strides must be multiples of %d", who, vec);
  if (int rc = check_ring(who, ring, r_ss, r_sh, R, keep, hk, dim, vdim, vec)) return rc;
  if (int rc = check_prep(who, prep, h, hk, dim, vdim, vec)) return rc;
  if (int rc = check_rope(who, rope, rope_dims, rope_len, dim)) return rc;
  if (rope_dims && max_keys > rope_len) VY_FAIL(VY_ERR_ARG, "%s: %ld positions, rotary table of %d", who, (long)max_keys, rope_len);
  if (diff && (dim % (2 * vec) || sink || og >= 0 || rope_dims || keep || max_keys > R || diff->n_v < 1 || diff->n_v > vdim || vdim < 1 ||
               !prep || (prep->group && prep->group != dim / 2)))
    VY_FAIL(VY_ERR_ARG, "%s: bad differential attention", who);
  hipStream_t st = (hipStream_t)stream;
  const int map_dim = diff ? dim / 2 : dim;
  if (diff && (dtype == VY_F32 || map_dim > 256 || vdim > 256)) {
    if (int rc = vy_qkv_rows(p, ldp, oq, ok, ov, prep, ring, r_ss, r_sh, R, keep, rope, rope_dims, rope_len, 1, slots, start, nullptr, B, 1, h,
                             hk, dim, vdim, dtype, stream)) return rc;
    return vy_diff_attn_fwd((const char*)p + oq * (dtype == VY_BF16 ? 2 : 4), ldp, ring, r_ss, r_sh, R, diff, slots, start, nullptr, out, ldo,
                            B, 1, h, hk, dim, vdim, scale, dtype, stream);
  }
  if (dtype == VY_F32 || map_dim > 256 || vdim > 256) {
    // row-wise kernel over the ring: the new row goes in first
    int rc;
    if (prep) rc = vy_qkv_rows(p, ldp, oq, ok, ov, prep, ring, r_ss, r_sh, R, keep, rope, rope_dims, rope_len, 1, slots, start, nullptr, B, 1,
                               h, hk, dim, vdim, dtype, stream);
    else rc = vy_window_rows(p, ldp, ok, ov, ring, r_ss, r_sh, R, keep, rope, rope_dims, rope_len, 1, 1, slots, start, nullptr, B, 1,
                             hk, dim, vdim, dtype, stream);
    if (rc) return rc;
    const int64_t e = dtype == VY_BF16 ? 2 : 4;
    const vy_attn_window win{0, sink, 1, INT32_MAX, prep ? nullptr : rope, prep ? 0 : rope_dims, rope_len, 0, 0};   // (prep: rotated already)
    const char* gate = og >= 0 ? (const char*)p + og * e : nullptr;
    return vy_attn_fwd_ex((const char*)p + oq * e, ldp, dim, ldp, ring, r_ss, r_sh, dim + vdim, (const char*)ring + (int64_t)dim * e,
                          r_ss, r_sh, dim + vdim, out, ldo, ldo, gate, ldp, ldp, start, slots, B, h, hk, 1, R, dim, vdim, scale,
                          &win, dtype, stream);
  }
  DecodeArgs a{};
  a.p = (const bf16*)p; a.ldp = ldp; a.oq = oq; a.ok = ok; a.ov = ov; a.og = og;
  a.ring = (bf16*)ring; a.r_ss = r_ss; a.r_sh = r_sh; a.R = R; a.keep = keep;
  if (prep) {
    a.q_norm = prep->q_norm; a.k_norm = prep->k_norm; a.n_q = prep->n_q; a.n_k = prep->n_k; a.eps = prep->eps; a.lambda = prep->lambda;
    a.group = prep->group; a.temp_every = prep->temp_every; a.temp_coef = prep->temp_coef;
    a.vm = (const bf16*)prep->v_mix; a.ldm = prep->ldm;
    a.n_v = prep->n_v; a.m_v = prep->m_v ? prep->m_v : prep->n_v; a.m_vp = prep->m_v ? prep->m_vp : vdim;
    a.vo = (bf16*)prep->v_out; a.ldvo = prep->ldo;
  }
  a.rope = (const float2*)rope; a.half = rope_dims / 2; a.rope_len = rope_len > 0 ? rope_len : 1;
  a.slots = slots; a.start = start; a.out = (bf16*)out; a.ldo = ldo;
  a.h = h; a.hk = hk; a.dim = map_dim; a.vdim = vdim; a.scale = scale; a.sink = sink;
  if (diff) { a.lambda2 = diff->lambda; a.out_scale = diff->out_scale; a.eps_out = diff->eps; a.n_v = diff->n_v; }
  a.passes = (h / hk + 15) / 16;
  const int64_t rows = max_keys < R ? max_keys : R;
  a.ns = slices_of(B * hk * a.passes, rows);
  if (a.ns > 1 || diff) {
    const int64_t parts = B * h * (diff ? 2 : 1) * a.ns, need = parts * ((int64_t)vdim + 2) * 4;
    if (!ws || ws_bytes < need || (uintptr_t)ws % 16) VY_FAIL(VY_ERR_ARG, "%s: workspace too small or unaligned", who);
    a.part_o = (float*)ws;
    a.part_ml = a.part_o + parts * vdim;
  }
  const dim3 grid((unsigned)a.ns, (unsigned)(hk * a.passes), (unsigned)B);
  if (diff) {
    if (map_dim <= 64) decode_go<64, 2>(a, grid, st);
    else if (map_dim <= 128) decode_go<128, 2>(a, grid, st);
    else decode_go<256, 2>(a, grid, st);
    hipLaunchKernelGGL(window_finish_diff_kernel, dim3((unsigned)h, (unsigned)B), dim3(256), 0, st, a);
    VY_CHECK_LAUNCH(who);
    return VY_OK;
  }
  if (dim <= 64) decode_go<64>(a, grid, st);
  else if (dim <= 128) decode_go<128>(a, grid, st);
  else decode_go<256>(a, grid, st);
  if (a.ns > 1) hipLaunchKernelGGL(window_finish_kernel, dim3((unsigned)h, (unsigned)B), dim3(256), 0, st, a);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}
