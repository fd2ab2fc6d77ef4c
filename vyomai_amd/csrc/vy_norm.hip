// Norms around an fp32 residual stream, for decoders that keep the residual sum in 32-bit and put a norm before and
// (optionally) after every sublayer.  Weights are fp32; a row may be padded (N columns used of NP, the padding zero in
// every operand and kept zero in every result), so widths that are not a multiple of 8 run on the same kernels.
//
//   vy_residual_norm   x += norm(y) * w_post  (or x = table[ids], or x += y) and h = norm(x) * w_pre, one pass: the
//                      end of one sublayer and the beginning of the next.  vy_residual_norm_routed: y also collects the
//                      weighted rows of a token's experts
//   vy_latent_norm     the two RMS norms behind a packed [query latent | key/value latent | ...] projection; the
//                      key/value latent also goes to its cache rows
//   vy_rmsnorm_gate    RMSNorm(x) * w * sigmoid(gate)
//   vy_head_norm_gate  x / rms(x) * w * silu(gate), every head by itself
#include "vy_common.h"

namespace {

// reduction over the TPR threads of a row: one wave, or the four waves of the workgroup
template <int TPR>
__device__ __forceinline__ float row_sum(float v, float* red, int slot) {
  v = vy_wave_sum(v);
  if constexpr (TPR == 64) return v;
  else {
    const int wave = threadIdx.x >> 6;
    if ((threadIdx.x & 63) == 0) red[slot * 4 + wave] = v;
    __syncthreads();
    return red[slot * 4] + red[slot * 4 + 1] + red[slot * 4 + 2] + red[slot * 4 + 3];
  }
}
__device__ __forceinline__ float rsqrt_refined(float ms) {
  const float r = rsqrtf(ms);
  return r * (1.5f - 0.5f * ms * r * r);
}

template <typename T> __device__ __forceinline__ void load4(const T* p, float (&v)[4]);
template <> __device__ __forceinline__ void load4<float>(const float* p, float (&v)[4]) {
  const f32x4 t = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = t[e];
}
template <> __device__ __forceinline__ void load4<bf16>(const bf16* p, float (&v)[4]) {
  const bf16x4 t = *reinterpret_cast<const bf16x4*>(p);
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = (float)t[e];
}
template <typename T> __device__ __forceinline__ void store4(T* p, const float (&v)[4]);
template <> __device__ __forceinline__ void store4<float>(float* p, const float (&v)[4]) {
  *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
}
template <> __device__ __forceinline__ void store4<bf16>(bf16* p, const float (&v)[4]) {
  bf16x4 t;
#pragma unroll
  for (int e = 0; e < 4; ++e) t[e] = (bf16)v[e];
  *reinterpret_cast<bf16x4*>(p) = t;
}

struct ResNormArgs {
  float* x; int64_t ldx;
  const void* y; int64_t ldy;
  const void* table; int64_t ldt; const int64_t* ids; int64_t V; int* err;
  const float* w_post; const float* w_pre;
  void* h; int64_t ldh;
  int64_t M; int N, NP; float eps_post, eps_pre;
  int* advance; const int* slots; int n_adv;   // decode: advance[slots[i]] += 1 once per step (workgroup 0)
  float table_scale;                           // x = table_scale * table[ids]
  const void* er; int64_t lder; const int* epos; const float* ew; int top;   // routed rows: y += sum_k ew[row][k] er[epos[row][k]]
};

// statistics of v (CH quads per thread) over the row's first N columns, then v <- (v - mean) * rstd (RMS: mean = 0)
template <int TPR, int CH, bool RMS>
__device__ __forceinline__ void row_stats(const float (&v)[CH][4], int t, int N, int NP, float eps, float* red, int slot,
                                          float& mean, float& rstd) {
  mean = 0.f;
  if constexpr (!RMS) {
    float s = 0.f;
#pragma unroll
    for (int c = 0; c < CH; ++c)
#pragma unroll
      for (int e = 0; e < 4; ++e) s += v[c][e];
    mean = row_sum<TPR>(s, red, slot) / (float)N;
  }
  float q = 0.f;
#pragma unroll
  for (int c = 0; c < CH; ++c)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int col = (t + TPR * c) * 4 + e;
      const float dlt = col < N ? v[c][e] - mean : 0.f;
      q += dlt * dlt;
    }
  rstd = rsqrt_refined(row_sum<TPR>(q, red, slot + 1) / (float)N + eps);
}

template <typename T, int TPR, int CH, bool RMS, bool ROUTED>
__global__ __launch_bounds__(256) void residual_norm_kernel(ResNormArgs p) {
  __shared__ float red[16];
  const int t = TPR == 64 ? threadIdx.x & 63 : threadIdx.x;
  const int64_t row = TPR == 64 ? (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6) : (int64_t)blockIdx.x;
  if (p.advance && blockIdx.x == 0)
    for (int i = threadIdx.x; i < p.n_adv; i += 256) p.advance[p.slots ? p.slots[i] : i] += 1;
  if (row >= p.M) return;   // (whole waves; TPR = 256 has one row per workgroup)
  float x[CH][4], y[CH][4];
  float* xr = p.x + row * p.ldx;
  const T* src = (const T*)p.y + row * p.ldy;
  bool bad = false;
  if (p.ids) {
    const int64_t id = p.ids[row];
    bad = id < 0 || id >= p.V;
    if (bad && p.err && t == 0) *p.err = 1;
    src = (const T*)p.table + (bad ? 0 : id) * p.ldt;
  }
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int col = (t + TPR * c) * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) { x[c][e] = 0.f; y[c][e] = 0.f; }
    if (col < p.NP) {
      if (p.ids || p.y) load4<T>(src + col, y[c]);
      if (!p.ids) load4<float>(xr + col, x[c]);
    }
  }
  if (p.ids) {
#pragma unroll
    for (int c = 0; c < CH; ++c)
#pragma unroll
      for (int e = 0; e < 4; ++e) y[c][e] *= p.table_scale;
  }
  if constexpr (ROUTED) {
#pragma unroll 4
    for (int k = 0; k < p.top; ++k) {
      const int er = p.epos ? p.epos[row * p.top + k] : (int)(row * p.top + k);
      const float w = er >= 0 ? p.ew[row * p.top + k] : 0.f;
      const T* src_e = (const T*)p.er + (int64_t)(er >= 0 ? er : 0) * p.lder;
#pragma unroll
      for (int c = 0; c < CH; ++c) {
        const int col = (t + TPR * c) * 4;
        if (col < p.NP && er >= 0) {
          float v[4];
          load4<T>(src_e + col, v);
#pragma unroll
          for (int e = 0; e < 4; ++e) y[c][e] = fmaf(w, v[e], y[c][e]);
        }
      }
    }
  }
  if (ROUTED || p.ids || p.y) {
    float mean = 0.f, rstd = 1.f;
    const bool post = !p.ids && p.w_post;
    if (post) row_stats<TPR, CH, RMS>(y, t, p.N, p.NP, p.eps_post, red, 0, mean, rstd);
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      const int col = (t + TPR * c) * 4;
      if (col < p.NP) {
        if (post) {
          float w[4];
          load4<float>(p.w_post + col, w);
#pragma unroll
          for (int e = 0; e < 4; ++e) x[c][e] += (y[c][e] - mean) * rstd * w[e];
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e) x[c][e] += bad ? 0.f : y[c][e];
        }
        store4<float>(xr + col, x[c]);
      }
    }
  }
  if (p.h && !p.w_pre) {   // no norm: the stream itself
    T* hr = (T*)p.h + row * p.ldh;
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      const int col = (t + TPR * c) * 4;
      if (col < p.NP) store4<T>(hr + col, x[c]);
    }
  } else if (p.h) {
    float mean, rstd;
    row_stats<TPR, CH, RMS>(x, t, p.N, p.NP, p.eps_pre, red, 2, mean, rstd);
    T* hr = (T*)p.h + row * p.ldh;
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      const int col = (t + TPR * c) * 4;
      if (col < p.NP) {
        float w[4], o[4];
        load4<float>(p.w_pre + col, w);
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = (x[c][e] - mean) * rstd * w[e];   // w = 0 in the padding
        store4<T>(hr + col, o);
      }
    }
  }
}

template <typename T, bool RMS, bool ROUTED>
int residual_norm_go(const ResNormArgs& a, hipStream_t st) {
  const dim3 block(256);
#define RN_GO(TPR, CH) hipLaunchKernelGGL((residual_norm_kernel<T, TPR, CH, RMS, ROUTED>), grid, block, 0, st, a)
  // wide enough batches keep every CU busy with a wave per row; a decode step gives each row a workgroup
  if (a.M >= 1024 && a.NP <= 2048) {
    const dim3 grid((unsigned)vy_cdiv(a.M, 4));
    if (a.NP <= 512) RN_GO(64, 2);
    else if (a.NP <= 1024) RN_GO(64, 4);
    else RN_GO(64, 8);
    return 0;
  }
  const dim3 grid((unsigned)a.M);
  if (a.NP <= 1024) RN_GO(256, 1);
  else if (a.NP <= 2048) RN_GO(256, 2);
  else if (a.NP <= 4096) RN_GO(256, 4);
  else if (a.NP <= 8192) RN_GO(256, 8);
  else if (a.NP <= 16384) RN_GO(256, 16);
  else return 1;
#undef RN_GO
  return 0;
}

template <typename T>
int residual_norm_any(const ResNormArgs& a, int rms, hipStream_t st) {
  if (a.er) return rms ? residual_norm_go<T, true, true>(a, st) : residual_norm_go<T, false, true>(a, st);
  return rms ? residual_norm_go<T, true, false>(a, st) : residual_norm_go<T, false, false>(a, st);
}

struct LatentNormArgs {
  const void* p; int64_t ldp;
  const float* w_q; void* q_out; int64_t ldq; int nq, npq;        // columns [0, npq), nq of them used (w_q NULL: no latent)
  const float* w_c; void* c_out; int64_t ldc; int nc, npc;        // columns [npq, npq + npc)
  void* cache; int64_t c_ss, c_st; int cap, ring;                 // cache rows: strides per slot and per token
  const int* slots; const int* start; const int* count;
  int64_t M; int L; float eps;
};

// one wave per (row, latent)
template <typename T, int CH>
__global__ __launch_bounds__(256) void latent_norm_kernel(LatentNormArgs a) {
  constexpr int VEC = VyChunk<T>::VEC;
  const int lane = threadIdx.x & 63;
  const int64_t u = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const bool both = a.w_q != nullptr;
  if (u >= (both ? 2 * a.M : a.M)) return;
  const bool kv = !both || (u & 1);
  const int64_t row = both ? u >> 1 : u;
  const int n = kv ? a.nc : a.nq, np = kv ? a.npc : a.npq;
  const T* src = (const T*)a.p + row * a.ldp + (kv ? a.npq : 0);
  const float* w = kv ? a.w_c : a.w_q;
  float v[CH][VEC];
  float q = 0.f;
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int col = (lane + 64 * c) * VEC;
    if (col < np) {
      VyChunk<T>::load(src + col, v[c]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) q += v[c][e] * v[c][e];   // (the padding columns are zero)
    }
  }
  const float rstd = rsqrt_refined(vy_wave_sum(q) / (float)n + a.eps);
  T* dst = kv ? (a.c_out ? (T*)a.c_out + row * a.ldc : nullptr) : (T*)a.q_out + row * a.ldq;
  T* cdst = nullptr;
  if (kv && a.cache) {
    const int b = (int)(row / a.L), l = (int)(row - (int64_t)b * a.L);
    const int slot = a.slots ? a.slots[b] : b;
    const int pos = a.start[slot] + l, n = a.count ? a.count[b] : a.L;
    const bool held = a.ring ? l + a.cap >= n : pos < a.cap;      // (of a ring: not overwritten by a later one of these tokens)
    if (l < n && held) cdst = (T*)a.cache + slot * a.c_ss + (a.ring ? pos % a.cap : pos) * a.c_st;
  }
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int col = (lane + 64 * c) * VEC;
    if (col < np) {
      float o[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] = v[c][e] * rstd * w[col + e];
      if (dst) VyChunk<T>::store(dst + col, o);
      if (cdst) VyChunk<T>::store(cdst + col, o);
    }
  }
}

template <typename T>
int latent_norm_go(const LatentNormArgs& a, hipStream_t st) {
  const int np = a.w_q && a.npq > a.npc ? a.npq : a.npc;
  const int nch = (np + VyChunk<T>::VEC - 1) / VyChunk<T>::VEC;
  const dim3 grid((unsigned)vy_cdiv(a.w_q ? 2 * a.M : a.M, 4)), block(256);
  if (nch <= 64) hipLaunchKernelGGL((latent_norm_kernel<T, 1>), grid, block, 0, st, a);
  else if (nch <= 128) hipLaunchKernelGGL((latent_norm_kernel<T, 2>), grid, block, 0, st, a);
  else if (nch <= 256) hipLaunchKernelGGL((latent_norm_kernel<T, 4>), grid, block, 0, st, a);
  else if (nch <= 512) hipLaunchKernelGGL((latent_norm_kernel<T, 8>), grid, block, 0, st, a);
  else if (nch <= 1024) hipLaunchKernelGGL((latent_norm_kernel<T, 16>), grid, block, 0, st, a);
  else return 1;
  return 0;
}

template <typename T, int CH>
__global__ __launch_bounds__(256) void rmsnorm_gate_kernel(const T* __restrict__ x, int64_t ldx, const float* __restrict__ w,
                                                           const T* __restrict__ gate, int64_t ldg, T* __restrict__ y,
                                                           int64_t ldy, int N, int NP, float eps) {
  __shared__ float red[4];
  constexpr int VEC = VyChunk<T>::VEC;
  const int64_t row = blockIdx.x;
  float v[CH][VEC], g[CH][VEC];
  float q = 0.f;
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int col = ((int)threadIdx.x + 256 * c) * VEC;
    if (col < NP) {
      VyChunk<T>::load(x + row * ldx + col, v[c]);
      VyChunk<T>::load(gate + row * ldg + col, g[c]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) q += v[c][e] * v[c][e];
    }
  }
  const float rstd = rsqrt_refined(row_sum<256>(q, red, 0) / (float)N + eps);
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int col = ((int)threadIdx.x + 256 * c) * VEC;
    if (col < NP) {
      float o[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] = v[c][e] * rstd * w[col + e] * vy_sigmoid(g[c][e]);
      VyChunk<T>::store(y + row * ldy + col, o);
    }
  }
}

// LPH lanes per head (a power of two up to a wave), one 16-byte chunk per lane and pass
template <typename T, int LPH>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(const T* __restrict__ x, int64_t ldx, const float* __restrict__ w,
                                                             const T* __restrict__ gate, int64_t ldg, T* __restrict__ y, int64_t ldy, int64_t units, int heads,
                                                             int N, int NP, float eps) {
  constexpr int VEC = VyChunk<T>::VEC;
  const int sub = threadIdx.x % LPH;
  const int64_t u = (int64_t)blockIdx.x * (256 / LPH) + threadIdx.x / LPH;
  const int64_t uc = u < units ? u : units - 1, row = uc / heads;
  const int head = (int)(uc - row * heads);
  const T* xr = x + row * ldx + (int64_t)head * NP;
  const T* gr = gate ? gate + row * ldg + (int64_t)head * NP : nullptr;
  float v[VEC], g[VEC], q = 0.f;
  for (int c = sub * VEC; c < NP; c += LPH * VEC) {
    VyChunk<T>::load(xr + c, v);
    if (gr) VyChunk<T>::load(gr + c, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) q += v[e] * v[e];   // (the padding columns are zero)
  }
#pragma unroll
  for (int o = LPH / 2; o > 0; o >>= 1) q += __shfl_xor(q, o, 64);
  const float rstd = rsqrt_refined(q / (float)N + eps);
  if (u >= units) return;
  for (int c = sub * VEC; c < NP; c += LPH * VEC) {
    if (LPH * VEC < NP) {   // several passes: read again (from cache)
      VyChunk<T>::load(xr + c, v);
      if (gr) VyChunk<T>::load(gr + c, g);
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] *= rstd;
    if (w) {
#pragma unroll
      for (int e = 0; e < VEC; e += 4) {
        float f[4];
        load4<float>(w + c + e, f);
#pragma unroll
        for (int i = 0; i < 4; ++i) v[e + i] *= f[i];
      }
    }
    if (gr) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] *= vy_silu(g[e]);
    }
    VyChunk<T>::store(y + row * ldy + (int64_t)head * NP + c, v);
  }
}

template <typename T>
void head_norm_gate_go(const void* x, int64_t ldx, const float* w, const void* gate, int64_t ldg, void* y, int64_t ldy, int64_t M, int heads, int N,
                       int NP, float eps, hipStream_t st) {
  const int nch = NP / VyChunk<T>::VEC;
  const int64_t units = M * heads;
#define HN_GO(L) hipLaunchKernelGGL((head_norm_gate_kernel<T, L>), dim3((unsigned)vy_cdiv(units, 256 / L)), dim3(256), 0, st, (const T*)x, ldx, w, (const T*)gate, ldg, (T*)y, ldy, units, heads, N, NP, eps)
  if (nch <= 1) HN_GO(1);
  else if (nch <= 4) HN_GO(4);
  else if (nch <= 8) HN_GO(8);
  else if (nch <= 16) HN_GO(16);
  else if (nch <= 32) HN_GO(32);
  else HN_GO(64);
#undef HN_GO
}

}  // namespace

// internal: the step driver also advances the sequence lengths in this launch (advance[slots[i]] += 1 for i < n_adv)
int vy_residual_norm_ex(float* x, int64_t ldx, const void* y, int64_t ldy, const void* table, int64_t ldt, const int64_t* ids,
                        int64_t V, int32_t* err, float table_scale, const vy_routed_rows* routed, const float* w_post,
                        float eps_post, const float* w_pre, float eps_pre, void* h, int64_t ldh, int64_t M, int64_t N, int64_t NP,
                        int rms, int* advance, const int* slots, int n_adv, int dtype, void* stream) {
  const char* who = "vy_residual_norm";
  if (!x || M <= 0 || N <= 0 || NP < N) VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (NP % 4 || ldx % 4 || ldy % 4 || ldt % 4 || ldh % 4 || ldx < NP) VY_FAIL(VY_ERR_ARG, "%s: padded widths and row strides must be multiples of 4", who);
  if (ids && !table) VY_FAIL(VY_ERR_ARG, "%s: token ids without a table", who);
  ResNormArgs a{};
  a.x = x; a.ldx = ldx; a.y = y; a.ldy = ldy; a.table = table; a.ldt = ldt; a.ids = ids; a.V = V; a.err = err;
  a.w_post = w_post; a.w_pre = w_pre; a.h = h; a.ldh = ldh; a.M = M; a.N = (int)N; a.NP = (int)NP;
  a.eps_post = eps_post; a.eps_pre = eps_pre; a.advance = advance; a.slots = slots; a.n_adv = n_adv;
  a.table_scale = table_scale;
  if (routed) {
    if (ids || !routed->rows || !routed->weight || routed->top <= 0 || routed->ld % 4 || routed->ld < NP)
      VY_FAIL(VY_ERR_ARG, "%s: bad routed rows", who);
    a.er = routed->rows; a.lder = routed->ld; a.epos = routed->pos; a.ew = routed->weight; a.top = routed->top;
  }
  hipStream_t st = (hipStream_t)stream;
  int rc;
  if (dtype == VY_BF16) rc = residual_norm_any<bf16>(a, rms, st);
  else if (dtype == VY_F32) rc = residual_norm_any<float>(a, rms, st);
  else VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  if (rc) VY_FAIL(VY_ERR_UNSUPPORTED, "%s: width %ld", who, (long)NP);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}

extern "C" int vy_residual_norm(float* x, int64_t ldx, const void* y, int64_t ldy, const void* table, int64_t ldt,
                                const int64_t* ids, int64_t V, int32_t* err_flag, const float* w_post, float eps_post,
                                const float* w_pre, float eps_pre, void* h, int64_t ldh, int64_t M, int64_t N, int64_t NP,
                                int rms, int dtype, void* stream) {
  return vy_residual_norm_ex(x, ldx, y, ldy, table, ldt, ids, V, err_flag, 1.f, nullptr, w_post, eps_post, w_pre, eps_pre, h,
                             ldh, M, N, NP, rms, nullptr, nullptr, 0, dtype, stream);
}

extern "C" int vy_residual_norm_routed(float* x, int64_t ldx, const void* y, int64_t ldy, const void* table, int64_t ldt,
                                       const int64_t* ids, int64_t V, int32_t* err_flag, float table_scale,
                                       const vy_routed_rows* routed, const float* w_post, float eps_post, const float* w_pre,
                                       float eps_pre, void* h, int64_t ldh, int64_t M, int64_t N, int64_t NP, int rms, int dtype,
                                       void* stream) {
  return vy_residual_norm_ex(x, ldx, y, ldy, table, ldt, ids, V, err_flag, table_scale, routed, w_post, eps_post, w_pre, eps_pre,
                             h, ldh, M, N, NP, rms, nullptr, nullptr, 0, dtype, stream);
}

extern "C" int vy_latent_norm(const void* p, int64_t ldp, const float* w_q, void* q_out, int64_t ldq, int32_t nq, int32_t npq,
                              const float* w_c, void* c_out, int64_t ldc, int32_t nc, int32_t npc, void* cache, int64_t c_ss,
                              int64_t c_st, int32_t cap, int ring, const int32_t* slots, const int32_t* start,
                              const int32_t* count, int64_t B, int64_t L, float eps, int dtype, void* stream) {
  const char* who = "vy_latent_norm";
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!p || !w_c || B <= 0 || L <= 0 || nc <= 0 || npq < 0 || npc < nc || (w_q && (!q_out || nq <= 0 || npq < nq))) VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (npq % vec || npc % vec || ldp % vec || ldq % vec || ldc % vec || c_ss % vec || c_st % vec)
    VY_FAIL(VY_ERR_ARG, "%s: widths and strides must be multiples of %d", who, vec);
  if (cache && (!start || cap <= 0)) VY_FAIL(VY_ERR_ARG, "%s: cache without start positions / capacity", who);
  LatentNormArgs a{p, ldp, w_q, q_out, ldq, nq, npq, w_c, c_out, ldc, nc, npc, cache, c_ss, c_st, cap, ring, slots, start, count,
                   B * L, (int)L, eps};
  int rc;
  if (dtype == VY_BF16) rc = latent_norm_go<bf16>(a, (hipStream_t)stream);
  else if (dtype == VY_F32) rc = latent_norm_go<float>(a, (hipStream_t)stream);
  else VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  if (rc) VY_FAIL(VY_ERR_UNSUPPORTED, "%s: latent width %d / %d", who, npq, npc);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}

extern "C" int vy_head_norm_gate(const void* x, int64_t ldx, const float* w, const void* gate, int64_t ldg, void* y, int64_t ldy,
                                 int64_t M, int32_t heads, int64_t N, int64_t NP, float eps, int dtype, void* stream) {
  const char* who = "vy_head_norm_gate";
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!x || !y || M <= 0 || heads <= 0 || N <= 0 || NP < N || NP > 1 << 20 || M * heads > INT32_MAX)
    VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (NP % vec || ldx % vec || ldg % vec || ldy % vec) VY_FAIL(VY_ERR_ARG, "%s: widths and strides must be multiples of %d", who, vec);
  if (dtype == VY_BF16) head_norm_gate_go<bf16>(x, ldx, w, gate, ldg, y, ldy, M, heads, (int)N, (int)NP, eps, (hipStream_t)stream);
  else head_norm_gate_go<float>(x, ldx, w, gate, ldg, y, ldy, M, heads, (int)N, (int)NP, eps, (hipStream_t)stream);
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}

extern "C" int vy_rmsnorm_gate(const void* x, int64_t ldx, const float* w, const void* gate, int64_t ldg, void* y, int64_t ldy,
                               int64_t M, int64_t N, int64_t NP, float eps, int dtype, void* stream) {
  const char* who = "vy_rmsnorm_gate";
  const int vec = dtype == VY_BF16 ? 8 : 4;
  if (!x || !w || !gate || !y || M <= 0 || N <= 0 || NP < N) VY_FAIL(VY_ERR_ARG, "%s: bad arguments", who);
  if (NP % vec || ldx % vec || ldg % vec || ldy % vec) VY_FAIL(VY_ERR_ARG, "%s: widths and strides must be multiples of %d", who, vec);
  const dim3 grid((unsigned)M), block(256);
  hipStream_t st = (hipStream_t)stream;
#define RG_GO(T, CH) hipLaunchKernelGGL((rmsnorm_gate_kernel<T, CH>), grid, block, 0, st, (const T*)x, ldx, w, (const T*)gate, ldg, (T*)y, ldy, (int)N, (int)NP, eps)
#define RG_DISPATCH(T)                                          \
  do {                                                          \
    const int64_t nch = vy_cdiv(NP, vec);                       \
    if (nch <= 256) RG_GO(T, 1);                                \
    else if (nch <= 512) RG_GO(T, 2);                           \
    else if (nch <= 1024) RG_GO(T, 4);                          \
    else if (nch <= 4096) RG_GO(T, 16);                         \
    else VY_FAIL(VY_ERR_UNSUPPORTED, "%s: width %ld", who, (long)NP); \
  } while (0)
  if (dtype == VY_BF16) RG_DISPATCH(bf16);
  else if (dtype == VY_F32) RG_DISPATCH(float);
  else VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
#undef RG_DISPATCH
#undef RG_GO
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}
