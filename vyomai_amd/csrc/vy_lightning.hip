// Linear attention with a per-head decay:
//   S_t = decay S_(t-1) + k_t v_t^T ,  o_t = S_t^T q_t
// with q, k, v = silu of the projections (lightning attention), or q and k rotated by their position and k scaled (retention).
//
// Two forms of the same sums:
//   * decay_recurrent_kernel: token by token, the state in registers (fp32).  Decode steps, fp32 models, and head widths
//     the chunked form does not cover.
//   * chunked (bf16 prefill), C = VY_DECAY_CHUNK tokens at a time on MFMA, three launches:
//       chunk_kv_kernel    U_c = sum_j decay^(m-1-j) k_j v_j^T over the m tokens of chunk c         (all chunks at once)
//       chunk_scan_kernel  S_(c+1) = decay^m S_c + U_c, elementwise along the chunks; leaves S_c where U_c was
//       chunk_out_kernel   O = [lower(Q K^T) * decay^(i-j)] V + decay^(i+1) Q S_c                    (all chunks at once)
//
// 32-bit throughout where it enters the recurrence: decays are fp32 tables made in double precision on the host, the state
// is fp32, and every MFMA operand that carries a decay or a state (decayed keys, decayed scores, S_c) is fed as TWO bf16
// numbers hi + lo (~16 bits of mantissa); only q, k, v themselves -- projections -- are plain bf16.  Rotated q and k (ROT) are no
// projections any more: they are made in fp32 on the way in and go on as hi + lo as well.
#include "vy_common.h"

namespace {

constexpr int C = VY_DECAY_CHUNK;

struct DecayArgs {
  const void* p; int64_t ldp; int64_t oq, ok, ov;
  float* state; const float* pow;          // [slot][h][dk][dv]; [h][C + 1]
  const int* slots; const int* start; const int* count;
  void* out; int64_t ldo;
  int B, L, h, dk, dv, silu, nc;
  float* U;                                // [B * h][nc][dk][dv]
  const float2* rope; int half, rope_len;  // half = 0: no rotation; pairs of neighbouring columns
  float k_scale;
};

// (cos, sin) of the first pair of a token's row of the table (clamped: padding rows only)
__device__ __forceinline__ const float2* trig_row(const DecayArgs& a, int pos) {
  return a.rope + (int64_t)(pos < a.rope_len ? pos : a.rope_len - 1) * a.half;
}
// N consecutive columns d0 .. (both even) of a row
template <int N>
__device__ __forceinline__ void rotate(const float2* trig, int half, int d0, float (&v)[N]) {
  if (d0 + N <= 2 * half && (half & 1) == 0 && N % 4 == 0) {   // whole 16-byte pieces of the table's row
#pragma unroll
    for (int e = 0; e < N; e += 4) {
      const f32x4 cs = *reinterpret_cast<const f32x4*>(trig + ((d0 + e) >> 1));
      const float u = v[e], w = v[e + 1], x = v[e + 2], y = v[e + 3];
      v[e] = u * cs[0] - w * cs[1];
      v[e + 1] = w * cs[0] + u * cs[1];
      v[e + 2] = x * cs[2] - y * cs[3];
      v[e + 3] = y * cs[2] + x * cs[3];
    }
    return;
  }
#pragma unroll
  for (int e = 0; e < N; e += 2) {
    const int i = (d0 + e) >> 1;
    if (i < half) {
      const float2 cs = trig[i];
      const float u = v[e], w = v[e + 1];
      v[e] = u * cs.x - w * cs.y;
      v[e + 1] = w * cs.x + u * cs.y;
    }
  }
}

__device__ __forceinline__ float activate(float x, int silu) { return silu ? vy_silu(x) : x; }
__device__ __forceinline__ void split_bf16(float x, bf16& hi, bf16& lo) {
  const float h = vy_round_bf16(x);
  hi = (bf16)h;
  lo = (bf16)(x - h);
}

// ---- recurrence ------------------------------------------------------------------------------
// workgroup = COLS value columns of one (b, head); thread (rg, col) keeps rows rg, rg + RG, ... of the state column.
// TT tokens are staged at a time; the RG partial dot products of an output are added after each stage.
template <typename T, int COLS, int RPT, int TT>
__global__ __launch_bounds__(256) void decay_recurrent_kernel(DecayArgs a) {
  constexpr int RG = 256 / COLS, DK = RG * RPT;
  __shared__ float qs[TT][DK], ks[TT][DK];
  __shared__ float vs[TT][COLS];
  __shared__ float red[TT][RG][COLS + 1];
  const int col = threadIdx.x % COLS, rg = threadIdx.x / COLS;
  const int head = blockIdx.y, b = blockIdx.z;
  const int c0 = (int)blockIdx.x * COLS, vc = c0 + col;
  const int slot = a.slots ? a.slots[b] : b;
  const int n = a.count ? min(a.count[b], a.L) : a.L;
  const float decay = a.pow[(int64_t)head * (C + 1) + 1];
  float* S = a.state + ((int64_t)slot * a.h + head) * a.dk * a.dv;
  float s[RPT];
  const int first = a.start[slot];
  const bool fresh = first == 0;
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg + RG * i;
    s[i] = r < a.dk && vc < a.dv ? S[(int64_t)r * a.dv + vc] : 0.f;
  }
  const T* P = (const T*)a.p + (int64_t)b * a.L * a.ldp;
  T* O = (T*)a.out + (int64_t)b * a.L * a.ldo + head * a.dv;
  for (int t0 = 0; t0 < n; t0 += TT) {
    const int m = min(TT, n - t0);
    for (int i = threadIdx.x; i < m * DK; i += 256) {
      const int t = i / DK, d = i % DK;
      const T* row = P + (int64_t)(t0 + t) * a.ldp + head * a.dk + d;
      const bool ok = d < a.dk;
      float q = ok ? activate(VyT<T>::ld(row + a.oq), a.silu) : 0.f;
      float k = ok ? activate(VyT<T>::ld(row + a.ok), a.silu) : 0.f;
      if (d < 2 * a.half) {
        const int to = d & 1 ? -1 : 1;   // the other column of the pair
        const float2 cs = trig_row(a, first + t0 + t)[d >> 1];
        const float s = d & 1 ? cs.y : -cs.y;
        q = q * cs.x + activate(VyT<T>::ld(row + a.oq + to), a.silu) * s;
        k = k * cs.x + activate(VyT<T>::ld(row + a.ok + to), a.silu) * s;
      }
      qs[t][d] = q;
      ks[t][d] = k * a.k_scale;
    }
    for (int i = threadIdx.x; i < m * COLS; i += 256) {
      const int t = i / COLS, d = c0 + i % COLS;
      vs[t][i % COLS] = d < a.dv ? activate(VyT<T>::ld(P + (int64_t)(t0 + t) * a.ldp + a.ov + head * a.dv + d), a.silu) : 0.f;
    }
    __syncthreads();
    for (int t = 0; t < m; ++t) {
      const float v = vs[t][col];
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < RPT; ++i) {
        const float before = fresh && t0 + t == 0 ? 0.f : s[i];   // an empty slot's state is zero, whatever lies there
        s[i] = fmaf(decay, before, ks[t][rg + RG * i] * v);
        o = fmaf(s[i], qs[t][rg + RG * i], o);
      }
      red[t][rg][col] = o;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < m * COLS; i += 256) {
      const int t = i / COLS, cc = i % COLS;
      float o = 0.f;
#pragma unroll
      for (int r = 0; r < RG; ++r) o += red[t][r][cc];
      if (c0 + cc < a.dv) VyT<T>::st(O + (int64_t)(t0 + t) * a.ldo + c0 + cc, o);
    }
  }
  // the padding behind a short sequence: finite values for whatever reads whole batches
  for (int64_t t = n + rg; t < a.L; t += RG)
    if (vc < a.dv) VyT<T>::st(O + t * a.ldo + vc, 0.f);
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg + RG * i;
    if (r < a.dk && vc < a.dv) S[(int64_t)r * a.dv + vc] = s[i];
  }
}

// ---- chunked form ----------------------------------------------------------------------------
__device__ __forceinline__ bf16x8 load8(const bf16* p, bool ok, int silu) {
  bf16x8 r = {};
  if (ok) {
    r = *reinterpret_cast<const bf16x8*>(p);
    if (silu) {
#pragma unroll
      for (int e = 0; e < 8; ++e) r[e] = (bf16)vy_silu((float)r[e]);
    }
  }
  return r;
}

// fragment of a transposed operand: 16 columns (block n) x 32 rows (block tt) of a row-major LDS tile
template <int OFF>
__device__ __forceinline__ bf16x8 tr_frag(unsigned lane_addr, int pitch) {
  union { struct { s16x4 a, b; } s; bf16x8 v; } u;
  u.s.a = vy_lds_tr16_off<OFF>(lane_addr);
  u.s.b = vy_lds_tr16_off<OFF>(lane_addr + 16 * pitch);
  return u.v;
}

// eight key columns d .. of a chunk's token t: rotated and scaled (ROT), else as loaded
template <bool ROT>
__device__ __forceinline__ void key8(const DecayArgs& a, const bf16* p, bool ok, int pos, int d, float (&v)[8]) {
  const bf16x8 k8 = load8(p, ok, a.silu);
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = (float)k8[e];
  if constexpr (ROT) {
    if (a.half) rotate(trig_row(a, pos), a.half, d, v);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] *= a.k_scale;
  }
}

// grid (chunks, value blocks of 64, B * h)
template <int DKP, bool ROT>
__global__ __launch_bounds__(256) void chunk_kv_kernel(DecayArgs a) {
  constexpr int KP = (DKP + 8) * 2, VP = (64 + 8) * 2;
  __shared__ __attribute__((aligned(16))) char smem[C * (2 * KP + VP)];
  char* kh = smem;
  char* kl = smem + C * KP;
  char* vt = smem + 2 * C * KP;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r16 = lane & 15, kq = lane >> 4;
  const int ch = blockIdx.x, bh = blockIdx.z, b = bh / a.h, head = bh - b * a.h;
  const int v0 = (int)blockIdx.y * 64;
  const int n = a.count ? min(a.count[b], a.L) : a.L;
  const int m = max(0, min(C, n - ch * C));            // tokens of this chunk
  const int first = ROT ? a.start[a.slots ? a.slots[b] : b] + ch * C : 0;
  const float* pw = a.pow + (int64_t)head * (C + 1);
  const bf16* P = (const bf16*)a.p + ((int64_t)b * a.L + ch * C) * a.ldp;
  for (int i = threadIdx.x; i < C * (DKP / 8); i += 256) {
    const int t = i / (DKP / 8), d = (i % (DKP / 8)) * 8;
    const bool ok = t < m && d < a.dk;
    float k8[8];
    key8<ROT>(a, P + (int64_t)t * a.ldp + a.ok + head * a.dk + d, ok, first + t, d, k8);
    const float w = t < m ? pw[m - 1 - t] : 0.f;
    bf16x8 hi, lo;
#pragma unroll
    for (int e = 0; e < 8; ++e) { bf16 x, y; split_bf16(k8[e] * w, x, y); hi[e] = x; lo[e] = y; }
    *reinterpret_cast<bf16x8*>(kh + t * KP + d * 2) = hi;
    *reinterpret_cast<bf16x8*>(kl + t * KP + d * 2) = lo;
  }
  for (int i = threadIdx.x; i < C * 8; i += 256) {
    const int t = i >> 3, d = (i & 7) * 8;
    const bool ok = t < m && v0 + d < a.dv;
    *reinterpret_cast<bf16x8*>(vt + t * VP + d * 2) = load8(P + (int64_t)t * a.ldp + a.ov + head * a.dv + v0 + d, ok, a.silu);
  }
  __syncthreads();
  float* U = a.U + ((int64_t)bh * a.nc + ch) * a.dk * a.dv;
  const int lr = 4 * kq + (r16 >> 2), lc = (4 * (r16 & 3)) * 2;
  const unsigned khb = vy_lds_addr(kh) + lr * KP + lc, klb = vy_lds_addr(kl) + lr * KP + lc, vb = vy_lds_addr(vt) + lr * VP + lc;
  for (int blk = wave; blk < DKP / 16; blk += 4) {      // 16 key rows of the state
    if (blk * 16 >= a.dk) break;
    f32x4 acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int tt = 0; tt < C / 32; ++tt) {
      bf16x8 fh = tr_frag<0>(khb + tt * 32 * KP + blk * 32, KP), fl = tr_frag<0>(klb + tt * 32 * KP + blk * 32, KP);
      bf16x8 fv[4];
      vy_static_for<4>([&](auto i_c) {
        constexpr int i = decltype(i_c)::value;
        fv[i] = tr_frag<i * 32>(vb + tt * 32 * VP, VP);
      });
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      vy_tie(fh);
      vy_tie(fl);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        vy_tie(fv[i]);
        acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fl, fv[i], acc[i], 0, 0, 0);
        acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fh, fv[i], acc[i], 0, 0, 0);
      }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int r = blk * 16 + 4 * kq + e, c = v0 + 16 * i + r16;
        if (r < a.dk && c < a.dv) U[(int64_t)r * a.dv + c] = acc[i][e];
      }
  }
}

// S_c as hi / lo quads in place of the four floats of U_c: one 16-byte element per thread and chunk
__global__ __launch_bounds__(256) void chunk_scan_kernel(DecayArgs a) {
  const int bh = blockIdx.y, b = bh / a.h, head = bh - b * a.h;
  const int64_t elems = (int64_t)a.dk * a.dv;
  const int64_t e0 = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (e0 >= elems) return;
  const int slot = a.slots ? a.slots[b] : b;
  const int n = a.count ? min(a.count[b], a.L) : a.L;
  const float* pw = a.pow + (int64_t)head * (C + 1);
  float* S = a.state + ((int64_t)slot * a.h + head) * elems + e0;
  float* U = a.U + (int64_t)bh * a.nc * elems + e0;
  f32x4 s = {0.f, 0.f, 0.f, 0.f};
  if (a.start[slot] != 0) s = *reinterpret_cast<const f32x4*>(S);
  const float full = pw[C];
  constexpr int UN = 4;                       // chunks per batch of loads; the next batch is requested before this one is used
  f32x4 u[UN], nx[UN];
  auto fetch = [&](int c0, f32x4 (&r)[UN]) {
#pragma unroll
    for (int i = 0; i < UN; ++i) r[i] = *reinterpret_cast<const f32x4*>(U + min(c0 + i, a.nc - 1) * elems);
  };
  fetch(0, u);
  for (int c0 = 0; c0 < a.nc; c0 += UN) {
    if (c0 + UN < a.nc) fetch(c0 + UN, nx);
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      if (c0 + i >= a.nc) break;
      union { struct { bf16x4 hi, lo; } h; f32x4 f; } w;
#pragma unroll
      for (int e = 0; e < 4; ++e) { bf16 x, y; split_bf16(s[e], x, y); w.h.hi[e] = x; w.h.lo[e] = y; }
      *reinterpret_cast<f32x4*>(U + (c0 + i) * elems) = w.f;
      const int m = max(0, min(C, n - (c0 + i) * C));
      const float d = m == C ? full : pw[m];
#pragma unroll
      for (int e = 0; e < 4; ++e) s[e] = fmaf(d, s[e], u[i][e]);
    }
#pragma unroll
    for (int i = 0; i < UN; ++i) u[i] = nx[i];
  }
  *reinterpret_cast<f32x4*>(S) = s;
}

// grid (chunks, value blocks of 64, B * h): wave w computes rows 16 w .. + 15 of the chunk (C = 64)
template <int DKP, bool ROT>
__global__ __launch_bounds__(256) void chunk_out_kernel(DecayArgs a) {
  static_assert(C == 64, "one 16-row block per wave");
  constexpr int KP = (DKP + 8) * 2, VP = (64 + 8) * 2;
  constexpr int KS = DKP / 32, KB = ROT ? 2 : 1;        // key images: hi, lo
  __shared__ __attribute__((aligned(16))) char smem[C * (KB * KP + VP) + 2 * DKP * VP + (C + 1) * 4];
  char* kt = smem;
  char* vt = smem + KB * C * KP;
  char* sh = vt + C * VP;
  char* sl = sh + DKP * VP;
  float* pw = reinterpret_cast<float*>(sl + DKP * VP);
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r16 = lane & 15, kq = lane >> 4;
  const int ch = blockIdx.x, bh = blockIdx.z, b = bh / a.h, head = bh - b * a.h;
  const int v0 = (int)blockIdx.y * 64;
  const int rows = min(C, a.L - ch * C);
  const bf16* P = (const bf16*)a.p + ((int64_t)b * a.L + ch * C) * a.ldp;
  const float* Sg = a.U + ((int64_t)bh * a.nc + ch) * a.dk * a.dv;
  const int first = ROT ? a.start[a.slots ? a.slots[b] : b] + ch * C : 0;
  for (int i = threadIdx.x; i < C * (DKP / 8); i += 256) {
    const int t = i / (DKP / 8), d = (i % (DKP / 8)) * 8;
    const bf16* src = P + (int64_t)t * a.ldp + a.ok + head * a.dk + d;
    const bool ok = t < rows && d < a.dk;
    if constexpr (ROT) {
      float k8[8];
      key8<true>(a, src, ok, first + t, d, k8);
      bf16x8 hi, lo;
#pragma unroll
      for (int e = 0; e < 8; ++e) { bf16 x, y; split_bf16(k8[e], x, y); hi[e] = x; lo[e] = y; }
      *reinterpret_cast<bf16x8*>(kt + t * KP + d * 2) = hi;
      *reinterpret_cast<bf16x8*>(kt + C * KP + t * KP + d * 2) = lo;
    } else {
      *reinterpret_cast<bf16x8*>(kt + t * KP + d * 2) = load8(src, ok, a.silu);
    }
  }
  for (int i = threadIdx.x; i < C * 8; i += 256) {
    const int t = i >> 3, d = (i & 7) * 8;
    *reinterpret_cast<bf16x8*>(vt + t * VP + d * 2) =
        load8(P + (int64_t)t * a.ldp + a.ov + head * a.dv + v0 + d, t < rows && v0 + d < a.dv, a.silu);
  }
  for (int i = threadIdx.x; i < DKP * 16; i += 256) {
    const int r = i >> 4, c = (i & 15) * 4;
    union { struct { bf16x4 hi, lo; } h; f32x4 f; } w;
    w.f = f32x4{0.f, 0.f, 0.f, 0.f};
    if (r < a.dk && v0 + c < a.dv) w.f = *reinterpret_cast<const f32x4*>(Sg + (int64_t)r * a.dv + v0 + c);
    *reinterpret_cast<bf16x4*>(sh + r * VP + c * 2) = w.h.hi;
    *reinterpret_cast<bf16x4*>(sl + r * VP + c * 2) = w.h.lo;
  }
  for (int i = threadIdx.x; i <= C; i += 256) pw[i] = a.pow[(int64_t)head * (C + 1) + i];
  // the wave's query rows, in the k order of the transposed state fragments (4 kq .. and 16 + 4 kq ..)
  const int qi = 16 * wave + r16;
  bf16x8 qf[KS], ql[ROT ? KS : 1];
  {
    const bf16* Q = P + (int64_t)min(qi, rows - 1) * a.ldp + a.oq + head * a.dk;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) {
        const int d = 32 * ks + 16 * hf + 4 * kq;
        bf16x4 q4 = {};
        if (d < a.dk) q4 = *reinterpret_cast<const bf16x4*>(Q + d);
        if constexpr (ROT) {
          float v[4];
#pragma unroll
          for (int e = 0; e < 4; ++e) v[e] = activate((float)q4[e], a.silu);
          if (a.half) rotate(trig_row(a, first + qi), a.half, d, v);
#pragma unroll
          for (int e = 0; e < 4; ++e) { bf16 x, y; split_bf16(v[e], x, y); qf[ks][4 * hf + e] = x; ql[ks][4 * hf + e] = y; }
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e) qf[ks][4 * hf + e] = (bf16)activate((float)q4[e], a.silu);
        }
      }
    }
  }
  __syncthreads();
  const int lr = 4 * kq + (r16 >> 2), lc = (4 * (r16 & 3)) * 2;
  const unsigned shb = vy_lds_addr(sh) + lr * VP + lc, slb = vy_lds_addr(sl) + lr * VP + lc, vb = vy_lds_addr(vt) + lr * VP + lc;
  f32x4 o[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  // O^T += S^T Q^T
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) {
    bf16x8 fh[4], fl[4];
    vy_static_for<4>([&](auto i_c) {
      constexpr int i = decltype(i_c)::value;
      fh[i] = tr_frag<i * 32>(shb + ks * 32 * VP, VP);
      fl[i] = tr_frag<i * 32>(slb + ks * 32 * VP, VP);
    });
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      vy_tie(fh[i]);
      vy_tie(fl[i]);
      o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fl[i], qf[ks], o[i], 0, 0, 0);
      if constexpr (ROT) o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fh[i], ql[ks], o[i], 0, 0, 0);
      o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fh[i], qf[ks], o[i], 0, 0, 0);
    }
  }
  const float dq = pw[qi + 1];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) o[i][e] *= dq;
  // O^T += V^T (decayed scores)^T over 32 keys at a time
#pragma unroll
  for (int tt = 0; tt < C / 32; ++tt) {
    if (32 * tt > 16 * wave + 15) break;
    f32x4 sc[2];
#pragma unroll
    for (int blk = 0; blk < 2; ++blk) {
      sc[blk] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        union { struct { bf16x4 a, b; } h; bf16x8 v; } kf;
        const char* kr = kt + (32 * tt + 16 * blk + r16) * KP + (32 * ks + 4 * kq) * 2;
        kf.h.a = *reinterpret_cast<const bf16x4*>(kr);
        kf.h.b = *reinterpret_cast<const bf16x4*>(kr + 32);
        if constexpr (ROT) {
          union { struct { bf16x4 a, b; } h; bf16x8 v; } kl;
          kl.h.a = *reinterpret_cast<const bf16x4*>(kr + C * KP);
          kl.h.b = *reinterpret_cast<const bf16x4*>(kr + C * KP + 32);
          sc[blk] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kl.v, qf[ks], sc[blk], 0, 0, 0);
          sc[blk] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf.v, ql[ks], sc[blk], 0, 0, 0);
        }
        sc[blk] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf.v, qf[ks], sc[blk], 0, 0, 0);
      }
    }
    bf16x8 ph, pl;
#pragma unroll
    for (int blk = 0; blk < 2; ++blk)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int kj = 32 * tt + 16 * blk + 4 * kq + r;
        const float s = kj <= qi ? sc[blk][r] * pw[qi - kj] : 0.f;
        bf16 x, y;
        split_bf16(s, x, y);
        ph[4 * blk + r] = x;
        pl[4 * blk + r] = y;
      }
    bf16x8 fv[4];
    vy_static_for<4>([&](auto i_c) {
      constexpr int i = decltype(i_c)::value;
      fv[i] = tr_frag<i * 32>(vb + tt * 32 * VP, VP);
    });
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      vy_tie(fv[i]);
      o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fv[i], pl, o[i], 0, 0, 0);
      o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fv[i], ph, o[i], 0, 0, 0);
    }
  }
  if (qi < rows) {
    bf16* O = (bf16*)a.out + ((int64_t)b * a.L + ch * C + qi) * a.ldo + head * a.dv + v0;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = 16 * i + 4 * kq;
      if (v0 + c < a.dv) {
        bf16x4 w;
#pragma unroll
        for (int e = 0; e < 4; ++e) w[e] = (bf16)o[i][e];
        *reinterpret_cast<bf16x4*>(O + c) = w;
      }
    }
  }
}

bool chunked(int64_t L, int dk, int dtype) { return dtype == VY_BF16 && L > 1 && dk <= 128; }

template <typename T>
int recurrent_go(const DecayArgs& a, hipStream_t st) {
  const dim3 grid((unsigned)vy_cdiv(a.dv, 16), a.h, a.B), block(256);
  if (a.L == 1) {
    // a decode step streams the state: whole 256-byte row pieces where enough workgroups remain, else narrow columns
    const int64_t wide = vy_cdiv(a.dv, 64) * a.h * a.B;
    const dim3 wgrid((unsigned)vy_cdiv(a.dv, 64), a.h, a.B);
    if (wide >= 512 && a.dk <= 64) hipLaunchKernelGGL((decay_recurrent_kernel<T, 64, 16, 1>), wgrid, block, 0, st, a);
    else if (wide >= 512 && a.dk <= 128) hipLaunchKernelGGL((decay_recurrent_kernel<T, 64, 32, 1>), wgrid, block, 0, st, a);
    else if (a.dk <= 64) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 4, 1>), grid, block, 0, st, a);
    else if (a.dk <= 128) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 8, 1>), grid, block, 0, st, a);
    else if (a.dk <= 256) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 16, 1>), grid, block, 0, st, a);
    else if (a.dk <= 512) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 32, 1>), grid, block, 0, st, a);
    else return 1;
    return 0;
  }
  if (a.dk <= 64) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 4, 16>), grid, block, 0, st, a);
  else if (a.dk <= 128) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 8, 16>), grid, block, 0, st, a);
  else if (a.dk <= 256) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 16, 8>), grid, block, 0, st, a);
  else if (a.dk <= 512) hipLaunchKernelGGL((decay_recurrent_kernel<T, 16, 32, 8>), grid, block, 0, st, a);
  else return 1;
  return 0;
}

}  // namespace

extern "C" int64_t vy_decay_attn_ws_bytes(int64_t B, int64_t L, int32_t h, int32_t dk, int32_t dv, int dtype) {
  return chunked(L, dk, dtype) ? B * h * vy_cdiv(L, C) * dk * dv * 4 : 0;
}

extern "C" int vy_decay_attn(const void* p, int64_t ldp, int64_t oq, int64_t ok, int64_t ov, float* state,
                             const float* decay_pow, const int32_t* slots, const int32_t* start, const int32_t* count,
                             void* out, int64_t ldo, int64_t B, int64_t L, int32_t h, int32_t dk, int32_t dv, int silu,
                             const float* rope, int32_t rope_dims, int32_t rope_len, float k_scale, void* ws, int64_t ws_bytes,
                             int dtype, void* stream) {
  const char* who = "vy_decay_attn";
  if (!p || !state || !decay_pow || !start || !out) VY_FAIL(VY_ERR_ARG, "%s: null pointer", who);
  if (B <= 0 || L <= 0 || h <= 0 || dk <= 0 || dv <= 0 || L > INT32_MAX) VY_FAIL(VY_ERR_ARG, "%s: empty problem", who);
  if (dk % 8 || dv % 8 || ldp % 8 || ldo % 8 || oq % 8 || ok % 8 || ov % 8) VY_FAIL(VY_ERR_ARG, "%s: widths, strides and offsets must be multiples of 8", who);
  if (dtype != VY_BF16 && dtype != VY_F32) VY_FAIL(VY_ERR_ARG, "%s: bad dtype %d", who, dtype);
  if (B * h > 65535) VY_FAIL(VY_ERR_UNSUPPORTED, "%s: %ld (sequence, head) pairs", who, (long)(B * h));
  if (rope_dims < 0 || rope_dims % 2 || rope_dims > dk || (rope_dims && (!rope || rope_len < 1)))
    VY_FAIL(VY_ERR_ARG, "%s: rotary table of %d columns, %d positions for heads of %d", who, rope_dims, rope_len, dk);
  hipStream_t st = (hipStream_t)stream;
  DecayArgs a{p, ldp, oq, ok, ov, state, decay_pow, slots, start, count, out, ldo, (int)B, (int)L, h, dk, dv, silu,
              (int)vy_cdiv(L, C), (float*)ws, (const float2*)rope, rope_dims / 2, rope_len > 0 ? rope_len : 1, k_scale};
  if (chunked(L, dk, dtype)) {
    if (!ws || ws_bytes < vy_decay_attn_ws_bytes(B, L, h, dk, dv, dtype)) VY_FAIL(VY_ERR_ARG, "%s: workspace too small", who);
    const dim3 grid(a.nc, (unsigned)vy_cdiv(dv, 64), (unsigned)(B * h)), block(256);
    const dim3 sgrid((unsigned)vy_cdiv((int64_t)dk * dv, 1024), (unsigned)(B * h));
#define CH_GO(D, ROT)                                                           \
  do {                                                                          \
    hipLaunchKernelGGL((chunk_kv_kernel<D, ROT>), grid, block, 0, st, a);       \
    hipLaunchKernelGGL(chunk_scan_kernel, sgrid, block, 0, st, a);              \
    hipLaunchKernelGGL((chunk_out_kernel<D, ROT>), grid, block, 0, st, a);      \
  } while (0)
    const bool rot = a.half || k_scale != 1.f;
    if (dk <= 32) { if (rot) CH_GO(32, true); else CH_GO(32, false); }
    else if (dk <= 64) { if (rot) CH_GO(64, true); else CH_GO(64, false); }
    else { if (rot) CH_GO(128, true); else CH_GO(128, false); }
#undef CH_GO
  } else if (dtype == VY_BF16 ? recurrent_go<bf16>(a, st) : recurrent_go<float>(a, st)) {
    VY_FAIL(VY_ERR_UNSUPPORTED, "%s: key width %d > 512", who, dk);
  }
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}
