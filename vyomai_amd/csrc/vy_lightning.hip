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
#include "vy_decay.h"

namespace {

using namespace vy_decay;

// ---- chunked form ----------------------------------------------------------------------------
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
              (int)vy_cdiv(L, C), (float*)ws, (const float2*)rope, rope_dims / 2, rope_len > 0 ? rope_len : 1, k_scale, nullptr, nullptr, nullptr};
  if (chunked(L, dk, dtype)) {
    if (!ws || ws_bytes < vy_decay_attn_ws_bytes(B, L, h, dk, dv, dtype)) VY_FAIL(VY_ERR_ARG, "%s: workspace too small", who);
    const dim3 grid(a.nc, (unsigned)vy_cdiv(dv, 64), (unsigned)(B * h)), block(256);
    const dim3 sgrid((unsigned)vy_cdiv((int64_t)dk * dv, 1024), (unsigned)(B * h));
#define CH_GO(D, ROT)                                                           \
  do {                                                                          \
    hipLaunchKernelGGL((chunk_kv_kernel<D, ROT>), grid, block, 0, st, a);       \
    hipLaunchKernelGGL(chunk_scan_kernel<false>, sgrid, block, 0, st, a);              \
    hipLaunchKernelGGL((chunk_out_kernel<D, ROT>), grid, block, 0, st, a);      \
  } while (0)
    const bool rot = a.half || k_scale != 1.f;
    if (dk <= 32) { if (rot) CH_GO(32, true); else CH_GO(32, false); }
    else if (dk <= 64) { if (rot) CH_GO(64, true); else CH_GO(64, false); }
    else { if (rot) CH_GO(128, true); else CH_GO(128, false); }
#undef CH_GO
  } else if (dtype == VY_BF16 ? recurrent_go<bf16, false>(a, st) : recurrent_go<float, false>(a, st)) {
    VY_FAIL(VY_ERR_UNSUPPORTED, "%s: key width %d > 512", who, dk);
  }
  VY_CHECK_LAUNCH(who);
  return VY_OK;
}
