// End of a mixer and choice of experts in one launch (decode, bf16, up to 64 tokens): a workgroup takes one token from the residual
// sum to the experts it goes to.
//
//   x += norm(y) w_post ;  h = norm(x) w_pre or x ;  z = w_router h (fp32) ;  choice of experts and their weights (vy_moe.h)
//
// The router's matrix comes from L2 for all tokens but the first; its first rows are requested before the norm, so that a single
// token waits for memory once.  Each of 16 waves takes every 16th expert, h goes round through LDS.
#include "vy_moe.h"

namespace {

using namespace vy_moe_dev;

struct RouteArgs {
  float* x; int64_t ldx;
  const bf16* y; int64_t ldy;
  const float* w_post; const float* w_pre;   // nullable: no norm
  bf16* h; int64_t ldh;
  const bf16* w; ChooseArgs choose;          // w [E][NP]
  int N, NP, rms;
  float eps;
};

constexpr int NW = 16, QUADS = 64 * NW;      // threads of a workgroup

__device__ __forceinline__ float all_sum(float v, float* red) {
  v = vy_wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < NW; ++i) s += red[i];
  return s;
}

// v <- (v - mean) / sqrt(var + eps) over the first N columns (RMS: mean = 0); red: 2 NW floats
template <int CH>
__device__ __forceinline__ void norm(float (&v)[CH][4], const RouteArgs& p, float* red) {
  float mean = 0.f;
  if (!p.rms) {
    float s = 0.f;
#pragma unroll
    for (int c = 0; c < CH; ++c)
#pragma unroll
      for (int e = 0; e < 4; ++e) s += v[c][e];   // (the padding is zero)
    mean = all_sum(s, red) / (float)p.N;
  }
  float q = 0.f;
#pragma unroll
  for (int c = 0; c < CH; ++c)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[c][e] = ((int)threadIdx.x + QUADS * c) * 4 + e < p.N ? v[c][e] - mean : 0.f;
      q += v[c][e] * v[c][e];
    }
  const float ms = all_sum(q, red + NW) / (float)p.N + p.eps, r = rsqrtf(ms), f = r * (1.5f - 0.5f * ms * r * r);
#pragma unroll
  for (int c = 0; c < CH; ++c)
#pragma unroll
    for (int e = 0; e < 4; ++e) v[c][e] *= f;
}

// CH quads of columns per thread, EPL experts per lane of the choice
template <int CH, int EPL>
__global__ __launch_bounds__(64 * NW) void residual_route_kernel(RouteArgs p) {
  constexpr int UE = 4, UK = 4;    // experts and 512-column pieces in flight per wave
  __shared__ __attribute__((aligned(16))) bf16 hs[QUADS * 4 * CH];
  __shared__ float red[4 * NW], logits[64 * EPL], groups[2 * 64 * EPL];
  const int lane = threadIdx.x & 63, t = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int64_t row = blockIdx.x;
  const int E = p.choose.E, K = p.NP;
  const bf16x8 zero8 = {};
  bf16x8 w[UE][UK];
  auto request = [&](int e0, int k0) {
#pragma unroll
    for (int i = 0; i < UE; ++i)
#pragma unroll
      for (int j = 0; j < UK; ++j) {
        const int e = e0 + NW * i, k = k0 + 512 * j + lane * 8;
        w[i][j] = e < E && k < K ? *reinterpret_cast<const bf16x8*>(p.w + (int64_t)e * K + k) : zero8;
      }
  };
  float x[CH][4], y[CH][4];
  float* xr = p.x + row * p.ldx;
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int col = (t + QUADS * c) * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) { x[c][e] = 0.f; y[c][e] = 0.f; }
    if (col < p.NP) {
      const bf16x4 y4 = *reinterpret_cast<const bf16x4*>(p.y + row * p.ldy + col);
      VyChunk<float>::load(xr + col, x[c]);
#pragma unroll
      for (int e = 0; e < 4; ++e) y[c][e] = (float)y4[e];
    }
  }
  request(wave, 0);
  if (p.w_post) norm<CH>(y, p, red);
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int col = (t + QUADS * c) * 4;
    if (col < p.NP) {
      float f[4] = {1.f, 1.f, 1.f, 1.f};
      if (p.w_post) VyChunk<float>::load(p.w_post + col, f);
#pragma unroll
      for (int e = 0; e < 4; ++e) x[c][e] += y[c][e] * f[e];
      VyChunk<float>::store(xr + col, x[c]);
    }
  }
  if (p.w_pre) norm<CH>(x, p, red + 2 * NW);
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int col = (t + QUADS * c) * 4;
    if (col < p.NP) {
      float f[4] = {1.f, 1.f, 1.f, 1.f};
      if (p.w_pre) VyChunk<float>::load(p.w_pre + col, f);
      bf16x4 o;
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = (bf16)(x[c][e] * f[e]);
      *reinterpret_cast<bf16x4*>(hs + col) = o;
      *reinterpret_cast<bf16x4*>(p.h + row * p.ldh + col) = o;
    }
  }
  __syncthreads();
  for (int e0 = wave; e0 < E; e0 += NW * UE) {
    float s[UE] = {};
    for (int k0 = 0; k0 < K; k0 += 512 * UK) {
      if (e0 != wave || k0) request(e0, k0);
#pragma unroll
      for (int j = 0; j < UK; ++j) {
        const int k = k0 + 512 * j + lane * 8;
        const bf16x8 v = k < K ? *reinterpret_cast<const bf16x8*>(hs + k) : zero8;
#pragma unroll
        for (int i = 0; i < UE; ++i) s[i] = vy_rows::dot8(w[i][j], v, s[i]);
      }
    }
#pragma unroll
    for (int i = 0; i < UE; ++i) {
      const float z = vy_wave_sum(s[i]);
      if (lane == 0 && e0 + NW * i < E) logits[e0 + NW * i] = z;
    }
  }
  __syncthreads();
  if (wave) return;
  int id;
  float weight;
  choose_one<EPL>(p.choose, row, logits, lane, groups, id, weight);
  if (lane < p.choose.top) {
    p.choose.ids[row * p.choose.top + lane] = id;
    p.choose.weight[row * p.choose.top + lane] = weight;
  }
}

template <int CH>
void route_go(const RouteArgs& a, int M, hipStream_t st) {
  const dim3 grid((unsigned)M), block(64 * NW);
  if (a.choose.E <= 64) hipLaunchKernelGGL((residual_route_kernel<CH, 1>), grid, block, 0, st, a);
  else if (a.choose.E <= 128) hipLaunchKernelGGL((residual_route_kernel<CH, 2>), grid, block, 0, st, a);
  else hipLaunchKernelGGL((residual_route_kernel<CH, 4>), grid, block, 0, st, a);
}

}  // namespace

// internal (vy_hybrid.hip): norm weights nullable; d checked by vy_moe_few.  VY_ERR_UNSUPPORTED: separate launches take it
int vy_residual_route(float* x, int64_t ldx, const void* y, int64_t ldy, const float* w_post, const float* w_pre, float eps, void* h,
                      int64_t ldh, int64_t M, int64_t N, int64_t NP, int rms, const vy_moe* d, int32_t* ids, float* weight, int dtype,
                      void* stream) {
  if (dtype != VY_BF16 || M < 1 || M > 64 || NP > 2 * QUADS * 4 || NP % 8 || d->experts > 256 || d->width != NP) return VY_ERR_UNSUPPORTED;
  RouteArgs a{x, ldx, (const bf16*)y, ldy, w_post, w_pre, (bf16*)h, ldh, (const bf16*)d->w_router,
              ChooseArgs{nullptr, M, d->experts, d->top, d->groups, d->keep, d->score == VY_SCORE_SIGMOID, d->group_best, d->normalize,
                         d->scale, nullptr, 1, ids, weight, nullptr, nullptr, nullptr},
              (int)N, (int)NP, rms, eps};
  if (NP <= QUADS * 4) route_go<1>(a, (int)M, (hipStream_t)stream);
  else route_go<2>(a, (int)M, (hipStream_t)stream);
  VY_CHECK_LAUNCH("vy_residual_route");
  return VY_OK;
}
