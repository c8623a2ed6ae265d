// Mixture-of-experts routing: group-limited top-k of softmax scores (weights: those scores, or a softmax over the chosen
// logits only), and the sort of (token, k) pairs by expert.
#include "lm_device.h"
#include "lm.h"

namespace shai_lm {

// max over the wave by lane shifts inside the register file (rows of 16, then the two row broadcasts)
template <int CTRL>
__device__ __forceinline__ float dpp_max(float v) {
  const int neg_inf = 0xff800000;
  const int o = __builtin_amdgcn_update_dpp(neg_inf, __float_as_int(v), CTRL, 0xf, 0xf, false);
  return fmaxf(v, __int_as_float(o));
}
__device__ __forceinline__ float wave_max_dpp(float v) {
  v = dpp_max<0x111>(v);   // row_shr 1, 2, 4, 8
  v = dpp_max<0x112>(v);
  v = dpp_max<0x114>(v);
  v = dpp_max<0x118>(v);
  v = dpp_max<0x142>(v);   // row_bcast 15, 31
  v = dpp_max<0x143>(v);
  return __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), 63));
}

// One wave per token; lane l holds experts l, l + 64, ...  All comparisons break ties by the lower expert index, and
// picks are by a strictly decreasing (score, index) order, so every pick is a distinct expert whatever the scores are.
// `sc` is the wave's LDS scratch, [E + groups] floats.  Every wave of the workgroup calls it (barriers inside).
template <int NE>
__device__ __forceinline__ void route_token(const RouteArgs& p, int t, float* sc) {
  const int lane = threadIdx.x & 63;
  float* gs = sc + p.E;
  const bool live = t < p.T;
  float z[NE];
  float m = -INFINITY;
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    z[i] = live && e < p.E ? p.logits[(long)t * p.E + e] + (p.bias ? p.bias[e] : 0.f) : -INFINITY;
    if (!(z[i] == z[i])) z[i] = -INFINITY;      // a padding row may carry NaN: it still needs valid picks
    if (p.renorm && e < p.E) z[i] = fmaxf(z[i], -3e38f);
    m = fmaxf(m, z[i]);
  }
  m = wave_max_dpp(m);
  if (m == -INFINITY) m = 0.f;
  if (!p.renorm) {                               // scores: softmax over all experts (else the logits themselves)
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      z[i] = expf(z[i] - m);
      sum += lane + 64 * i < p.E ? z[i] : 0.f;
    }
    sum = wave_sum(sum);
    const float inv = sum > 0.f ? 1.f / sum : 0.f;
#pragma unroll
    for (int i = 0; i < NE; ++i) z[i] *= inv;
  }
#pragma unroll
  for (int i = 0; i < NE; ++i)
    if (lane + 64 * i < p.E) sc[lane + 64 * i] = z[i];
  __syncthreads();
  const int per = p.E / p.groups;
  for (int g = lane; g < p.groups; g += 64) {
    float b = -INFINITY;
    for (int j = 0; j < per; ++j) b = fmaxf(b, sc[g * per + j]);
    gs[g] = b;
  }
  __syncthreads();
  // a group is kept when fewer than `keep` groups beat it
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    if (e < p.E && p.keep < p.groups) {
      const int g = e / per;
      const float mine = gs[g];
      int better = 0;
      for (int j = 0; j < p.groups; ++j) better += gs[j] > mine || (gs[j] == mine && j < g);
      if (better >= p.keep) z[i] = -INFINITY;
    }
    if (e >= p.E) z[i] = -INFINITY;
  }
  float mine = -INFINITY;                        // renorm: lane k's pick
  for (int k = 0; k < p.top; ++k) {
    float best = -INFINITY;
    int bi = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = lane + 64 * i;
      if (z[i] > best) { best = z[i]; bi = e; } // ascending e: the first of equal scores stays
    }
    const float bv = wave_max_dpp(best);
    const unsigned long long who = __ballot(best == bv);
    if (__popcll(who) == 1) {
      bi = __builtin_amdgcn_readlane(bi, __ffsll(who) - 1);
    } else {                                      // equal scores in several lanes: the lowest expert
      if (best != bv) bi = 0x7fffffff;
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) bi = min(bi, __shfl_xor(bi, o, 64));
    }
#pragma unroll
    for (int i = 0; i < NE; ++i)
      if (lane + 64 * i == bi) z[i] = -INFINITY;
    if (lane == k) mine = bv;
    if (live && lane == 0) {
      p.ids[(long)t * p.top + k] = bi;
      if (!p.renorm) p.wts[(long)t * p.top + k] = bv;
    }
  }
  if (p.renorm) {
    const float e = lane < p.top ? expf(mine - m) : 0.f, sum = wave_sum(e);
    if (live && lane < p.top) p.wts[(long)t * p.top + lane] = e / sum;
  }
}

template <int NE>
__global__ void __launch_bounds__(256) route_kernel(const RouteArgs p) {
  extern __shared__ float sh[];
  const int wid = threadIdx.x >> 6;
  route_token<NE>(p, blockIdx.x * 4 + wid, sh + wid * (p.E + p.groups));
}

void launch_route(const RouteArgs& a, hipStream_t s) {
  const int grid = (a.T + 3) / 4;
  const size_t lds = sizeof(float) * 4 * (a.E + a.groups);
  if (a.E <= 64) route_kernel<1><<<grid, 256, lds, s>>>(a);
  else if (a.E <= 128) route_kernel<2><<<grid, 256, lds, s>>>(a);
  else if (a.E <= 256) route_kernel<4><<<grid, 256, lds, s>>>(a);
  else route_kernel<16><<<grid, 256, lds, s>>>(a);
  SHAI_CHECK_LAUNCH();
}

// One workgroup: LDS histogram, scan, tile list, scatter.  The order of rows inside an expert is arbitrary (each row is
// computed alone, and the combine reads a token's slots in k order), so LDS atomics are enough.
__device__ __forceinline__ void plan_body(const PlanArgs& p, int* cnt, int* start, int* tile0) {
  const int tid = threadIdx.x;
  const int4* ids4 = reinterpret_cast<const int4*>(p.ids);
  const int n4 = p.P / 4;
  for (int e = tid; e < p.E; e += 1024) cnt[e] = 0;
  __syncthreads();
#pragma unroll 4
  for (int i = tid; i < n4; i += 1024) {
    const int4 v = ids4[i];
    atomicAdd(&cnt[v.x], 1);
    atomicAdd(&cnt[v.y], 1);
    atomicAdd(&cnt[v.z], 1);
    atomicAdd(&cnt[v.w], 1);
  }
  for (int i = 4 * n4 + tid; i < p.P; i += 1024) atomicAdd(&cnt[p.ids[i]], 1);
  __syncthreads();
  if (tid < 64) {                                // wave 0: exclusive scans of the counts and of the tile counts
    int base = 0, tbase = 0;
    for (int e0 = 0; e0 < p.E; e0 += 64) {
      const int e = e0 + tid;
      const int c = e < p.E ? cnt[e] : 0;
      const int n = (c + p.bm - 1) / p.bm;
      int a = c, b = n;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int ua = __shfl_up(a, o, 64), ub = __shfl_up(b, o, 64);
        if (tid >= o) { a += ua; b += ub; }
      }
      if (e < p.E) {
        start[e] = base + a - c;
        tile0[e] = tbase + b - n;
      }
      base += __shfl(a, 63, 64);
      tbase += __shfl(b, 63, 64);
    }
    if (tid == 0) {
      start[p.E] = base;
      tile0[p.E] = tbase;
    }
  }
  __syncthreads();
  for (int e = tid; e <= p.E; e += 1024) p.offsets[e] = start[e];
  for (int e = tid; e < p.E; e += 1024) {
    const int n = tile0[e + 1] - tile0[e];
    for (int j = 0; j < n; ++j) {
      p.tiles[2 * (tile0[e] + j)] = e;
      p.tiles[2 * (tile0[e] + j) + 1] = start[e] + j * p.bm;
    }
  }
  for (int i = tile0[p.E] + tid; i < p.n_tiles; i += 1024) {
    p.tiles[2 * i] = -1;
    p.tiles[2 * i + 1] = 0;
  }
  __syncthreads();
  for (int e = tid; e < p.E; e += 1024) cnt[e] = start[e];
  __syncthreads();
  auto place = [&](int i, int e) {
    const int s = atomicAdd(&cnt[e], 1);
    p.token_of[s] = i / p.top;
    p.slot_of[i] = s;
  };
#pragma unroll 4
  for (int i = tid; i < n4; i += 1024) {
    const int4 v = ids4[i];
    place(4 * i, v.x);
    place(4 * i + 1, v.y);
    place(4 * i + 2, v.z);
    place(4 * i + 3, v.w);
  }
  for (int i = 4 * n4 + tid; i < p.P; i += 1024) place(i, p.ids[i]);
}

__global__ void __launch_bounds__(1024) plan_kernel(const PlanArgs p) {
  __shared__ int cnt[1024], start[1025], tile0[1025];
  plan_body(p, cnt, start, tile0);
}

void launch_plan(const PlanArgs& a, hipStream_t s) {
  plan_kernel<<<1, 1024, 0, s>>>(a);
  SHAI_CHECK_LAUNCH();
}

// A decode step's few tokens: one wave routes each, then the same workgroup sorts the picks (they pass through global
// memory inside the workgroup: written before the barrier, read after it).
template <int NE>
__global__ void __launch_bounds__(1024) route_plan_kernel(const RouteArgs r, const PlanArgs p) {
  __shared__ int cnt[256], start[257], tile0[257];
  extern __shared__ float sh[];
  const int wid = threadIdx.x >> 6;
  route_token<NE>(r, wid, sh + wid * (r.E + r.groups));
  __syncthreads();
  plan_body(p, cnt, start, tile0);
}

void launch_route_plan(const RouteArgs& r, const PlanArgs& a, hipStream_t s) {
  const size_t lds = sizeof(float) * 16 * (r.E + r.groups);
  if (r.E <= 64) route_plan_kernel<1><<<1, 1024, lds, s>>>(r, a);
  else if (r.E <= 128) route_plan_kernel<2><<<1, 1024, lds, s>>>(r, a);
  else route_plan_kernel<4><<<1, 1024, lds, s>>>(r, a);
  SHAI_CHECK_LAUNCH();
}

}  // namespace shai_lm
