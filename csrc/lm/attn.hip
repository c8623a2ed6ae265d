// Attention inside fixed-size chunks of the sequence or inside a sliding window, over a paged cache
// ([blocks, G, 64, dk | dv]).
//
// Position i sees the keys lo .. i with lo = i - i % chunk or, with a window, i - chunk + 1; scores are (q . k) * scale,
// softmaxed in fp32, and the output is multiplied by sigmoid of a gate logit per head or per element.  The rows of a step
// are [q | k | v | gate] (one GEMM), or [q | gate] where another layer has written the cache.  Without a gate they are
// [q | k], the values are the keys before their norm and rotation, a head's scores have a factor of their own and its
// denominator a sink.
//
// kv_store      the step's k / v rows into the cache.
// head_prep     the same with q and k rotated by position and divided by their root mean square, or normed with a gain and
//               then rotated (q in place).
// prefill       bf16: flash attention, 4 waves x 32 queries, scores swapped (S^T = K Q^T) so that a lane holds one
//               query's scores; P feeds O^T = V^T P^T from registers as a bf16 pair (value + remainder, 16 significant
//               bits).  Only the 64-key blocks of the chunks that the workgroup's queries lie in are visited.
//               fp32: attn_rows.  The latent form (LAT) is the same kernel on keys and values expanded per head from
//               cached latents: plain causal, no gate, a sink per head in the denominator.
// decode        bf16: one workgroup per (sequence, kv head, split); each wave takes whole 64-key blocks, K straight from
//               memory into the matrix cores (the group's query heads are the 16 columns), fp32 P against V on the
//               VALU; the new token's k / v are written to the cache by the workgroup that reads them.  With rotation
//               and norm of q and k (PREP) every workgroup prepares its query heads in LDS first.
// attn_rows     fp32 (any sizes): one wave per (row, head), plain online softmax.
#include "lm_device.h"

namespace shai_lm {

typedef short s4v __attribute__((ext_vector_type(4)));
constexpr float kLog2e = 1.4426950408889634f;

// the first key that position pos sees
__device__ __forceinline__ int first_key(const AttnArgs& p, int pos) {
  return p.window ? max(0, pos - p.chunk + 1) : pos - pos % p.chunk;
}

template <typename T>
__global__ void __launch_bounds__(256) kv_store_kernel(const AttnArgs p) {
  constexpr int V = 16 / sizeof(T);
  const long t = blockIdx.x;
  const int slot = p.slots[t];
  if (slot < 0) return;
  const T* row = static_cast<const T*>(p.qkvg) + t * p.ld;
  const int blk = slot >> 6, in = slot & 63;
  const int nk = p.G * p.dk / V, nv = p.G * p.dv / V;
  for (int i = threadIdx.x; i < nk + nv; i += 256) {
    const bool isv = i >= nk;
    const int e = (isv ? i - nk : i) * V, d = isv ? p.dv : p.dk, g = e / d;
    T* dst = static_cast<T*>(isv ? p.vc : p.kc) + (((long)blk * p.G + g) * 64 + in) * d + (e - g * d);
    *reinterpret_cast<uint4_*>(dst) = *reinterpret_cast<const uint4_*>(row + (isv ? p.v_off : p.H * p.dk) + e);
  }
}

void launch_kv_store(const AttnArgs& a, bool f32, hipStream_t s) {
  if (f32) kv_store_kernel<float><<<a.T, 256, 0, s>>>(a);
  else kv_store_kernel<bf16_t><<<a.T, 256, 0, s>>>(a);
  SHAI_CHECK_LAUNCH();
}

// 8 consecutive elements
__device__ __forceinline__ void load8(const bf16_t* p, float* x) { unpack8(*reinterpret_cast<const uint4_*>(p), x); }
__device__ __forceinline__ void load8(const float* p, float* x) {
  *reinterpret_cast<float4_*>(x) = load4(p);
  *reinterpret_cast<float4_*>(x + 4) = load4(p + 4);
}
__device__ __forceinline__ void store8(bf16_t* p, const float* x) { *reinterpret_cast<uint4_*>(p) = pack8(x); }
__device__ __forceinline__ void store8(float* p, const float* x) {
  store4(p, *reinterpret_cast<const float4_*>(x));
  store4(p + 4, *reinterpret_cast<const float4_*>(x + 4));
}

// One head by n / 8 lanes of a wave, lane j holding elements 8 j .. 8 j + 7: dimension i < rot / 2 turned with i + rot / 2 by
// the row's angles, then the head divided by its root mean square over `dim` (the pads behind are zero); with `gain` the norm
// comes first.  `stage`: n floats of LDS.  Every lane of the wave calls it.
__device__ __forceinline__ void turn_and_norm(float (&x)[8], float* stage, const float* rope, int rot, int dim, float eps,
                                              int j, int lanes, const float* gain) {
  const int half = rot >> 1;
  if (gain) {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) ss += x[i] * x[i];
    for (int o = lanes >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    const float r = 1.f / sqrtf(ss / (float)dim + eps);
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] *= r * gain[8 * j + i];
  }
  store8(stage + 8 * j, x);
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int e = 8 * j + i;
    if (e < rot) {
      const bool low = e < half;
      const float other = stage[low ? e + half : e - half];
      const float* t = rope + 2 * (low ? e : e - half);
      x[i] = x[i] * t[0] + (low ? -other : other) * t[1];
    }
    ss += x[i] * x[i];
  }
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  if (gain) return;
  for (int o = lanes >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
  const float r = 1.f / sqrtf(ss / (float)dim + eps);
#pragma unroll
  for (int i = 0; i < 8; ++i) x[i] *= r;
}

template <typename T, int DK>
__global__ void __launch_bounds__(256) head_prep_kernel(const AttnArgs p) {
  constexpr int LPH = DK / 8, HP = 256 / LPH;    // lanes per head, heads at a time
  __shared__ __attribute__((aligned(16))) float stage[HP][DK];
  __shared__ __attribute__((aligned(16))) float angle[DK];
  const long t = blockIdx.x;
  const int tid = threadIdx.x, slot = p.slots[t];
  T* row = const_cast<T*>(static_cast<const T*>(p.qkvg)) + t * p.ld;
  for (int i = tid; i < p.rot; i += 256) angle[i] = p.rope[t * p.rot + i];
  __syncthreads();
  const int n = p.H + (p.own_kv && slot >= 0 ? p.G : 0), j = tid % LPH, blk = slot >> 6, in = slot & 63;
  for (int h0 = 0; h0 < n; h0 += HP) {
    const int h = h0 + tid / LPH;
    float x[8];
    load8(row + (long)min(h, n - 1) * DK + 8 * j, x);
    turn_and_norm(x, stage[tid / LPH], angle, p.rot, p.dim, p.eps, j, LPH, h < p.H ? p.q_gain : p.k_gain);
    if (h < p.H) store8(row + (long)h * DK + 8 * j, x);
    else if (h < n) store8(static_cast<T*>(p.kc) + (((long)blk * p.G + h - p.H) * 64 + in) * DK + 8 * j, x);
  }
  if (n == p.H) return;
  const T* v = row + p.v_off;
  for (int i = tid; i < p.G * p.dv / 8; i += 256) {
    const int e = 8 * i, g = e / p.dv;
    float x[8];
    load8(v + e, x);
    store8(static_cast<T*>(p.vc) + (((long)blk * p.G + g) * 64 + in) * p.dv + (e - g * p.dv), x);
  }
}

template <typename T>
static void head_prep(const AttnArgs& a, hipStream_t s) {
  if (a.dk == 64) head_prep_kernel<T, 64><<<a.T, 256, 0, s>>>(a);
  else if (a.dk == 128) head_prep_kernel<T, 128><<<a.T, 256, 0, s>>>(a);
  else head_prep_kernel<T, 256><<<a.T, 256, 0, s>>>(a);
}

void launch_head_prep(const AttnArgs& a, bool f32, hipStream_t s) {
  if (f32) head_prep<float>(a, s);
  else head_prep<bf16_t>(a, s);
  SHAI_CHECK_LAUNCH();
}

// the step's keys and values into the cache (and, with rotation and norm, the queries prepared in place)
static void store_step(const AttnArgs& a, bool f32, hipStream_t s) {
  if (a.rope) launch_head_prep(a, f32, s);
  else if (a.own_kv) launch_kv_store(a, f32, s);
}

// ------------------------------------------------------------------------------------------------ any-size rows
template <typename T>
__global__ void __launch_bounds__(256) attn_rows_kernel(const AttnArgs p) {
  __shared__ float sq[4][256];
  __shared__ float sp[4][64];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int b = blockIdx.z, i = blockIdx.x, h = blockIdx.y * 4 + w;
  const int q_len = p.q_lens ? p.q_lens[b] : 1;
  if (i >= q_len || h >= p.H) return;            // whole waves: no barrier below, only wave-local LDS
  const long t = (p.q_lens ? p.q_start[b] : b) + i;
  const int pos = p.ctx[b] - q_len + i, lo = first_key(p, pos);
  const int g = h / (p.H / p.G);
  const T* row = static_cast<const T*>(p.qkvg) + t * p.ld;
  for (int d = lane; d < p.dk; d += 64) sq[w][d] = load1(row + (long)h * p.dk + d);
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  const float scale = p.scale * (p.temp ? p.temp[h] : 1.f);
  float o[4] = {0.f, 0.f, 0.f, 0.f}, m = -INFINITY, l = 0.f;
  for (int kb = lo >> 6; kb <= pos >> 6; ++kb) {
    const long cell = ((long)p.bt[(long)b * p.max_blocks + kb] * p.G + g) * 64;
    const int key = kb * 64 + lane;
    float s = -INFINITY;
    if (key >= lo && key <= pos) {
      const T* kr = static_cast<const T*>(p.kc) + (cell + lane) * p.dk;
      float acc = 0.f;
      for (int d = 0; d < p.dk; d += 4) {
        const float4_ k4 = load4(kr + d), q4 = load4(&sq[w][d]);
        acc += k4[0] * q4[0] + k4[1] * q4[1] + k4[2] * q4[2] + k4[3] * q4[3];
      }
      s = acc * scale;
    }
    const float mn = fmaxf(m, wave_max(s));      // finite: the first block holds lo, every later one a visible key
    const float alpha = expf(m - mn), e = expf(s - mn);
    m = mn;
    l = l * alpha + wave_sum(e);
    sp[w][lane] = e;
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    const T* vr = static_cast<const T*>(p.vc) + cell * p.dv;
    const int j0 = max(0, lo - kb * 64), j1 = min(63, pos - kb * 64);
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      const int col = lane + 64 * c;
      if (col < p.dv) {
        float acc = o[c] * alpha;
        for (int j = j0; j <= j1; ++j) acc += sp[w][j] * load1(vr + (long)j * p.dv + col);
        o[c] = acc;
      }
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  }
  float up = p.out_scale;
  if (p.sink) {
    const float sk = p.sink[h], top = fmaxf(m, sk), a = expf(m - top);
    l = l * a + expf(sk - top);
    up *= a;
  }
  const T* gate = row + p.gate_off + (long)h * p.gate_w;
  T* out = static_cast<T*>(p.o) + t * p.ldo + (long)h * p.dv;
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    const int col = lane + 64 * c;
    if (col < p.dv) store1(out + col, o[c] * ((p.gate_w ? sigmoid_f(load1(gate + (p.gate_w > 1 ? col : 0))) : up) / l));
  }
}

// ------------------------------------------------------------------------------------------------ prefill (bf16)
template <int D>
__device__ __forceinline__ int k_swz(int row, int ch) {
  if constexpr (D % 128 == 0) return row * D + ((ch ^ (row & 15)) << 3);
  else return row * D + ((ch ^ ((row >> 1) & 7)) << 3);
}
template <int D>
__device__ __forceinline__ int v_swz(int row, int ch) {
  if constexpr (D >= 128) return row * D + ((ch ^ ((row & 3) << 2)) << 3);
  else return row * D + ((ch ^ (((row >> 1) & 1) << 2)) << 3);
}

template <int DK, int DV, bool LAT>
__global__ void __launch_bounds__(256, DK + DV > (LAT ? 320 : 256) ? 1 : 2) attn_prefill_kernel(const AttnArgs p) {
  constexpr int KT = 64, CK = DK / 8, CV = DV / 8, NK = KT * CK / 256, NV = KT * CV / 256;
  constexpr int NS = DK / 16, ND = DV / 32;
  extern __shared__ __attribute__((aligned(16))) bf16_t smem[];
  bf16_t* sK = smem;
  bf16_t* sV = smem + 2 * KT * DK;
  const int tid = threadIdx.x, lane = tid & 63, wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int fr = lane & 31, fh = lane >> 5;
  const int b = blockIdx.z, h = blockIdx.y;
  const int hk = h / (p.H / p.G);
  const int q_len = p.q_lens[b], q0 = blockIdx.x * 128;
  if (q0 >= q_len) return;
  const int ctx = p.ctx[b], c_off = ctx - q_len;
  const int qi = q0 + wid * 32 + fr, pos = qi + c_off, lo = LAT ? 0 : first_key(p, pos);
  const long row0 = p.q_start[b];
  const bf16_t* rows = static_cast<const bf16_t*>(p.qkvg) + row0 * p.ld;

  bf16x8 qf[NS];
  {
    const bf16_t* qp = rows + (long)min(qi, q_len - 1) * p.ld + (long)h * DK;
#pragma unroll
    for (int s = 0; s < NS; ++s)
      qf[s] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4_*>(qp + 16 * s + 8 * fh));
  }
  // blocks from the first query's first key to the last query's position
  const int p_first = q0 + c_off, p_last = min(q0 + 127, q_len - 1) + c_off;
  const int t0 = LAT ? 0 : first_key(p, p_first) >> 6, t1 = (p_last >> 6) + 1;
  const int lo_last = LAT ? 0 : first_key(p, p_last);

  // LAT: keys and values go to LDS by DMA, the bank swizzle applied to the source.  Rows past the context repeat the last
  // one (their scores are masked); columns past a key's parts hold other finite values (the queries are zero there).
  auto stage_tile = [&](int t, int st) {
    if constexpr (LAT) {
      const int ld = p.np + DV;
      const bf16_t* kv = static_cast<const bf16_t*>(p.kv) + ((long)p.kv_start[b] * p.H + h) * ld;
      const bf16_t* lat = static_cast<const bf16_t*>(p.lat) + (long)p.kv_start[b] * p.lat_ld + p.rank;
#pragma unroll
      for (int i = 0; i < NK; ++i) {
        const int id = tid + 256 * i, r = id / CK, col = k_swz<DK>(r, id % CK) - r * DK;
        const long row = min(t * KT + r, ctx - 1);
        const bf16_t* src = col < p.np ? kv + row * p.H * ld + col : lat + row * p.lat_ld + min(col - p.np, p.lat_pad);
        dma16(src, sK + st * KT * DK + (256 * i + 64 * wid) * 8);
      }
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int id = tid + 256 * i, r = id / CV, col = v_swz<DV>(r, id % CV) - r * DV;
        const bf16_t* src = kv + (long)min(t * KT + r, ctx - 1) * p.H * ld + p.np + col;
        dma16(src, sV + st * KT * DV + (256 * i + 64 * wid) * 8);
      }
    }
  };
  uint4_ rk[LAT ? 1 : NK], rv[LAT ? 1 : NV];
  auto load_tile = [&](int t) {
    if constexpr (!LAT) {
      const long cell = ((long)p.bt[(long)b * p.max_blocks + t] * p.G + hk) * 64;
      const bf16_t* kb = static_cast<const bf16_t*>(p.kc) + cell * DK;
      const bf16_t* vb = static_cast<const bf16_t*>(p.vc) + cell * DV;
      const int left = ctx - t * KT;               // rows of this block that hold keys of the sequence
#pragma unroll
      for (int i = 0; i < NK; ++i) {
        const int id = tid + 256 * i;
        rk[i] = id / CK < left ? *reinterpret_cast<const uint4_*>(kb + (long)id * 8) : uint4_{0u, 0u, 0u, 0u};
      }
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int id = tid + 256 * i;
        rv[i] = id / CV < left ? *reinterpret_cast<const uint4_*>(vb + (long)id * 8) : uint4_{0u, 0u, 0u, 0u};
      }
    }
  };
  auto store_tile = [&](int st) {
    if constexpr (!LAT) {
#pragma unroll
      for (int i = 0; i < NK; ++i) {
        const int id = tid + 256 * i;
        *reinterpret_cast<uint4_*>(sK + st * KT * DK + k_swz<DK>(id / CK, id % CK)) = rk[i];
      }
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int id = tid + 256 * i;
        *reinterpret_cast<uint4_*>(sV + st * KT * DV + v_swz<DV>(id / CV, id % CV)) = rv[i];
      }
    }
  };

  float16_ o[ND];
#pragma unroll
  for (int d = 0; d < ND; ++d)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[d][r] = 0.f;
  float m_run = -INFINITY, l_run = 0.f;
  const float sl2 = p.scale * kLog2e * (!LAT && p.temp ? p.temp[h] : 1.f);
  const int g16 = lane >> 4, i16 = lane & 15, tq = i16 >> 2, tp = i16 & 3;

  if constexpr (LAT) {
    stage_tile(t0, 0);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  } else {
    load_tile(t0);
    store_tile(0);
  }
  __syncthreads();
  for (int t = t0; t < t1; ++t) {
    const int cur = (t - t0) & 1;
    if (t + 1 < t1) {
      if constexpr (LAT) stage_tile(t + 1, cur ^ 1);
      else load_tile(t + 1);
    }
    const bf16_t* ks = sK + cur * KT * DK;
    const bf16_t* vs = sV + cur * KT * DV;
    float16_ sacc[2];
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
#pragma unroll
      for (int r = 0; r < 16; ++r) sacc[kb][r] = 0.f;
#pragma unroll
      for (int s = 0; s < NS; ++s) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(ks + k_swz<DK>(kb * 32 + fr, 2 * s + fh));
        sacc[kb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[s], sacc[kb], 0, 0, 0);
      }
    }
    const int key0 = t * KT;
    // scale first (it may be negative or zero), then mask
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int r = 0; r < 16; ++r) sacc[kb][r] *= sl2;
    if (key0 + KT - 1 > p_first || key0 < lo_last) {
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int key = key0 + kb * 32 + (r & 3) + 8 * (r >> 2) + 4 * fh;
          sacc[kb][r] = key > pos || key < lo ? -INFINITY : sacc[kb][r];
        }
    }
    float m4[4] = {-INFINITY, -INFINITY, -INFINITY, -INFINITY};
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int r = 0; r < 16; ++r) m4[r & 3] = fmaxf(m4[r & 3], sacc[kb][r]);
    float mloc = fmaxf(fmaxf(m4[0], m4[1]), fmaxf(m4[2], m4[3]));
    mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
    const float m_new = fmaxf(m_run, mloc);
    const bool grew = __any(m_new > m_run);
    const float m_use = m_new == -INFINITY ? 0.f : m_new;
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_use);
    m_run = m_new;
    float ls4[4] = {0.f, 0.f, 0.f, 0.f};
    bf16x8 pf[2][2], pl[2][2];                   // P as bf16 plus its bf16 remainder: 16 significant bits
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const float e = __builtin_amdgcn_exp2f(sacc[kb][r] - m_use);
        sacc[kb][r] = e;
        ls4[r & 3] += e;
      }
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        bf16x8 v, u;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          v[j] = (__bf16)sacc[kb][8 * s + j];
          u[j] = (__bf16)(sacc[kb][8 * s + j] - (float)v[j]);
        }
        pf[kb][s] = v;
        pl[kb][s] = u;
      }
    }
    l_run = l_run * alpha + ((ls4[0] + ls4[1]) + (ls4[2] + ls4[3]));
    if (grew) {
#pragma unroll
      for (int d = 0; d < ND; ++d)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[d][r] *= alpha;
    }
#pragma unroll
    for (int d = 0; d < ND; ++d) {
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          const int r0 = kb * 32 + 16 * s + 4 * fh + tq;
          const int col = d * 32 + 16 * (g16 & 1) + 4 * tp;
          const int ch = col >> 3, half = (col >> 2) & 1;
          const bf16_t* a0 = vs + v_swz<DV>(r0, ch) + 4 * half;
          const bf16_t* a1 = vs + v_swz<DV>(r0 + 8, ch) + 4 * half;
          const s4v u0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4v*)(a0));
          const s4v u1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4v*)(a1));
          short8 vv;
#pragma unroll
          for (int j = 0; j < 4; ++j) { vv[j] = u0[j]; vv[4 + j] = u1[j]; }
          o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, vv), pf[kb][s], o[d], 0, 0, 0);
          o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, vv), pl[kb][s], o[d], 0, 0, 0);
        }
      }
    }
    if constexpr (LAT) asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    else if (t + 1 < t1) store_tile(cur ^ 1);
    __syncthreads();
  }
  const float l_tot = l_run + __shfl_xor(l_run, 32, 64);
  if (qi < q_len) {
    float inv;
    if (LAT || p.sink) {
      const float sk = p.sink[h] * kLog2e, top = fmaxf(m_run, sk), a = __builtin_amdgcn_exp2f(m_run - top);
      inv = (LAT ? a : a * p.out_scale) / (l_tot * a + __builtin_amdgcn_exp2f(sk - top));
    } else {
      inv = (p.gate_w > 1 ? 1.f : p.gate_w ? sigmoid_f(bf2f(rows[(long)qi * p.ld + p.gate_off + h])) : p.out_scale) / l_tot;
    }
    bf16_t* op = static_cast<bf16_t*>(p.o) + (row0 + qi) * p.ldo + (long)h * DV;
#pragma unroll
    for (int d = 0; d < ND; ++d)
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const int col = d * 32 + 8 * g + 4 * fh;
        float4_ y = float4_{o[d][4 * g], o[d][4 * g + 1], o[d][4 * g + 2], o[d][4 * g + 3]} * inv;
        if constexpr (!LAT) {
          if (p.gate_w > 1) {
            const float4_ z = load4(rows + (long)qi * p.ld + p.gate_off + (long)h * DV + col);
#pragma unroll
            for (int i = 0; i < 4; ++i) y[i] *= sigmoid_f(z[i]);
          }
        }
        store4(op + col, y);
      }
  }
}

template <int DK, int DV, bool LAT = false>
static void prefill(const AttnArgs& a, hipStream_t s) {
  constexpr int lds = 2 * 64 * (DK + DV) * 2;
  (void)hipFuncSetAttribute(reinterpret_cast<const void*>(attn_prefill_kernel<DK, DV, LAT>),
                            hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  attn_prefill_kernel<DK, DV, LAT><<<dim3((a.max_q + 127) / 128, a.H, a.B), 256, lds, s>>>(a);
}

void launch_latent_prefill(const AttnArgs& a, hipStream_t s) {
  if (a.dk == 64 && a.dv == 64) prefill<64, 64, true>(a, s);
  else if (a.dk == 128 && a.dv == 64) prefill<128, 64, true>(a, s);
  else if (a.dk == 128 && a.dv == 128) prefill<128, 128, true>(a, s);
  else if (a.dk == 192 && a.dv == 128) prefill<192, 128, true>(a, s);
  else prefill<256, 256, true>(a, s);
  SHAI_CHECK_LAUNCH();
}

#define SHAI_LM_HEADS(FN, ...)                                      \
  do {                                                              \
    if (a.dk == 64 && a.dv == 64) FN<64, 64>(__VA_ARGS__);          \
    else if (a.dk == 64 && a.dv == 128) FN<64, 128>(__VA_ARGS__);   \
    else if (a.dk == 128 && a.dv == 64) FN<128, 64>(__VA_ARGS__);   \
    else if (a.dk == 128 && a.dv == 128) FN<128, 128>(__VA_ARGS__); \
    else FN<256, 256>(__VA_ARGS__);                                 \
  } while (0)

void launch_attn_prefill(const AttnArgs& a, bool f32, hipStream_t s) {
  if (f32) attn_rows_kernel<float><<<dim3(a.max_q, (a.H + 3) / 4, a.B), 256, 0, s>>>(a);
  else SHAI_LM_HEADS(prefill, a, s);
  SHAI_CHECK_LAUNCH();
}

// ------------------------------------------------------------------------------------------------ decode (bf16)
// what a head's summed output is multiplied by: the denominator L (of exponents to the base 2 above M) with its sink, the gate
__device__ __forceinline__ float out_factor(const AttnArgs& p, const bf16_t* row, int h, int d, float M, float L) {
  float up = p.gate_w ? sigmoid_f(bf2f(row[p.gate_off + (long)h * p.gate_w + (p.gate_w > 1 ? d : 0)])) : p.out_scale;
  if (p.sink) {
    const float sk = p.sink[h] * kLog2e, top = fmaxf(M, sk), a = __builtin_amdgcn_exp2f(M - top);
    L = L * a + __builtin_amdgcn_exp2f(sk - top);
    up *= a;
  }
  return up / L;
}

// One workgroup: kv head g's query heads h0 .. h0 + R - 1 (R <= 16, RH = R rounded up) of sequence b, one split of the
// visible 64-key blocks.  Wave w takes blocks w, w + 4, ... of the split.
template <int DK, int DV, int RH, bool PREP>
__global__ void __launch_bounds__(256) attn_decode_kernel(const AttnArgs p, int per_group, int store) {
  constexpr int LPK = DV / 8, KP = 64 / LPK, IT = 64 / KP;   // V: LPK lanes per key, KP keys at a time
  constexpr int VB = IT > 16 ? 16 : IT;                      // V loads in flight
  __shared__ float sp[4][64][RH];
  __shared__ __attribute__((aligned(16))) float so[4][RH][DV];
  __shared__ __attribute__((aligned(16))) bf16_t sq[PREP ? RH : 1][PREP ? DK : 8];
  static_assert(!PREP || 4 * RH * DV >= (RH + 1) * DK, "prepared heads are staged in so");
  __shared__ float sm[4][16], sl[4][16];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int c = lane & 15, q4 = lane >> 4;
  const int group = p.H / p.G, parts = (group + per_group - 1) / per_group;
  const int g = blockIdx.x / parts, part = blockIdx.x % parts;
  const int b = blockIdx.y, split = blockIdx.z;
  const int h0 = g * group + part * per_group, R = min(per_group, group - part * per_group);
  const int pos = p.ctx[b] - 1, lo = first_key(p, pos);
  const int b0 = lo >> 6, b1 = (pos >> 6) + 1;
  const int per = (b1 - b0 + p.splits - 1) / p.splits;
  const int s0 = b0 + split * per, s1 = min(b1, s0 + per);
  const bf16_t* row = static_cast<const bf16_t*>(p.qkvg) + (long)b * p.ld;
  bf16_t* kc = static_cast<bf16_t*>(p.kc);
  bf16_t* vc = static_cast<bf16_t*>(p.vc);

  // this step's k / v: stored by the only workgroup that reads them (the one with the last block)
  const int slot = p.slots[b];
  if (store && slot >= 0 && s1 == b1 && s0 < s1) {
    const long cell = ((long)(slot >> 6) * p.G + g) * 64 + (slot & 63);
    const bf16_t* kn = row + (long)p.H * DK + (long)g * DK;
    const bf16_t* vn = row + p.v_off + (long)g * DV;
    if (tid < DK / 8) {
      if constexpr (!PREP) reinterpret_cast<uint4_*>(kc + cell * DK)[tid] = reinterpret_cast<const uint4_*>(kn)[tid];
    } else if (tid >= 64 && tid - 64 < DV / 8)
      reinterpret_cast<uint4_*>(vc + cell * DV)[tid - 64] = reinterpret_cast<const uint4_*>(vn)[tid - 64];
  }
  if constexpr (PREP) {                          // the heads of this workgroup, and k where it is stored
    constexpr int LPH = DK / 8, HP = 256 / LPH;
    const bool key = store && slot >= 0 && s1 == b1 && s0 < s1;
    const int n = R + key, j = tid % LPH;
    for (int i0 = 0; i0 < n; i0 += HP) {
      const int i = i0 + tid / LPH, ii = min(i, n - 1);
      float x[8];
      load8(row + (long)(ii < R ? h0 + ii : p.H + g) * DK + 8 * j, x);
      // the spare lanes repeat the last head with the same values
      turn_and_norm(x, &so[0][0][0] + ii * DK, p.rope + (long)b * p.rot, p.rot, p.dim, p.eps, j, LPH,
                    ii < R ? p.q_gain : p.k_gain);
      if (i < R) store8(&sq[i][8 * j], x);
      else if (i < n) store8(kc + (((long)(slot >> 6) * p.G + g) * 64 + (slot & 63)) * DK + 8 * j, x);
    }
  }
  __syncthreads();

  uint4_ qf[DK / 64][2];
#pragma unroll
  for (int s = 0; s < DK / 64; ++s)
#pragma unroll
    for (int u = 0; u < 2; ++u)
      qf[s][u] = c < R ? *reinterpret_cast<const uint4_*>((PREP ? &sq[min(c, RH - 1)][0] : row + (long)(h0 + c) * DK) +
                                                          64 * s + 16 * q4 + 8 * u)
                       : uint4_{0u, 0u, 0u, 0u};
  float o[RH][8];
#pragma unroll
  for (int r = 0; r < RH; ++r)
#pragma unroll
    for (int j = 0; j < 8; ++j) o[r][j] = 0.f;
  float m = -INFINITY, l = 0.f;                  // of head c (replicated over q4)
  const float sl2 = p.scale * kLog2e * (p.temp ? p.temp[h0 + min(c, R - 1)] : 1.f);
  const int vk = lane / LPK, vcol = (lane % LPK) * 8;

  for (int kb = s0 + w; kb < s1; kb += 4) {
    const long cell = ((long)p.bt[(long)b * p.max_blocks + kb] * p.G + g) * 64;
    const bf16_t* kp = kc + (cell + c) * DK + 16 * q4;
    const bf16_t* vp = vc + (cell + vk) * DV + vcol;
    float4_ s[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      s[t] = float4_{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int d = 0; d < DK / 64; ++d)
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const uint4_ kf = *reinterpret_cast<const uint4_*>(kp + (long)16 * t * DK + 64 * d + 8 * u);
          s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, kf),
                                                         __builtin_bit_cast(bf16x8, qf[d][u]), s[t], 0, 0, 0);
        }
    }
    uint4_ v[VB];
#pragma unroll
    for (int i = 0; i < VB; ++i) v[i] = *reinterpret_cast<const uint4_*>(vp + (long)i * KP * DV);
    float mx = -INFINITY;
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int key = kb * 64 + 16 * t + 4 * q4 + i;
        s[t][i] = key < lo || key > pos ? -INFINITY : s[t][i] * sl2;
        mx = fmaxf(mx, s[t][i]);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m, mx);               // finite: every visited block holds a visible key
    const float alpha = __builtin_amdgcn_exp2f(m - mn);
    m = mn;
    float sum = 0.f;
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float e = __builtin_amdgcn_exp2f(s[t][i] - mn);
        sum += e;
        if (c < RH) sp[w][16 * t + 4 * q4 + i][c] = e;
      }
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    l = l * alpha + sum;
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
#pragma unroll
    for (int r = 0; r < RH; ++r) {
      const float ar = __shfl(alpha, r, 64);
#pragma unroll
      for (int j = 0; j < 8; ++j) o[r][j] *= ar;
    }
#pragma unroll
    for (int i0 = 0; i0 < IT; i0 += VB) {
      if (i0 > 0) {
#pragma unroll
        for (int i = 0; i < VB; ++i) v[i] = *reinterpret_cast<const uint4_*>(vp + (long)(i0 + i) * KP * DV);
      }
#pragma unroll
      for (int i = 0; i < VB; ++i) {
        float f[8];
        unpack8(v[i], f);
        const float* pr = &sp[w][(i0 + i) * KP + vk][0];
#pragma unroll
        for (int r = 0; r < RH; ++r) {
          const float pv = pr[r];
#pragma unroll
          for (int j = 0; j < 8; ++j) o[r][j] = fmaf(pv, f[j], o[r][j]);
        }
      }
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  }
  // fold the key lanes of the wave, then the waves
#pragma unroll
  for (int r = 0; r < RH; ++r)
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      float x = o[r][j];
#pragma unroll
      for (int d = LPK; d < 64; d <<= 1) x += __shfl_xor(x, d, 64);
      if (vk == 0) so[w][r][vcol + j] = x;
    }
  if (lane < 16) {
    sm[w][lane] = m;
    sl[w][lane] = l;
  }
  __syncthreads();
  for (int i = tid; i < R * DV; i += 256) {
    const int r = i / DV, d = i - r * DV, h = h0 + r;
    const float M = fmaxf(fmaxf(sm[0][r], sm[1][r]), fmaxf(sm[2][r], sm[3][r]));
    float L = 0.f, x = 0.f;
    if (M > -INFINITY) {
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const float e = __builtin_amdgcn_exp2f(sm[k][r] - M);
        L += sl[k][r] * e;
        x += so[k][r][d] * e;
      }
    }
    if (p.splits == 1) {
      static_cast<bf16_t*>(p.o)[(long)b * p.ldo + h * DV + d] = f2bf(x * out_factor(p, row, h, d, M, L));
    } else {
      float* ws = p.ws + (((long)b * p.H + h) * p.splits + split) * (DV + 2);
      ws[d] = x;
      if (d == 0) {
        ws[DV] = M;
        ws[DV + 1] = L;
      }
    }
  }
}

__global__ void __launch_bounds__(256) attn_decode_fold_kernel(const AttnArgs p) {
  __shared__ float se[64];
  __shared__ float total, top;
  const int h = blockIdx.x, b = blockIdx.y, d = threadIdx.x;
  const float* ws = p.ws + ((long)b * p.H + h) * p.splits * (p.dv + 2);
  if (d < 64) {                                  // one lane per split (at most 64)
    const float* q = ws + (long)min(d, p.splits - 1) * (p.dv + 2) + p.dv;
    const float m = d < p.splits ? q[0] : -INFINITY, l = q[1];
    const float M = wave_max(m);                 // whole wave: every lane takes part in the shuffles
    const float e = d < p.splits ? __builtin_amdgcn_exp2f(m - M) : 0.f;
    se[d] = e;
    const float L = wave_sum(l * e);
    if (d == 0) {
      total = L;
      top = M;
    }
  }
  __syncthreads();
  if (d >= p.dv) return;
  float x = 0.f;
#pragma unroll 8
  for (int s = 0; s < p.splits; ++s) x += ws[(long)s * (p.dv + 2) + d] * se[s];
  static_cast<bf16_t*>(p.o)[(long)b * p.ldo + h * p.dv + d] =
      f2bf(x * out_factor(p, static_cast<const bf16_t*>(p.qkvg) + (long)b * p.ld, h, d, top, total));
}

template <int DK, int DV, bool PREP>
static void decode_heads(const AttnArgs& a, hipStream_t s) {
  const int group = a.H / a.G;
  // heads per workgroup: 16 columns, 8 at the largest head size (LDS); more heads take several workgroups
  constexpr int MAXR = DV > 128 ? 8 : 16;
  const int per = group < MAXR ? group : MAXR, parts = (group + per - 1) / per;
  const dim3 grid(a.G * parts, a.B, a.splits);
  const int store = parts == 1 && a.own_kv;
  if (per == 1) attn_decode_kernel<DK, DV, 1, PREP><<<grid, 256, 0, s>>>(a, per, store);
  else if (per <= 4) attn_decode_kernel<DK, DV, 4, PREP><<<grid, 256, 0, s>>>(a, per, store);
  else if (per <= 8) attn_decode_kernel<DK, DV, 8, PREP><<<grid, 256, 0, s>>>(a, per, store);
  else if constexpr (DV <= 128) attn_decode_kernel<DK, DV, 16, PREP><<<grid, 256, 0, s>>>(a, per, store);
  if (a.splits > 1) attn_decode_fold_kernel<<<dim3(a.H, a.B), 256, 0, s>>>(a);
}

template <int DK, int DV>
static void decode(const AttnArgs& a, hipStream_t s) {
  if (a.H / a.G > (DV > 128 ? 8 : 16)) {         // no single workgroup reads the new row: its own launch
    store_step(a, false, s);
    decode_heads<DK, DV, false>(a, s);
  } else if (a.rope) {
    decode_heads<DK, DV, true>(a, s);
  } else {
    decode_heads<DK, DV, false>(a, s);
  }
}

void launch_attn_decode(const AttnArgs& a, bool f32, hipStream_t s) {
  if (f32) {
    store_step(a, true, s);
    attn_rows_kernel<float><<<dim3(1, (a.H + 3) / 4, a.B), 256, 0, s>>>(a);
  } else {
    SHAI_LM_HEADS(decode, a, s);
  }
  SHAI_CHECK_LAUNCH();
}

}  // namespace shai_lm
