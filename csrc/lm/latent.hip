// Latent attention: the cache holds one row [latent c | rotated key part] per token, shared by all heads.  Head h's key
// is (W_uk,h c, rotated part) and its value W_uv,h c; a learned sink per head joins the softmax's denominator.
//
// latent_prep    after the down projection: norms of both latents, rotation of the key part, cache write.
// latent_decode  bf16, single rows (decode steps, short portions): queries moved into latent space (q W_uk,h), so that a
//                cached row serves as key and value of every head.  One workgroup per (row, 16 or 32 heads, split); half
//                pages of 32 tokens go to two LDS stages by DMA (buffer_load ... lds; its range check zero-fills rows
//                past the context), the next one in flight behind the products of the one before: scores S^T = C Q^T (a
//                wave per 16 keys and 16 heads, Q in registers), O^T = C^T P^T (a wave per quarter of the latent) with P
//                as a bf16 value plus its bf16 remainder.
// latent_rows    any size, fp32 or bf16: one wave per (row, head), plain online softmax.
// latent_gather  cached rows of whole sequences back to back, for the prefill form: long portions expand keys and values
//                per head and run the flash kernel (attn.hip).
#include "lm_device.h"
#include <type_traits>

namespace shai_lm {

typedef short s4v __attribute__((ext_vector_type(4)));
constexpr float kLog2e = 1.4426950408889634f;

// MANY: d is partial sums; they are added once, into LDS.
template <typename T, bool MANY>
__global__ void __launch_bounds__(256) latent_prep_kernel(const LatentPrepArgs p) {
  __shared__ float red[2][4];
  extern __shared__ __attribute__((aligned(16))) float sum[];
  int turn = 0;
  const long t = blockIdx.x;
  const int n = p.qp + p.rp + p.op;
  const float* d = p.d + t * n;
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x * 4; c < p.qp + p.rp + (MANY ? p.op : 0); c += 1024) {
    float4_ v = load4(d + c);
    if constexpr (MANY) {
      for (int i = 1; i < p.parts; i += 3) {
        float4_ e[3];
#pragma unroll
        for (int j = 0; j < 3; ++j) e[j] = load4(d + (long)min(i + j, p.parts - 1) * p.T * n + c);
        v += e[0];
        if (i + 1 < p.parts) v += e[1];
        if (i + 2 < p.parts) v += e[2];
      }
      store4(sum + c, v);
    }
    const float ss = v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
    if (c < p.qp) sq += ss;
    else if (c < p.qp + p.rp) sk += ss;
  }
  if constexpr (MANY) d = sum;                   // complete after the barriers of the sums below
  const float* k = d + p.qp;
  sq = block_sum256(sq, red, turn);
  sk = block_sum256(sk, red, turn);
  const float rq = 1.f / sqrtf(sq / (float)p.q_rank + p.eps), rk = 1.f / sqrtf(sk / (float)p.kv_rank + p.eps);
  T* cq = static_cast<T*>(p.cq) + t * p.qp;
  for (int c = threadIdx.x * 4; c < p.qp; c += 1024) store4(cq + c, load4(d + c) * rq * load4(p.wq + c));
  const int slot = p.slots[t];
  if (slot < 0) return;
  T* row = static_cast<T*>(p.cache) + (long)slot * (p.rp + p.op);
  for (int c = threadIdx.x * 4; c < p.rp; c += 1024) store4(row + c, load4(k + c) * rk * load4(p.wkv + c));
  for (int c = threadIdx.x * 2; c < p.op; c += 512) {
    float u = 0.f, v = 0.f;
    if (c < p.rot) {
      const float cs = p.rope[t * p.rot + c], sn = p.rope[t * p.rot + c + 1];
      const float a = k[p.rp + c], b = k[p.rp + c + 1];
      u = a * cs - b * sn;
      v = b * cs + a * sn;
    }
    store1(row + p.rp + c, u);
    store1(row + p.rp + c + 1, v);
  }
}

void launch_latent_prep(const LatentPrepArgs& a, bool f32, hipStream_t s) {
  const int lds = (a.qp + a.rp + a.op) * 4;
  if (f32 && a.parts > 1) latent_prep_kernel<float, true><<<a.T, 256, lds, s>>>(a);
  else if (f32) latent_prep_kernel<float, false><<<a.T, 256, 0, s>>>(a);
  else if (a.parts > 1) latent_prep_kernel<bf16_t, true><<<a.T, 256, lds, s>>>(a);
  else latent_prep_kernel<bf16_t, false><<<a.T, 256, 0, s>>>(a);
  SHAI_CHECK_LAUNCH();
}

// One workgroup per (page, listed sequence).
__global__ void __launch_bounds__(256) latent_gather_kernel(const LatentGatherArgs p) {
  const int i = blockIdx.y, page = blockIdx.x, n = min(64, p.ctx[i] - page * 64);
  if (n <= 0) return;
  const int per = p.ld_bytes / 16;
  const long src = (long)p.bt[(long)p.seqs[i] * p.max_blocks + page] * 64;
  const uint4_* in = reinterpret_cast<const uint4_*>(static_cast<const char*>(p.cache) + src * p.ld_bytes);
  uint4_* out = reinterpret_cast<uint4_*>(static_cast<char*>(p.out) + ((long)p.start[i] + page * 64) * p.ld_bytes);
  for (int e = threadIdx.x; e < n * per; e += 256) out[e] = in[e];
}

void launch_latent_gather(const LatentGatherArgs& a, hipStream_t s) {
  latent_gather_kernel<<<dim3((a.max_ctx + 63) / 64, a.n), 256, 0, s>>>(a);
  SHAI_CHECK_LAUNCH();
}

// ------------------------------------------------------------------------------------------------ any size
constexpr int kRowsMax = 1024;                   // latent columns: 16 per lane

template <typename T>
__global__ void __launch_bounds__(256) latent_rows_kernel(const LatentArgs p) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int ld = p.rp + p.op;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int e = blockIdx.x, h = blockIdx.y * 4 + w;
  if (h >= p.H) return;                          // whole waves: no barrier below, only wave-local LDS
  float* sq = sm + w * (ld + 64);
  float* sp = sq + ld;
  const T* ql = static_cast<const T*>(p.ql) + ((long)e * p.H + h) * p.rp;
  const T* qr = static_cast<const T*>(p.q) + (long)e * p.ldq + (long)h * p.head + p.np;
  for (int d = lane; d < ld; d += 64)
    sq[d] = d < p.rp ? load1(ql + d) : d < p.rp + p.rot ? load1(qr + d - p.rp) : 0.f;
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  const int last = p.ctx[e] - 1;
  const int* bt = p.bt + (long)(p.seqs ? p.seqs[e] : e) * p.max_blocks;
  float o[kRowsMax / 64];
#pragma unroll
  for (int c = 0; c < kRowsMax / 64; ++c) o[c] = 0.f;
  float m = -INFINITY, l = 0.f;
  for (int kb = 0; kb <= last >> 6; ++kb) {
    const T* page = static_cast<const T*>(p.cache) + (long)bt[kb] * 64 * ld;
    float s = -INFINITY;
    if (kb * 64 + lane <= last) {
      const T* kr = page + (long)lane * ld;
      float acc = 0.f;
      for (int d = 0; d < ld; d += 4) {
        const float4_ k4 = load4(kr + d), q4 = load4(sq + d);
        acc += k4[0] * q4[0] + k4[1] * q4[1] + k4[2] * q4[2] + k4[3] * q4[3];
      }
      s = acc * p.scale;
    }
    const float mn = fmaxf(m, wave_max(s));      // finite: every page holds a visible key
    const float alpha = expf(m - mn), pe = expf(s - mn);
    m = mn;
    l = l * alpha + wave_sum(pe);
    sp[lane] = pe;
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    const int n = min(64, last + 1 - kb * 64);
#pragma unroll
    for (int c = 0; c < kRowsMax / 64; ++c)
      if (64 * c < p.rp) {
        float acc = o[c] * alpha;
        for (int j = 0; j < n; ++j) acc += sp[j] * load1(page + (long)j * ld + lane + 64 * c);
        o[c] = acc;
      }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  }
  const float top = fmaxf(m, p.sink[h]), a = expf(m - top);
  const float inv = a / (l * a + expf(p.sink[h] - top));
  T* out = static_cast<T*>(p.o) + ((long)e * p.H + h) * p.rp;
#pragma unroll
  for (int c = 0; c < kRowsMax / 64; ++c)
    if (64 * c < p.rp) store1(out + lane + 64 * c, o[c] * inv);
}

void launch_latent_rows(const LatentArgs& a, bool f32, hipStream_t s) {
  const dim3 grid(a.n, (a.H + 3) / 4);
  const int lds = 4 * (a.rp + a.op + 64) * 4;
  if (f32) latent_rows_kernel<float><<<grid, 256, lds, s>>>(a);
  else latent_rows_kernel<bf16_t><<<grid, 256, lds, s>>>(a);
  SHAI_CHECK_LAUNCH();
}

// ------------------------------------------------------------------------------------------------ single rows, bf16
template <int CR>
__device__ __forceinline__ int lat_swz(int row, int ch) {      // element offset of 16-byte chunk `ch` of a row
  return row * CR + ((ch ^ (CR % 128 == 0 ? row & 7 : (row >> 1) & 7)) << 3);
}

template <int RP, int OP, int NG>
__global__ void __launch_bounds__(256, 2) latent_decode_kernel(const LatentArgs p) {
  constexpr int CR = RP + OP, KS = CR / 32, CH = CR / 8, ND = RP / 64, NL = 32 * CH / 256;
  static_assert(32 * CH % 256 == 0, "whole DMA instructions per wave");
  extern __shared__ __attribute__((aligned(16))) bf16_t smem[];
  bf16_t* sP = smem + 2 * 32 * CR;               // [value | remainder][16 NG][4][8]
  float* sM = reinterpret_cast<float*>(sP + 2 * 16 * NG * 32);       // [2][16 NG]
  constexpr int PL = 16 * NG * 32;               // elements of one half of sP
  const int tid = threadIdx.x, lane = tid & 63, c = lane & 15, q4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int kt = w & 1, sg = w >> 1;             // this wave's scores: 16 keys, 16 heads
  const bool scores = sg < NG;
  const int e = blockIdx.y, h0 = blockIdx.x * 16 * NG, split = blockIdx.z;
  const int pos = p.ctx[e] - 1, nb = (pos >> 5) + 1;                 // half pages
  const int s0 = (int)((long)split * nb / p.splits), s1 = (int)((long)(split + 1) * nb / p.splits);
  const int* bt = p.bt + (long)(p.seqs ? p.seqs[e] : e) * p.max_blocks;
  const bf16_t* cache = static_cast<const bf16_t*>(p.cache);

  // source offsets of this lane's 16-byte chunks of a half page; the bank swizzle is applied here
  uint32_t off[NL];
#pragma unroll
  for (int i = 0; i < NL; ++i) {
    const int id = (w * NL + i) * 64 + lane, r = id / CH;
    off[i] = (uint32_t)(lat_swz<CR>(r, id % CH) * 2);
  }
  auto stage = [&](int t) {
    const bf16_t* src = cache + ((long)bt[t >> 1] * 64 + (t & 1) * 32) * CR;
    const int rows = min(32, pos + 1 - t * 32);
    const __amdgpu_buffer_rsrc_t r = rsrc(src, rows * CR * 2);
    bf16_t* dst = smem + ((t - s0) & 1) * 32 * CR + w * NL * 512;
#pragma unroll
    for (int i = 0; i < NL; ++i)
      dma16(r, dst + i * 512, off[i]);
  };
  if (s0 < s1) stage(s0);

  // 8 values of head h's query at column k (zero past the rotated part and past the last head)
  auto query = [&](int h, int k) {
    if (h >= p.H) return uint4_{0u, 0u, 0u, 0u};
    if (k < RP) return *reinterpret_cast<const uint4_*>(static_cast<const bf16_t*>(p.ql) + ((long)e * p.H + h) * RP + k);
    if (k - RP < p.rot)                          // the row's pads after the rotated part are zero up to a multiple of 8
      return *reinterpret_cast<const uint4_*>(static_cast<const bf16_t*>(p.q) + (long)e * p.ldq + (long)h * p.head +
                                              p.np + k - RP);
    return uint4_{0u, 0u, 0u, 0u};
  };
  uint4_ qf[KS];
#pragma unroll
  for (int k = 0; k < KS; ++k) qf[k] = query(scores ? h0 + 16 * sg + c : p.H, 32 * k + 8 * q4);

  float4_ o[ND][NG];
  float m[NG], l = 0.f;                          // l: this wave's keys and heads
#pragma unroll
  for (int g = 0; g < NG; ++g) {
    m[g] = -INFINITY;
#pragma unroll
    for (int d = 0; d < ND; ++d) o[d][g] = float4_{0.f, 0.f, 0.f, 0.f};
  }
  const float sl2 = p.scale * kLog2e;
  const int tq = c >> 2, tp = c & 3;

  for (int t = s0; t < s1; ++t) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();                             // this half page is complete, the one before is no longer read
    if (t + 1 < s1) stage(t + 1);
    const bf16_t* sC = smem + ((t - s0) & 1) * 32 * CR;
    float4_ s = float4_{0.f, 0.f, 0.f, 0.f};
    if (scores) {
      float4_ s2 = s;
#pragma unroll
      for (int k = 0; k < KS; k += 2) {
        const bf16x8 k0 = *reinterpret_cast<const bf16x8*>(sC + lat_swz<CR>(16 * kt + c, 4 * k + q4));
        const bf16x8 k1 = *reinterpret_cast<const bf16x8*>(sC + lat_swz<CR>(16 * kt + c, 4 * k + 4 + q4));
        s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0, __builtin_bit_cast(bf16x8, qf[k]), s, 0, 0, 0);
        s2 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k1, __builtin_bit_cast(bf16x8, qf[k + 1]), s2, 0, 0, 0);
      }
      s += s2;
      const int key0 = t * 32 + 16 * kt + 4 * q4;
      float mx = -INFINITY;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[i] = key0 + i > pos ? -INFINITY : s[i] * sl2;
        mx = fmaxf(mx, s[i]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      if (q4 == 0) sM[kt * 16 * NG + 16 * sg + c] = mx;
    }
    __syncthreads();
    float alpha[NG];
#pragma unroll
    for (int g = 0; g < NG; ++g) {
      const float mn = fmaxf(m[g], fmaxf(sM[16 * g + c], sM[16 * NG + 16 * g + c]));
      alpha[g] = __builtin_amdgcn_exp2f(m[g] - mn);             // mn is finite: every half page holds a visible key
      m[g] = mn;
    }
    if (scores) {
      const float mn = NG > 1 && sg > 0 ? m[NG - 1] : m[0], al = NG > 1 && sg > 0 ? alpha[NG - 1] : alpha[0];
      float ls = 0.f;
      typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
      bf16x4 hi, lo;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float x = __builtin_amdgcn_exp2f(s[i] - mn);
        ls += x;
        hi[i] = (__bf16)x;
        lo[i] = (__bf16)(x - (float)hi[i]);
      }
      l = l * al + ls;
      // key 16 kt + 4 q4 + i is k-slot 8 q4 + 4 kt + i of the product with C^T
      bf16_t* dst = sP + ((16 * sg + c) * 4 + q4) * 8 + 4 * kt;
      *reinterpret_cast<bf16x4*>(dst) = hi;
      *reinterpret_cast<bf16x4*>(dst + PL) = lo;
    }
#pragma unroll
    for (int g = 0; g < NG; ++g)
#pragma unroll
      for (int d = 0; d < ND; ++d) o[d][g] *= alpha[g];
    __syncthreads();
    bf16x8 ph[NG], pl[NG];
#pragma unroll
    for (int g = 0; g < NG; ++g) {
      const bf16_t* src = sP + ((16 * g + c) * 4 + q4) * 8;
      ph[g] = *reinterpret_cast<const bf16x8*>(src);
      pl[g] = *reinterpret_cast<const bf16x8*>(src + PL);
    }
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      const int col = w * (RP / 4) + 16 * d + 4 * tp, ch = col >> 3, half = (col >> 2) & 1;
      const bf16_t* a0 = sC + lat_swz<CR>(4 * q4 + tq, ch) + 4 * half;
      const bf16_t* a1 = sC + lat_swz<CR>(4 * q4 + tq + 16, ch) + 4 * half;
      const s4v u0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4v*)(a0));
      const s4v u1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4v*)(a1));
      short8 v;
#pragma unroll
      for (int j = 0; j < 4; ++j) { v[j] = u0[j]; v[4 + j] = u1[j]; }
#pragma unroll
      for (int g = 0; g < NG; ++g) {
        o[d][g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, v), ph[g], o[d][g], 0, 0, 0);
        o[d][g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, v), pl[g], o[d][g], 0, 0, 0);
      }
    }
  }
  // the denominator: over the lanes that share a head, then over the two waves of a head
  __syncthreads();
  if (scores) {
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (q4 == 0) sM[kt * 16 * NG + 16 * sg + c] = l;
  }
  __syncthreads();
#pragma unroll
  for (int g = 0; g < NG; ++g) {
    const int h = h0 + 16 * g + c;
    if (h >= p.H) continue;
    const float L = sM[16 * g + c] + sM[16 * NG + 16 * g + c];
    if (p.splits == 1) {
      const float sk = p.sink[h] * kLog2e, top = fmaxf(m[g], sk), a = __builtin_amdgcn_exp2f(m[g] - top);
      const float inv = a / (L * a + __builtin_amdgcn_exp2f(sk - top));
      bf16_t* out = static_cast<bf16_t*>(p.o) + ((long)e * p.H + h) * RP + w * (RP / 4) + 4 * q4;
#pragma unroll
      for (int d = 0; d < ND; ++d) store4(out + 16 * d, o[d][g] * inv);
    } else {
      float* ws = p.ws + (((long)e * p.H + h) * p.splits + split) * (RP + 4);
#pragma unroll
      for (int d = 0; d < ND; ++d) store4(ws + w * (RP / 4) + 4 * q4 + 16 * d, o[d][g]);
      if (w == 0 && q4 == 0) {
        ws[RP] = m[g];
        ws[RP + 1] = L;
      }
    }
  }
}

__global__ void __launch_bounds__(128) latent_fold_kernel(const LatentArgs p) {
  __shared__ float se[64];
  const int h = blockIdx.x, e = blockIdx.y, tid = threadIdx.x;
  const float* ws = p.ws + ((long)e * p.H + h) * p.splits * (p.rp + 4);
  if (tid < 64) {                                // one lane per split (at most 64)
    const float* q = ws + (long)min(tid, p.splits - 1) * (p.rp + 4) + p.rp;
    const float m = tid < p.splits ? q[0] : -INFINITY, l = q[1], sk = p.sink[h] * kLog2e;
    const float top = fmaxf(wave_max(m), sk);
    const float x = tid < p.splits ? __builtin_amdgcn_exp2f(m - top) : 0.f;
    const float L = wave_sum(l * x) + __builtin_amdgcn_exp2f(sk - top);
    se[tid] = x / L;
  }
  __syncthreads();
  bf16_t* out = static_cast<bf16_t*>(p.o) + ((long)e * p.H + h) * p.rp;
  for (int d = tid * 4; d < p.rp; d += 512) {
    float4_ x = float4_{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < p.splits; ++s) x += load4(ws + (long)s * (p.rp + 4) + d) * se[s];
    store4(out + d, x);
  }
}

bool latent_decode_fits(int rp, int op) { return op == 64 && (rp == 64 || rp == 128 || rp == 256 || rp == 512); }

template <int RP, int NG>
static void decode(const LatentArgs& a, hipStream_t s) {
  constexpr int CR = RP + 64;
  constexpr int lds = (2 * 32 * CR + 2 * 16 * NG * 32) * 2 + 2 * 16 * NG * 4;
  (void)hipFuncSetAttribute(reinterpret_cast<const void*>(latent_decode_kernel<RP, 64, NG>),
                            hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  latent_decode_kernel<RP, 64, NG><<<dim3((a.H + 16 * NG - 1) / (16 * NG), a.n, a.splits), 256, lds, s>>>(a);
  if (a.splits > 1) latent_fold_kernel<<<dim3(a.H, a.n), 128, 0, s>>>(a);
}

void launch_latent_decode(const LatentArgs& a, hipStream_t s) {
  auto go = [&](auto ng) {
    constexpr int NG = decltype(ng)::value;
    if (a.rp == 64) decode<64, NG>(a, s);
    else if (a.rp == 128) decode<128, NG>(a, s);
    else if (a.rp == 256) decode<256, NG>(a, s);
    else decode<512, NG>(a, s);
  };
  if (a.H <= 16) go(std::integral_constant<int, 1>{});
  else go(std::integral_constant<int, 2>{});
  SHAI_CHECK_LAUNCH();
}

}  // namespace shai_lm
