// Linear attention with a matrix state per head whose forget gate also decides what is written (HGRN2):
//   f = l + (1 - l) sigmoid(z + bias),  k = 1 - f,  S = diag(f) S + k v^T,  o = S^T silu(q),  out = o / rms(o) gain.
// S [dk, dv] is fp32 and kept per sequence slot; a sequence's first token starts from zero whatever the slot holds.
//
// rows     row by row, S in registers: decode steps of both formats (bound by the state's traffic) and fp32 prompts.
// chunks   bf16 prompts, 32 rows at a time on the matrix cores.  With b the running sum of log2 f inside a chunk,
//            o_t = sum_{s <= t} v_s sum_d q_t k_s 2^(b_t - b_s) + S^T (q_t 2^b_t),
//            S'  = 2^(b_end) S + sum_s (k_s 2^(b_end - b_s)) v_s^T.
//          Differences of b are never split around a far reference: pairs (s, t) in different 16-row halves meet at the
//          half's border, those in different 8-row blocks of a half at the block's border (both factors at most 1), and
//          those inside a block at its fourth row, where the logarithms, limited to -28 a row, keep the factors below
//          2^112.  (A factor of 2^-28 leaves nothing of a state in fp32.)  Every decayed q and k, the scores and the state
//          enter the products as a bf16 value plus its bf16 remainder; sums are fp32.
//          A wave prepares 32 of the dk channels and their part of the scores, and owns dv / waves columns of S (registers)
//          and of o.
//          A long sequence is cut into segments: totals composes every segment but the last into one step
//          (S -> D S + B), chunks folds the segments before its own.  Only totals pass between workgroups, in two launches.
#include "matrix_state.h"

namespace shai_lm {

// (f, 1 - f) of a forget logit: neither by cancellation
__device__ __forceinline__ void forget(float z, float l, float& f, float& k) {
  const float e = expf(-fabsf(z)), r = 1.f / (1.f + e), hi = r, lo = e * r;
  f = l + (1.f - l) * (z >= 0.f ? hi : lo);
  k = (1.f - l) * (z >= 0.f ? lo : hi);
}

// ------------------------------------------------------------------------------------------------ row by row
// Thread: 4 columns x DK / RG rows of S.
template <typename T, int DK, int DV, int NT>
__global__ void __launch_bounds__(NT) hgrn2_rows_kernel(const Hgrn2Args p) {
  constexpr int NC = DV / 4, RG = NT / NC, R = DK / RG, NW = NT / 64;
  static_assert(R % 4 == 0 && NC <= 64 && NT >= DV && NT >= DK, "shape");
  __shared__ __attribute__((aligned(16))) float sf[DK], sk[DK], sq[DK], sv[DV], so[NW][DV], red[NW];
  const int tid = threadIdx.x, h = blockIdx.x, b = blockIdx.y;
  const int c = (tid % NC) * 4, r0 = (tid / NC) * R;
  const int n = p.q_lens ? p.q_lens[b] : 1;
  if (n < 1) return;
  const long t0 = p.q_start ? p.q_start[b] : b;
  const int slot = p.slots[b];
  float* st = p.state + (((long)max(slot, 0) * p.H + h) * DK + r0) * DV + c;
  const bool old = slot >= 0 && p.pos[t0] > 0;
  float4_ S[R];
#pragma unroll
  for (int i = 0; i < R; ++i) S[i] = old ? load4(st + (long)i * DV) : float4_{0.f, 0.f, 0.f, 0.f};
  const long ldq = (long)p.H * (DK + DV);
  for (long t = t0; t < t0 + n; ++t) {
    const T* row = static_cast<const T*>(p.qv) + t * ldq;
    if (tid < DK) {
      const int d = h * DK + tid;
      float f, k;
      forget(p.z[t * p.H * DK + d] + p.bias[d], p.lower[d], f, k);
      sf[tid] = f;
      sk[tid] = k;
      sq[tid] = silu_exact(load1(row + d));
    }
    if (tid < DV) sv[tid] = load1(row + (long)p.H * DK + h * DV + tid);
    __syncthreads();
    const float4_ v = load4(sv + c);
    float4_ o = float4_{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < R; i += 4) {
      const float4_ f = load4(sf + r0 + i), k = load4(sk + r0 + i), q = load4(sq + r0 + i);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        S[i + j] = f[j] * S[i + j] + k[j] * v;
        o += q[j] * S[i + j];
      }
    }
#pragma unroll
    for (int d = NC; d < 64; d <<= 1)
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] += __shfl_xor(o[j], d, 64);
    if ((tid & 63) < NC) store4(&so[tid >> 6][c], o);
    __syncthreads();
    float y = 0.f;
    if (tid < DV) {
#pragma unroll
      for (int w = 0; w < NW; ++w) y += so[w][tid];
    }
    const float ss = wave_sum(y * y);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    if (tid < DV) {
      float sum = 0.f;
#pragma unroll
      for (int w = 0; w < DV / 64; ++w) sum += red[w];
      store1(static_cast<T*>(p.out) + (t * p.H + h) * DV + tid, y * (1.f / sqrtf(sum / (float)p.vdim + p.eps)) * p.gain[tid]);
    }
  }
  if (slot >= 0) {
#pragma unroll
    for (int i = 0; i < R; ++i) store4(st + (long)i * DV, S[i]);
  }
}

// ------------------------------------------------------------------------------------------------ 32 rows at a time
template <int DK, int DV, bool TOTALS>
__global__ void __launch_bounds__(DK * 2, DK > 128 ? 1 : 2) hgrn2_chunk_kernel(const Hgrn2Args p) {
  constexpr int C = 32, NW = DK / 32, NT = NW * 64, DVW = DV / NW, ND = DVW / 16, NK = DK / 16;
  constexpr int XS = 36, QS = DK + 4, VS = 40;
  constexpr int NV = (DV * 2 + NT - 1) / NT;      // value tasks of a thread: two columns x 8 rows each
  extern __shared__ __attribute__((aligned(16))) uint32_t lds[];
  uint32_t* sx = lds;                             // [NW][32][XS] a wave's decayed rows, then its part of the scores
  uint32_t* sq = sx + (TOTALS ? 0 : NW * C * XS); // [32][QS]     q 2^b
  uint32_t* sk = sq + (TOTALS ? 0 : C * QS);      // [DK][XS]     k 2^(b_end - b), by channel
  bf16_t* sv = reinterpret_cast<bf16_t*>(sk + DK * XS);   // [DV][VS] values by column
  float* sdec = reinterpret_cast<float*>(sv + DV * VS);   // [DK] 2^b_end
  float* red = sdec + DK;                         // [NW][32]
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x, seg = blockIdx.y, b = blockIdx.z;
  const int total = p.q_lens[b];
  if ((long)seg * p.len >= total || (TOTALS && (long)(seg + 1) * p.len >= total)) return;
  const int nseg = (total + p.len - 1) / p.len;
  const int n = min(p.len, total - seg * p.len);
  const long row0 = p.q_start[b] + (long)seg * p.len;
  const int slot = p.slots[b];
  const int g = lane >> 4, c16 = lane & 15;
  const int half = lane >> 5, ch = 32 * w + (lane & 31), d_ch = h * DK + ch;
  const long ldq = (long)p.H * (DK + DV), ldz = (long)p.H * DK;
  const bf16_t* qrow = static_cast<const bf16_t*>(p.qv) + row0 * ldq;
  const float* zrow = p.z + row0 * ldz + d_ch;
  const bf16_t* vrow = qrow + ldz + h * DV;
  const float bias = p.bias[d_ch], lower = p.lower[d_ch];
  constexpr long UNIT = (long)DK * DV + DK;
  float* ws = p.segments > 1 ? p.ws + ((long)b * p.segments * p.H + h) * UNIT : nullptr;   // + segment * H * UNIT

  // S rows 16 i + 4 g .., column 16 d + c16 of the wave's columns
  float4_ S[NK][ND];
  const long col0 = w * DVW + c16;
  auto each = [&](auto&& f) {
#pragma unroll
    for (int i = 0; i < NK; ++i)
#pragma unroll
      for (int d = 0; d < ND; ++d)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          float s = S[i][d][j];
          f(s, (long)(16 * i + 4 * g + j) * DV + col0 + 16 * d, 16 * i + 4 * g + j);
          S[i][d][j] = s;
        }
  };
  const float* st = p.state + ((long)max(slot, 0) * p.H + h) * DK * DV;
  const bool old = slot >= 0 && p.pos[p.q_start[b]] > 0;
  if (TOTALS || nseg == 1) {                      // the first segment's total contains the stored state
    each([&](float& s, long at, int) { s = seg == 0 && old ? st[at] : 0.f; });
    if (TOTALS && seg == 0) {                     // kept for `chunks` (its last segment writes the slot): the last segment's place
      float* keep = ws + (long)(nseg - 1) * p.H * UNIT;
      each([&](float& s, long at, int) { keep[at] = s; });
    }
  } else if (seg == 0) {
    const float* keep = ws + (long)(nseg - 1) * p.H * UNIT;
    each([&](float& s, long at, int) { s = keep[at]; });
  } else {
    each([&](float& s, long at, int) { s = ws[at]; });
    for (int k = 1; k < seg; ++k) {
      const float* B = ws + (long)k * p.H * UNIT;
      const float* D = B + (long)DK * DV;
      each([&](float& s, long at, int row) { s = D[row] * s + B[at]; });
    }
  }
  float log_total = 0.f;                          // TOTALS: of the thread's channel

  // the next chunk's inputs, loaded one chunk ahead
  float zn[16];
  bf16_t qn[16];
  uint32_t vn[NV][8];
  auto fetch = [&](int at) {
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const long t = min(at + 16 * half + i, n - 1);
      zn[i] = zrow[t * ldz];
      if constexpr (!TOTALS) qn[i] = qrow[t * ldq + d_ch];
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int id = min(tid + u * NT, DV * 2 - 1), pair = id % (DV / 2), oct = id / (DV / 2);
#pragma unroll
      for (int i = 0; i < 8; ++i)
        vn[u][i] = *reinterpret_cast<const uint32_t*>(vrow + (long)min(at + 8 * oct + i, n - 1) * ldq + 2 * pair);
    }
  };
  fetch(0);
  for (int at = 0; at < n; at += C) {
    // values by column
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int id = tid + u * NT, pair = id % (DV / 2), oct = id / (DV / 2);
      if (id < DV * 2) {
        uint4_ even, odd;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          even[i] = __builtin_amdgcn_perm(vn[u][2 * i + 1], vn[u][2 * i], 0x05040100u);
          odd[i] = __builtin_amdgcn_perm(vn[u][2 * i + 1], vn[u][2 * i], 0x07060302u);
        }
        *reinterpret_cast<uint4_*>(sv + (2 * pair) * VS + 8 * oct) = even;
        *reinterpret_cast<uint4_*>(sv + (2 * pair + 1) * VS + 8 * oct) = odd;
      }
    }
    // gates of this thread's channel: 16 rows, bl[i] = sum of log2 f inside the half
    float bl[16], k[16], q[16];
    float run = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const bool live = at + 16 * half + i < n;
      const float z = zn[i] + bias;
      const float e = __builtin_amdgcn_exp2f(-fabsf(z) * kInvLn2), r = __builtin_amdgcn_rcpf(1.f + e);
      const float up = z >= 0.f ? r : e * r, down = z >= 0.f ? e * r : r;     // sigmoid(z), sigmoid(-z)
      const float f = lower + (1.f - lower) * up, kk = (1.f - lower) * down;
      const float series = -kk * (1.f + kk * (0.5f + kk * (1.f / 3.f + kk * (0.25f + kk * 0.2f)))) * kInvLn2;
      const float lg = kk < 0.03f ? series : fmaxf(__builtin_amdgcn_logf(f), -28.f);
      run += live ? lg : 0.f;
      bl[i] = run;
      k[i] = live ? kk : 0.f;
      if constexpr (!TOTALS) {
        const float x = bf2f(qn[i]);
        q[i] = live ? x * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-x * kInvLn2)) : 0.f;
      }
    }
    if (at + C < n) fetch(at + C);
    const float mine = run, other = __shfl_xor(run, 32, 64);
    const float tot0 = half ? other : mine, tot1 = half ? mine : other;
    if (half == 0) sdec[ch] = __builtin_amdgcn_exp2f(tot0 + tot1);
    if constexpr (TOTALS) log_total += tot0 + tot1;

    float rest[16];                               // k decayed to the end of the half
#pragma unroll
    for (int i = 0; i < 16; ++i) rest[i] = k[i] * __builtin_amdgcn_exp2f(mine - bl[i]);
    {
      const float tail = half ? 1.f : __builtin_amdgcn_exp2f(tot1);
#pragma unroll
      for (int i = 0; i < 16; i += 4) {
        uint4_ y;
        uint32_t a0, a1, a2, a3;
        pack_pair(rest[i] * tail, rest[i + 1] * tail, a0, a1);
        pack_pair(rest[i + 2] * tail, rest[i + 3] * tail, a2, a3);
        y = uint4_{a0, a1, a2, a3};
        *reinterpret_cast<uint4_*>(sk + ch * XS + 16 * half + i) = y;
      }
    }
    if constexpr (!TOTALS) {
      float from[16];                             // q decayed from the start of the half
#pragma unroll
      for (int i = 0; i < 16; ++i) from[i] = q[i] * __builtin_amdgcn_exp2f(bl[i]);
      {
        const float lead = half ? __builtin_amdgcn_exp2f(tot0) : 1.f;
        uint32_t* dst = sq + (16 * half) * QS + ch;
#pragma unroll
        for (int i = 0; i < 16; i += 2) {
          uint32_t a0, a1;
          pack_pair(from[i] * lead, from[i + 1] * lead, a0, a1);
          dst[i * QS] = a0;
          dst[(i + 1) * QS] = a1;
        }
      }
      // the wave's 32 channels of the scores (rows: keys, columns: queries): halves, blocks, inside blocks
      uint32_t* x = sx + w * C * XS;
      uint32_t* xw = x + 16 * half * XS + (lane & 31);
      auto put = [&](auto&& f) {
#pragma unroll
        for (int i = 0; i < 16; i += 2) {
          uint32_t a0, a1;
          pack_pair(f(i), f(i + 1), a0, a1);
          xw[i * XS] = a0;
          xw[(i + 1) * XS] = a1;
        }
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      };
      auto frag = [&](int tile) {
        const uint32_t* src = x + (16 * tile + c16) * XS + 8 * g;
        return unpack(*reinterpret_cast<const uint4_*>(src), *reinterpret_cast<const uint4_*>(src + 4));
      };
      const float4_ zero = float4_{0.f, 0.f, 0.f, 0.f};
      put([&](int i) { return half ? from[i] : rest[i]; });
      Split f0 = frag(0), f1 = frag(1);
      const float4_ s16 = mac(f0, f1, zero);
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      put([&](int i) {
        const float d = i < 8 ? bl[7] - bl[i] : bl[i] - bl[7];
        return (i < 8 ? k[i] : q[i]) * __builtin_amdgcn_exp2f(d);
      });
      f0 = frag(0);
      f1 = frag(1);
      float4_ diag[2] = {mac(f0, f0, zero), mac(f1, f1, zero)};
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      put([&](int i) { return q[i] * __builtin_amdgcn_exp2f(bl[i] - bl[(i & 8) + 3]); });
      f0 = frag(0);
      f1 = frag(1);
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      put([&](int i) { return k[i] * __builtin_amdgcn_exp2f(bl[(i & 8) + 3] - bl[i]); });
      const float4_ in0 = mac(frag(0), f0, zero), in1 = mac(frag(1), f1, zero);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int key = 4 * g + j;
        const bool block = (key >> 3) == (c16 >> 3), see = key <= c16;
        diag[0][j] = !see ? 0.f : block ? in0[j] : diag[0][j];
        diag[1][j] = !see ? 0.f : block ? in1[j] : diag[1][j];
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      float4_* part = reinterpret_cast<float4_*>(x);
      part[lane] = diag[0];
      part[64 + lane] = s16;
      part[128 + lane] = diag[1];
    }
    __syncthreads();

    bf16x8 vf[ND];                                // values: column 16 d + c16, rows 8 g ..
#pragma unroll
    for (int d = 0; d < ND; ++d)
      vf[d] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4_*>(sv + (col0 + 16 * d) * VS + 8 * g));
    if constexpr (!TOTALS) {
      float4_ s[3] = {};
#pragma unroll
      for (int v = 0; v < NW; ++v) {
        const float4_* part = reinterpret_cast<const float4_*>(sx + v * C * XS);
#pragma unroll
        for (int i = 0; i < 3; ++i) s[i] += part[64 * i + lane];
      }
      const float4_ zero = float4_{0.f, 0.f, 0.f, 0.f};
      const Split pr[2] = {split8(s[0], zero), split8(s[1], s[2])};
      float4_ o[ND][2];
#pragma unroll
      for (int d = 0; d < ND; ++d) {              // rows in the scores' order: 4 g .. of the first half, then of the second
        const bf16_t* src = sv + (col0 + 16 * d) * VS + 4 * g;
        const uint2_ lo = *reinterpret_cast<const uint2_*>(src), hi = *reinterpret_cast<const uint2_*>(src + 16);
        const bf16x8 v = __builtin_bit_cast(bf16x8, uint4_{lo[0], lo[1], hi[0], hi[1]});
#pragma unroll
        for (int u = 0; u < 2; ++u) o[d][u] = mac(v, pr[u].lo, mac(v, pr[u].hi, zero));
      }
#pragma unroll
      for (int i = 0; i < NK; i += 2) {           // channels in the state's order: 4 g .. of two tiles
        Split qf[2];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const uint32_t* src = sq + (16 * u + c16) * QS + 16 * i + 4 * g;
          qf[u] = unpack(*reinterpret_cast<const uint4_*>(src), *reinterpret_cast<const uint4_*>(src + 16));
        }
#pragma unroll
        for (int d = 0; d < ND; ++d) {
          const Split sf = split8(S[i][d], S[i + 1][d]);
#pragma unroll
          for (int u = 0; u < 2; ++u) o[d][u] = mac(sf, qf[u], o[d][u]);
        }
      }
      // o: rows (columns of the head) 16 d + 4 g .., column (query) 16 u + c16
      float ss[2];
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        ss[u] = 0.f;
#pragma unroll
        for (int d = 0; d < ND; ++d)
#pragma unroll
          for (int j = 0; j < 4; ++j) ss[u] += o[d][u][j] * o[d][u][j];
        ss[u] += __shfl_xor(ss[u], 16, 64);
        ss[u] += __shfl_xor(ss[u], 32, 64);
        if (g == 0) red[w * C + 16 * u + c16] = ss[u];
      }
#pragma unroll
      for (int i = 0; i < NK; ++i) {
        const float4_ dec = load4(sdec + 16 * i + 4 * g);
        const uint32_t* src = sk + (16 * i + c16) * XS + 8 * g;
        const Split kf = unpack(*reinterpret_cast<const uint4_*>(src), *reinterpret_cast<const uint4_*>(src + 4));
#pragma unroll
        for (int d = 0; d < ND; ++d) S[i][d] = mac(kf.lo, vf[d], mac(kf.hi, vf[d], S[i][d] * dec));
      }
      __syncthreads();
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const int t = at + 16 * u + c16;
        float sum = 0.f;
#pragma unroll
        for (int v = 0; v < NW; ++v) sum += red[v * C + 16 * u + c16];
        const float r = 1.f / sqrtf(sum / (float)p.vdim + p.eps);
        bf16_t* out = static_cast<bf16_t*>(p.out) + ((row0 + t) * p.H + h) * DV + w * DVW + 4 * g;
        if (t < n) {
#pragma unroll
          for (int d = 0; d < ND; ++d) store4(out + 16 * d, o[d][u] * r * load4(p.gain + w * DVW + 16 * d + 4 * g));
        }
      }
    } else {
#pragma unroll
      for (int i = 0; i < NK; ++i) {
        const float4_ dec = load4(sdec + 16 * i + 4 * g);
        const uint32_t* src = sk + (16 * i + c16) * XS + 8 * g;
        const Split kf = unpack(*reinterpret_cast<const uint4_*>(src), *reinterpret_cast<const uint4_*>(src + 4));
#pragma unroll
        for (int d = 0; d < ND; ++d) S[i][d] = mac(kf.lo, vf[d], mac(kf.hi, vf[d], S[i][d] * dec));
      }
      __syncthreads();
    }
  }
  if constexpr (TOTALS) {
    float* B = ws + (long)seg * p.H * UNIT;
    each([&](float& s, long at, int) { B[at] = s; });
    if (half == 0) B[(long)DK * DV + ch] = __builtin_amdgcn_exp2f(log_total);
  } else if (slot >= 0 && seg == nseg - 1) {
    float* to = p.state + ((long)slot * p.H + h) * DK * DV;
    each([&](float& s, long at, int) { to[at] = s; });
  }
}

template <int DK, int DV, bool TOTALS>
static void chunks(const Hgrn2Args& a, hipStream_t s) {
  constexpr int NW = DK / 32;
  constexpr int lds = 4 * ((TOTALS ? 0 : NW * 32 * 36 + 32 * (DK + 4)) + DK * 36 + DV * 20 + DK + NW * 32);
  (void)hipFuncSetAttribute(reinterpret_cast<const void*>(hgrn2_chunk_kernel<DK, DV, TOTALS>),
                            hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  hgrn2_chunk_kernel<DK, DV, TOTALS><<<dim3(a.H, TOTALS ? a.segments - 1 : a.segments, a.B), NW * 64, lds, s>>>(a);
}

void launch_hgrn2_chunks(const Hgrn2Args& a, hipStream_t s) {
#define GO(DK, DV, TOT) chunks<DK, DV, TOT>(a, s)
  if (a.segments > 1) SHAI_LM_STATE(GO, true);
  SHAI_LM_STATE(GO, false);
#undef GO
  SHAI_CHECK_LAUNCH();
}

void launch_hgrn2_rows(const Hgrn2Args& a, bool f32, hipStream_t s) {
  const dim3 grid(a.H, a.B);
#define GO(DK, DV, T) hgrn2_rows_kernel<T, DK, DV, (DK > 128 ? 1024 : 256)><<<grid, DK > 128 ? 1024 : 256, 0, s>>>(a)
  if (f32) SHAI_LM_STATE(GO, float);
  else SHAI_LM_STATE(GO, bf16_t);
#undef GO
  SHAI_CHECK_LAUNCH();
}

}  // namespace shai_lm
