// Linear attention with a matrix state S [dk, dv] per head that is written by the delta rule,
//   S = diag(g) S,  u = b (v - S^T k),  S = S + k u^T,  o = S^T q,
// with a decay g per head or per key channel, or that only decays by a fixed factor (retention: S = g S + k v^T).  The inputs
// of the delta rule pass a short causal convolution and silu, its q and k are unit vectors; retention's q and k are rotated.
// out = o / rms(o) gain act(gate).  S is fp32 and kept per sequence slot; a sequence's first token starts from zero whatever the
// slot holds.  The convolutions' last inputs lie in a ring per slot, each at its position modulo the taps, so that a decode step
// reads the older ones while it writes its own.
//
// rows     row by row, S in registers, convolution to gate in one launch: decode steps of both formats (bound by the state's
//          traffic) and fp32 prompts.
// chunks   bf16 prompts in chunks of 32 rows, two launches.  With B_t the product of the decays up to row t of a chunk,
//            A[t, s] = b_t sum_d k_t k_s B_t / B_s (s < t),   P[t, s] = sum_d q_t k_s B_t / B_s (s <= t),
//            U = (I + A)^-1 diag(b) (V - (B K) S),   O = (B Q) S + P U,   S' = B_end S + (K B_end / B)^T U.
//          prep (a workgroup per chunk and head, all at once): convolution, norms, decays, the two score matrices, the inverse,
//          and every operand of the second launch in the order its lanes load it.
//          scan (a workgroup per sequence and head): chunk after chunk, each wave its columns of S (registers); operands are
//          loaded one chunk ahead, straight into registers.
//          Quotients of decays come from differences of running logarithms.  A decay per channel enters the matrix products
//          through a reference row that lies between the two rows (the end of a 16-row half or of an 8-row block), so both
//          factors are at most 1; rows of one 8-row block are multiplied out one by one in fp32.  Operands of matrix products
//          are a bf16 value plus its bf16 remainder; sums are fp32.
#include "matrix_state.h"

namespace shai_lm {

constexpr int kRetention = 0, kHead = 1, kChannel = 2;     // decay: fixed; per head; per key channel
constexpr float kLeast = -40.f;                            // base-2 logarithm of a decay that leaves nothing in fp32

__device__ __forceinline__ float softplus_exact(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
// base-2 logarithm of exp(-rate softplus(x))
__device__ __forceinline__ float log_decay(float x, float rate) {
  const float e = __builtin_amdgcn_exp2f(-fabsf(x) * kInvLn2);
  const float series = e * (1.f - e * (0.5f - e * (1.f / 3.f - e * (0.25f - e * 0.2f)))) * kInvLn2;
  const float sp = fmaxf(x, 0.f) * kInvLn2 + (e < 0.03f ? series : __builtin_amdgcn_logf(1.f + e));
  return fmaxf(-rate * sp, kLeast);
}
template <bool FAST>
__device__ __forceinline__ float gate_act(float z, int kind) {
  const float s = FAST ? __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-z * kInvLn2)) : sigmoid_f(z);
  return kind == 0 ? z * s : s;
}

// ------------------------------------------------------------------------------------------------ row by row
// Thread: 4 columns x DK / RG rows of S.  S^T k and S^T q are taken from the decayed state in one pass: with kq = k . q,
// o = S^T q + kq u.
template <typename T, int MODE, int DK, int DV, int NT>
__global__ void __launch_bounds__(NT) rule_rows_kernel(const RuleArgs p) {
  constexpr bool DELTA = MODE != kRetention;
  constexpr int NC = DV / 4, RG = NT / NC, R = DK / RG, NW = NT / 64, KW = DK / 64;
  static_assert(R % 4 == 0 && NC <= 64 && NT >= DV && NT >= 2 * DK, "shape");
  __shared__ __attribute__((aligned(16))) float sq[DK], sk[DK], sg[MODE == kChannel ? DK : 4], sv[DV];
  __shared__ __attribute__((aligned(16))) float sa[DELTA ? NW : 1][DV], so[NW][DV];
  __shared__ float red[NW], skq[NW], rout[NW];
  const int tid = threadIdx.x, h = blockIdx.x, b = blockIdx.y;
  const int c = (tid % NC) * 4, r0 = (tid / NC) * R;
  const int n = p.q_lens ? p.q_lens[b] : 1;
  if (n < 1) return;
  const long t0 = p.q_start ? p.q_start[b] : b;
  const int slot = p.slots[b], pos0 = p.pos[t0];
  const int g = h / (p.H / p.G), channels = 2 * p.G * DK + p.H * DV;
  float* st = p.state + (((long)max(slot, 0) * p.H + h) * DK + r0) * DV + c;
  const bool old = slot >= 0 && pos0 > 0;
  float4_ S[R];
#pragma unroll
  for (int i = 0; i < R; ++i) S[i] = old ? load4(st + (long)i * DV) : float4_{0.f, 0.f, 0.f, 0.f};
  const T* x = static_cast<const T*>(p.x);
  T* ring = DELTA ? static_cast<T*>(p.ring) + (long)max(slot, 0) * p.taps * channels : nullptr;
  // channel ch of row t after its convolution and silu
  auto conv = [&](long t, int ch) {
    float y = p.conv[(long)(p.taps - 1) * channels + ch] * load1(x + t * p.ldx + ch);
#pragma unroll 4
    for (int j = 1; j < p.taps; ++j) {
      const int at = pos0 + (int)(t - t0) - j;               // its position
      const bool here = t - j >= t0;
      const T* src = here ? x + (t - j) * p.ldx + ch : ring + (long)(max(at, 0) % p.taps) * channels + ch;
      if (here || (at >= 0 && slot >= 0)) y += p.conv[(long)(p.taps - 1 - j) * channels + ch] * load1(src);
    }
    return silu_exact(y);
  };
  for (long t = t0; t < t0 + n; ++t) {
    const T* row = x + t * p.ldx;
    float mine = 0.f;
    if (tid < 2 * DK) {
      const bool key = tid >= DK;
      const int d = key ? tid - DK : tid, first = DELTA ? (key ? p.G + g : g) * DK : (key ? p.H + h : h) * DK;
      if constexpr (DELTA) {
        mine = conv(t, first + d);
      } else {
        mine = load1(row + first + d);
        if (d < p.rot) {
          const int half = p.rot >> 1;
          const bool low = d < half;
          const float other = load1(row + first + (low ? d + half : d - half));
          const float* a = p.rope + t * p.rot + 2 * (low ? d : d - half);
          mine = mine * a[0] + (low ? -other : other) * a[1];
        }
      }
      (key ? sk : sq)[d] = mine;
    }
    if constexpr (DELTA) {
      const float ss = wave_sum(mine * mine);
      if ((tid & 63) == 0) red[tid >> 6] = ss;
    }
    const int v0 = (DELTA ? 2 * p.G * DK : 2 * p.H * DK) + h * DV;
    if (tid < DV) sv[tid] = DELTA ? conv(t, v0 + tid) : load1(row + v0 + tid);
    if constexpr (MODE == kChannel) {
      if (tid < DK) {
        const int d = h * DK + tid;
        sg[tid] = expf(-p.rate[h] * softplus_exact(p.decay[t * p.ldd + d] + p.bias[d]));
      }
    }
    __syncthreads();
    float rq = 1.f, rk = rsqrtf((float)p.dim), gh = MODE == kRetention ? p.rate[h] : 1.f, beta = 1.f;
    if constexpr (DELTA) {
      float s0 = 0.f, s1 = 0.f;
#pragma unroll
      for (int w = 0; w < KW; ++w) {
        s0 += red[w];
        s1 += red[KW + w];
      }
      rq = 1.f / sqrtf(s0 + 1e-6f) * (1.f / sqrtf((float)p.dim));
      rk = 1.f / sqrtf(s1 + 1e-6f);
      beta = sigmoid_f(p.beta[t * p.ldb + h]);
      if constexpr (MODE == kHead) gh = expf(-p.rate[h] * softplus_exact(p.decay[t * p.ldd + h] + p.bias[h]));
    } else {
      rk = 1.f / sqrtf((float)p.dim);
    }
    const float4_ v = load4(sv + c);
    float4_ a = float4_{0.f, 0.f, 0.f, 0.f}, o = a;
    float kq = 0.f;
#pragma unroll
    for (int i = 0; i < R; i += 4) {
      const float4_ k = load4(sk + r0 + i) * rk, q = load4(sq + r0 + i) * rq;
      const float4_ f = MODE == kChannel ? load4(sg + r0 + i) : float4_{gh, gh, gh, gh};
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        S[i + j] = f[j] * S[i + j];
        if constexpr (DELTA) {
          a += k[j] * S[i + j];
          kq += k[j] * q[j];
        } else {
          S[i + j] += k[j] * v;
        }
        o += q[j] * S[i + j];
      }
    }
#pragma unroll
    for (int d = NC; d < 64; d <<= 1) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        if constexpr (DELTA) a[j] += __shfl_xor(a[j], d, 64);
        o[j] += __shfl_xor(o[j], d, 64);
      }
      if constexpr (DELTA) kq += __shfl_xor(kq, d, 64);
    }
    if ((tid & 63) < NC) {
      if constexpr (DELTA) store4(&sa[tid >> 6][c], a);
      store4(&so[tid >> 6][c], o);
    }
    if (DELTA && (tid & 63) == 0) skq[tid >> 6] = kq;
    __syncthreads();
    float y = 0.f;
    if (tid < DV) {
#pragma unroll
      for (int w = 0; w < NW; ++w) y += so[w][tid];
    }
    if constexpr (DELTA) {
      float4_ sum = float4_{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int w = 0; w < NW; ++w) sum += load4(&sa[w][c]);
      const float4_ u = beta * (v - sum);
#pragma unroll
      for (int i = 0; i < R; i += 4) {
        const float4_ k = load4(sk + r0 + i) * rk;
#pragma unroll
        for (int j = 0; j < 4; ++j) S[i + j] += k[j] * u;
      }
      if (tid < DV) {
        float all = 0.f, s = 0.f;
#pragma unroll
        for (int w = 0; w < NW; ++w) {
          all += skq[w];
          s += sa[w][tid];
        }
        y += all * beta * (sv[tid] - s);
      }
    }
    const float ss = wave_sum(y * y);
    if ((tid & 63) == 0) rout[tid >> 6] = ss;
    __syncthreads();
    if (tid < DV) {
      float sum = 0.f;
#pragma unroll
      for (int w = 0; w < DV / 64; ++w) sum += rout[w];
      const float z = load1(static_cast<const T*>(p.gate) + t * p.ldg + h * DV + tid);
      const float r = 1.f / sqrtf(sum / (float)p.vdim + p.eps);
      store1(static_cast<T*>(p.out) + t * p.ldo + h * DV + tid, y * r * (DELTA ? p.gain[tid] : 1.f) * gate_act<false>(z, p.gate_kind));
    }
  }
  if (slot >= 0) {
#pragma unroll
    for (int i = 0; i < R; ++i) store4(st + (long)i * DV, S[i]);
    if (DELTA && !p.q_lens) {                     // this step's inputs, where no workgroup of the step reads
      T* to = ring + (long)(pos0 % p.taps) * channels;
      const T* row = x + t0 * p.ldx;
      if (tid < 2 * DK && h % (p.H / p.G) == 0) {
        const int ch = (tid >= DK ? p.G + g : g) * DK + (tid >= DK ? tid - DK : tid);
        to[ch] = row[ch];
      }
      const int ch = 2 * p.G * DK + h * DV + tid;
      if (tid < DV) to[ch] = row[ch];
    }
  }
}

// the last inputs of a prefill step into the rings (after every workgroup has read the older ones)
template <typename T>
__global__ void __launch_bounds__(256) ring_commit_kernel(const RingArgs p) {
  const int b = blockIdx.y, ch = blockIdx.x * 256 + threadIdx.x;
  const int slot = p.slots[b], n = p.q_lens[b];
  if (slot < 0 || slot >= p.n_slots || ch >= p.channels) return;
  const long t0 = p.q_start[b];
  T* ring = static_cast<T*>(p.ring) + (long)slot * p.taps * p.channels + ch;
  const T* x = static_cast<const T*>(p.x) + ch;
  for (int t = max(0, n - p.taps); t < n; ++t)
    ring[(long)((p.pos[t0] + t) % p.taps) * p.channels] = x[(t0 + t) * p.ldx];
}

void launch_ring_commit(const RingArgs& a, bool f32, hipStream_t s) {
  const dim3 grid((a.channels + 255) / 256, a.B);
  if (f32) ring_commit_kernel<float><<<grid, 256, 0, s>>>(a);
  else ring_commit_kernel<bf16_t><<<grid, 256, 0, s>>>(a);
  SHAI_CHECK_LAUNCH();
}

// ------------------------------------------------------------------------------------------------ 32 rows at a time
constexpr int kC = 32;
// A prepared chunk of one head, in 16-byte units: fragments are [64 lanes] of 16 bytes, values and remainders one after the
// other.  Row operands (time x channels, u: rows 16 u ..): a lane holds channels 32 i + 4 g .. and 32 i + 16 + 4 g .. of its row;
// column operands (channels x time) and score operands (time x time): times 4 g .. and 16 + 4 g ...
template <int DK, int DV>
struct Unit {
  static constexpr int NI = DK / 32, NK = DK / 16, ND = DV / 16;
  static constexpr int kd = 0;                               // B K     [u 2][i NI][2][64]
  static constexpr int qd = kd + 2 * NI * 128;               // B Q     the same
  static constexpr int ke = qd + 2 * NI * 128;               // K B_end / B  [i NK][2][64]
  static constexpr int tf = ke + NK * 128;                   // (I + A)^-1 diag(b)  [u 2][2][64]
  static constexpr int pf = tf + 256;                        // P
  static constexpr int vf = pf + 256;                        // V: [u 2][d ND][64 lanes] of 4 rows x 1 column, 8 bytes
  static constexpr int dec = vf + ND * 64;                   // B_end [DK]
  static constexpr int size = dec + DK / 4;
};
// chunks of earlier sequences never reach the next one's first
__device__ __forceinline__ long first_chunk(const RuleArgs& p, int b) { return p.q_start[b] / kC + b; }

long rule_chunk_bytes(int dk, int dv) { return 16L * (dk * 24 + 512 + dv * 4 + dk / 4); }

template <int MODE, int DK, int DV, int KT>
__global__ void __launch_bounds__(256) rule_prep_kernel(const RuleArgs p) {
  using U = Unit<DK, DV>;
  constexpr bool DELTA = MODE != kRetention;
  constexpr int LD = DK + 4, LS = 36, VQ = DK / 8, VV = DV / 8;
  static_assert(U::size * 16 == 16 * (DK * 24 + 512 + DV * 4 + DK / 4), "chunk size");
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* sq = lds;                                // [32][LD]
  float* sk = sq + kC * LD;
  float* sA = sk + kC * LD;                       // [32][LS]
  float* sP = sA + kC * LS;
  float* sT = sP + kC * LS;
  float* sbeta = sT + kC * LS;                    // [32]
  float* sb = sbeta + kC;                         // running logarithms: [32], or [32][LD] per channel
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int b = blockIdx.z, h = p.head0 + blockIdx.y, at = blockIdx.x * kC;
  const int total = p.q_lens[b];
  if (at >= total) return;
  const int live = min(kC, total - at);
  const long row0 = p.q_start[b] + at;
  const int slot = p.slots[b], pos0 = p.pos[p.q_start[b]];
  const int grp = h / (p.H / p.G), channels = 2 * p.G * DK + p.H * DV;
  const bf16_t* x = static_cast<const bf16_t*>(p.x) + row0 * p.ldx;
  const bf16_t* ring = DELTA ? static_cast<const bf16_t*>(p.ring) + (long)max(slot, 0) * p.taps * channels : nullptr;
  uint4_* unit = static_cast<uint4_*>(p.ws) + ((first_chunk(p, b) + blockIdx.x) * p.heads + blockIdx.y) * U::size;

  // ---- inputs: a task is 4 rows x 8 channels of q, k or v
  for (int id = tid; id < 2 * DK + DV; id += 256) {
    const int what = id < DK ? 0 : id < 2 * DK ? 1 : 2, e = id - what * DK;
    const int vec = what < 2 ? e % VQ : e % VV, rg = what < 2 ? e / VQ : e / VV;
    const int ch = 8 * vec + (what == 2 ? 2 * p.G * DK + h * DV : (DELTA ? what * p.G + grp : what * p.H + h) * DK);
    float y[4][8];
    if constexpr (DELTA) {
      float wt[KT][8];
#pragma unroll
      for (int j = 0; j < KT; ++j) {
        const float* cw = p.conv + (long)(p.taps - 1 - min(j, p.taps - 1)) * channels + ch;
        const float4_ lo = load4(cw), hi = load4(cw + 4);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          wt[j][i] = j < p.taps ? lo[i] : 0.f;
          wt[j][4 + i] = j < p.taps ? hi[i] : 0.f;
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int i = 0; i < 8; ++i) y[r][i] = 0.f;
#pragma unroll
      for (int i = 1 - KT; i < 4; ++i) {
        const int r = 4 * rg + i, step = at + r, pos = pos0 + step;          // row of the chunk, of the step, position
        const bf16_t* src = nullptr;
        if (r < live && i > -p.taps) {
          if (step >= 0) src = x + (long)r * p.ldx + ch;
          else if (pos >= 0 && slot >= 0) src = ring + (long)(pos % p.taps) * channels + ch;
        }
        float f[8];
        unpack8(src ? *reinterpret_cast<const uint4_*>(src) : uint4_{0u, 0u, 0u, 0u}, f);
#pragma unroll
        for (int rr = 0; rr < 4; ++rr)
          if (rr - i >= 0 && rr - i < KT) {
#pragma unroll
            for (int j = 0; j < 8; ++j) y[rr][j] += wt[rr - i][j] * f[j];
          }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int i = 0; i < 8; ++i) y[r][i] = 4 * rg + r < live ? silu_fast(y[r][i]) : 0.f;
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 4 * rg + r;
        unpack8(t < live ? *reinterpret_cast<const uint4_*>(x + (long)t * p.ldx + ch) : uint4_{0u, 0u, 0u, 0u}, y[r]);
        if (what < 2 && 8 * vec < p.rot && t < live) {
          const int half = p.rot >> 1;
          const bf16_t* head = x + (long)t * p.ldx + ch - 8 * vec;
          const float* a = p.rope + (row0 + t) * p.rot;
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const int d = 8 * vec + i;
            if (d < p.rot) {
              const bool low = d < half;
              const float other = bf2f(head[low ? d + half : d - half]);
              const float* cs = a + 2 * (low ? d : d - half);
              y[r][i] = y[r][i] * cs[0] + (low ? -other : other) * cs[1];
            }
          }
        }
      }
    }
    if (what < 2) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float scale = what ? 1.f / sqrtf((float)p.dim) : 1.f;
        if constexpr (DELTA) {
          float ss = 0.f;
#pragma unroll
          for (int i = 0; i < 8; ++i) ss += y[r][i] * y[r][i];
#pragma unroll
          for (int d = 1; d < VQ; d <<= 1) ss += __shfl_xor(ss, d, 64);
          scale = 1.f / sqrtf(ss + 1e-6f) * (what ? 1.f : 1.f / sqrtf((float)p.dim));
        }
        float* dst = (what ? sk : sq) + (4 * rg + r) * LD + 8 * vec;
        store4(dst, float4_{y[r][0], y[r][1], y[r][2], y[r][3]} * scale);
        store4(dst + 4, float4_{y[r][4], y[r][5], y[r][6], y[r][7]} * scale);
      }
    } else {
      uint2_* dst = reinterpret_cast<uint2_*>(unit + U::vf);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int col = 8 * vec + i;
        dst[((rg >> 2) * U::ND + (col >> 4)) * 64 + (rg & 3) * 16 + (col & 15)] =
            uint2_{pack2(y[0][i], y[1][i]), pack2(y[2][i], y[3][i])};
      }
    }
  }

  // ---- write strengths and running logarithms of the decays
  if constexpr (DELTA) {
    if (tid >= 64 && tid < 96) {
      const int t = tid - 64;
      sbeta[t] = t < live ? sigmoid_f(p.beta[(row0 + t) * p.ldb + h]) : 0.f;
    }
  }
  if constexpr (MODE == kRetention) {
    if (tid < kC) sb[tid] = (float)min(tid + 1, live) * fmaxf(p.rate[p.H + h], kLeast);
  } else if constexpr (MODE == kHead) {
    if (tid < 64) {                               // whole wave: lanes 32 .. take part in the shuffles
      const int t = tid & 31;
      float lg = t < live ? log_decay(p.decay[(row0 + min(t, live - 1)) * p.ldd + h] + p.bias[h], p.rate[h]) : 0.f;
#pragma unroll
      for (int d = 1; d < kC; d <<= 1) {
        const float other = __shfl_up(lg, d, 32);
        if (t >= d) lg += other;
      }
      if (tid < kC) sb[tid] = lg;
    }
  } else {
    constexpr int RG = 256 / DK, RR = kC / RG;    // groups of rows, rows of a group
    const int d = tid % DK, first = (tid / DK) * RR;
    const float bias = p.bias[h * DK + d], rate = p.rate[h];
    const float* z = p.decay + row0 * p.ldd + h * DK + d;
    float lg[RR], run = 0.f;
#pragma unroll
    for (int i = 0; i < RR; ++i) lg[i] = z[(long)min(first + i, live - 1) * p.ldd];
#pragma unroll
    for (int i = 0; i < RR; ++i) {
      run += first + i < live ? log_decay(lg[i] + bias, rate) : 0.f;
      lg[i] = run;
    }
    if constexpr (RG > 1) {
      sb[(tid / DK) * LD + d] = run;              // group totals, before the rows are stored
      __syncthreads();
      run = 0.f;
      for (int i = 0; i < tid / DK; ++i) run += sb[i * LD + d];
      __syncthreads();
    } else {
      run = 0.f;
    }
#pragma unroll
    for (int i = 0; i < RR; ++i) sb[(first + i) * LD + d] = lg[i] + run;
  }
  __syncthreads();

  // ---- scores: tiles (rows 16 .., keys 0 ..), (0, 0), (16, 16) by a wave each
  const int g = lane >> 4, c16 = lane & 15;
  const float4_ zero = float4_{0.f, 0.f, 0.f, 0.f};
  if (w < 3) {
    const int tr = w == 1 ? 0 : 16, tc = w == 2 ? 16 : 0;
    const int ref = w == 2 ? 23 : w == 1 ? 7 : 15;               // reference row of the decays per channel
    float4_ acc_a = zero, acc_p = zero;
    auto frag = [&](const float* m, int row, int d0, int sign) {  // sign: of the row's logarithm above the reference's; 0: drop
      float4_ lo = load4(m + row * LD + d0), hi = load4(m + row * LD + d0 + 4);
      if constexpr (MODE == kChannel) {
        const float4_ r0 = load4(sb + ref * LD + d0), r1 = load4(sb + ref * LD + d0 + 4);
        const float4_ b0 = load4(sb + row * LD + d0), b1 = load4(sb + row * LD + d0 + 4);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          lo[j] = sign ? lo[j] * __builtin_amdgcn_exp2f(sign > 0 ? b0[j] - r0[j] : r0[j] - b0[j]) : 0.f;
          hi[j] = sign ? hi[j] * __builtin_amdgcn_exp2f(sign > 0 ? b1[j] - r1[j] : r1[j] - b1[j]) : 0.f;
        }
      }
      return split8(lo, hi);
    };
    const int late = c16 >= 8;
#pragma unroll 2
    for (int i = 0; i < U::NI; ++i) {
      const int d0 = 32 * i + 8 * g;
      const Split kc = frag(sk, tc + c16, d0, w == 0 || !late ? -1 : 1);      // keys (a half's later rows as rows)
      const Split qr = frag(sq, tr + c16, d0, w == 0 || late ? 1 : 0);
      acc_p = mac(qr, kc, acc_p);
      if constexpr (DELTA) {
        if (w == 0) acc_a = mac(frag(sk, tr + c16, d0, 1), kc, acc_a);
        else acc_a = mac(kc, kc, acc_a);
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int t = tr + 4 * g + j, s = tc + c16;
      if constexpr (MODE == kChannel) {
        if (w == 0 || (4 * g + j >= 8 && !late)) {
          sA[t * LS + s] = sbeta[t] * acc_a[j];
          sP[t * LS + s] = acc_p[j];
        }
      } else if (s <= t) {
        const float dec = __builtin_amdgcn_exp2f(sb[t] - sb[s]);
        if constexpr (DELTA) sA[t * LS + s] = s < t ? sbeta[t] * dec * acc_a[j] : 0.f;
        sP[t * LS + s] = dec * acc_p[j];
      }
    }
  }
  if constexpr (MODE == kChannel) {               // pairs inside an 8-row block: a wave per block, a lane per pair
    const int t = 8 * w + (lane >> 3), s = 8 * w + (lane & 7);
    if (s <= t) {
      float a = 0.f, q = 0.f;
#pragma unroll 2
      for (int d = 0; d < DK; d += 4) {
        const float4_ bt = load4(sb + t * LD + d), bs = load4(sb + s * LD + d), ks = load4(sk + s * LD + d);
        const float4_ kt = load4(sk + t * LD + d), qt = load4(sq + t * LD + d);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float e = ks[j] * __builtin_amdgcn_exp2f(bt[j] - bs[j]);
          a += kt[j] * e;
          q += qt[j] * e;
        }
      }
      sA[t * LS + s] = s < t ? sbeta[t] * a : 0.f;
      sP[t * LS + s] = q;
    }
  }
  __syncthreads();

  // ---- (I + A)^-1: both 16 x 16 blocks on the diagonal by columns, then the one below them
  if constexpr (DELTA) {
    if (w == 0) {
      const int o = (lane >> 5) * 16, j = lane & 15;
      float col[16];
#pragma unroll
      for (int t = 0; t < 16; ++t) {
        float y = t == j ? 1.f : 0.f;
#pragma unroll
        for (int s = 0; s < t; ++s) y -= sA[(o + t) * LS + o + s] * col[s];
        col[t] = y;
      }
      if (!(lane & 16)) {
#pragma unroll
        for (int t = 0; t < 16; ++t) sT[(o + t) * LS + o + j] = col[t];
      }
    }
    __syncthreads();
    const int r = tid >> 4, c = tid & 15;
    float y = 0.f;
#pragma unroll
    for (int s = 0; s < 16; ++s) y += sA[(16 + r) * LS + s] * sT[s * LS + c];
    sT[r * LS + 16 + c] = y;                      // (above the diagonal: free)
    __syncthreads();
    y = 0.f;
#pragma unroll
    for (int s = 0; s < 16; ++s) y -= sT[(16 + r) * LS + 16 + s] * sT[s * LS + 16 + c];
    sT[(16 + r) * LS + c] = y;
    __syncthreads();
  }

  // ---- operands of the scan
  auto put = [&](int place, const Split& f) {
    unit[place + lane] = __builtin_bit_cast(uint4_, f.hi);
    unit[place + 64 + lane] = __builtin_bit_cast(uint4_, f.lo);
  };
  constexpr int NR = 2 * U::NI;
  for (int f = w; f < 2 * NR + U::NK + 4; f += 4) {
    if (f < 2 * NR) {                             // rows decayed from the chunk's start
      if (!DELTA && f < NR) continue;
      const int i = f % NR, row = 16 * (i / U::NI) + c16, d0 = 32 * (i % U::NI) + 4 * g;
      const float* src = (f < NR ? sk : sq) + row * LD + d0;
      float4_ lo = load4(src), hi = load4(src + 16);
      if constexpr (MODE == kChannel) {
        const float4_ b0 = load4(sb + row * LD + d0), b1 = load4(sb + row * LD + d0 + 16);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          lo[j] *= __builtin_amdgcn_exp2f(b0[j]);
          hi[j] *= __builtin_amdgcn_exp2f(b1[j]);
        }
      } else {
        const float e = __builtin_amdgcn_exp2f(sb[row]);
        lo *= e;
        hi *= e;
      }
      put((f < NR ? U::kd : U::qd) + i * 128, split8(lo, hi));
    } else if (f < 2 * NR + U::NK) {              // keys decayed to its end, by channel
      const int i = f - 2 * NR, ch = 16 * i + c16;
      float4_ y[2];
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int t = 16 * u + 4 * g + j;
          const float d = MODE == kChannel ? sb[31 * LD + ch] - sb[t * LD + ch] : sb[31] - sb[t];
          y[u][j] = sk[t * LD + ch] * __builtin_amdgcn_exp2f(d);
        }
      put(U::ke + i * 128, split8(y[0], y[1]));
    } else {                                      // the inverse (times the write strengths) and the scores of q
      const int i = f - 2 * NR - U::NK, u = i & 1, t = 16 * u + c16;
      const bool inv = i < 2;
      if (!DELTA && inv) continue;
      float4_ y[2];
#pragma unroll
      for (int v = 0; v < 2; ++v)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int s = 16 * v + 4 * g + j;
          y[v][j] = s > t ? 0.f : inv ? sT[t * LS + s] * sbeta[s] : sP[t * LS + s];
        }
      put((inv ? U::tf : U::pf) + u * 128, split8(y[0], y[1]));
    }
  }
  float* dec = reinterpret_cast<float*>(unit + U::dec);
  if (tid < DK) dec[tid] = __builtin_amdgcn_exp2f(MODE == kChannel ? sb[31 * LD + tid] : sb[31]);
}

// NW waves of ND x 16 columns each; AHEAD: the next chunk's operands are loaded as soon as this one's are used up
template <bool DELTA, int DK, int DV, int ND, bool AHEAD>
__global__ void __launch_bounds__(DV / ND * 4, 1) rule_scan_kernel(const RuleArgs p) {
  using U = Unit<DK, DV>;
  constexpr int NW = DV / (16 * ND), NI = U::NI, NK = U::NK;
  __shared__ float red[2][NW][kC];
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int g = lane >> 4, c16 = lane & 15;
  const int b = blockIdx.y, h = p.head0 + blockIdx.x;
  const int total = p.q_lens[b];
  if (total < 1) return;
  const int chunks = (total + kC - 1) / kC;
  const long row0 = p.q_start[b];
  const int slot = p.slots[b], col0 = w * ND * 16 + c16;
  const bool old = slot >= 0 && p.pos[row0] > 0;
  float* st = p.state + ((long)max(slot, 0) * p.H + h) * DK * DV + col0;

  float4_ S[NK][ND];                              // rows 16 i + 4 g .., column 16 d of the wave's
#pragma unroll
  for (int i = 0; i < NK; ++i)
#pragma unroll
    for (int d = 0; d < ND; ++d)
#pragma unroll
      for (int j = 0; j < 4; ++j) S[i][d][j] = old ? st[(long)(16 * i + 4 * g + j) * DV + 16 * d] : 0.f;
  float gain[ND];
#pragma unroll
  for (int d = 0; d < ND; ++d) gain[d] = DELTA ? p.gain[col0 + 16 * d] : 1.f;

  const uint4_* unit = static_cast<const uint4_*>(p.ws) + (first_chunk(p, b) * p.heads + blockIdx.x) * U::size;
  const long stride = (long)p.heads * U::size;
  auto frag = [&](const uint4_* u, int place) {
    return Split{__builtin_bit_cast(bf16x8, u[place + lane]), __builtin_bit_cast(bf16x8, u[place + 64 + lane])};
  };
  constexpr int A = AHEAD ? 1 : 0;
  Split kd[A && DELTA ? 2 : 1][A && DELTA ? NI : 1], qd[A ? 2 : 1][A ? NI : 1], ke[A ? NK : 1], tf[2], pf[2];
  uint2_ vf[2][ND];
  auto load_rows = [&](const uint4_* u) {
    if constexpr (AHEAD) {
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < NI; ++j) {
          if constexpr (DELTA) kd[i][j] = frag(u, U::kd + (i * NI + j) * 128);
          qd[i][j] = frag(u, U::qd + (i * NI + j) * 128);
        }
    }
  };
  auto load_keys = [&](const uint4_* u) {
    if constexpr (AHEAD) {
#pragma unroll
      for (int i = 0; i < NK; ++i) ke[i] = frag(u, U::ke + i * 128);
    }
  };
  auto load_rest = [&](const uint4_* u) {
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      if constexpr (DELTA) tf[i] = frag(u, U::tf + i * 128);
      pf[i] = frag(u, U::pf + i * 128);
#pragma unroll
      for (int d = 0; d < ND; ++d) vf[i][d] = reinterpret_cast<const uint2_*>(u + U::vf)[(i * U::ND + w * ND + d) * 64 + lane];
    }
  };
  load_rows(unit);
  load_rest(unit);
  load_keys(unit);
  for (int c = 0; c < chunks; ++c) {
    const uint4_* cur = unit;
    if (c + 1 < chunks) unit += stride;           // (the last chunk loads itself again)
    const int at = c * kC;
    float4_ dec[NK];
#pragma unroll
    for (int i = 0; i < NK; ++i) dec[i] = reinterpret_cast<const float4_*>(cur + U::dec)[4 * i + g];
    bf16_t z[2][4][ND];                           // gates of the rows and columns this lane will store
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const bf16_t* gate = static_cast<const bf16_t*>(p.gate) + (row0 + min(at + 16 * u + 4 * g + j, total - 1)) * p.ldg + h * DV + col0;
#pragma unroll
        for (int d = 0; d < ND; ++d) z[u][j][d] = gate[16 * d];
      }

    float4_ R[2][ND] = {}, O[2][ND] = {};
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      Split sf[ND];
#pragma unroll
      for (int d = 0; d < ND; ++d) sf[d] = split8(S[2 * i][d], S[2 * i + 1][d]);
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        if constexpr (DELTA) {
          const Split k = AHEAD ? kd[u][AHEAD ? i : 0] : frag(cur, U::kd + (u * NI + i) * 128);
#pragma unroll
          for (int d = 0; d < ND; ++d) R[u][d] = mac(k, sf[d], R[u][d]);
        }
        const Split q = AHEAD ? qd[AHEAD ? u : 0][AHEAD ? i : 0] : frag(cur, U::qd + (u * NI + i) * 128);
#pragma unroll
        for (int d = 0; d < ND; ++d) O[u][d] = mac(q, sf[d], O[u][d]);
      }
    }
    load_rows(unit);
    Split uf[ND];
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      float4_ v[2];
#pragma unroll
      for (int u = 0; u < 2; ++u)
        v[u] = float4_{__uint_as_float(vf[u][d][0] << 16), __uint_as_float(vf[u][d][0] & 0xffff0000u),
                       __uint_as_float(vf[u][d][1] << 16), __uint_as_float(vf[u][d][1] & 0xffff0000u)};
      if constexpr (DELTA) {
        const Split rf = split8(v[0] - R[0][d], v[1] - R[1][d]);
        const float4_ zero = float4_{0.f, 0.f, 0.f, 0.f};
        uf[d] = split8(mac(tf[0], rf, zero), mac(tf[1], rf, zero));
      } else {
        uf[d] = split8(v[0], v[1]);
      }
#pragma unroll
      for (int u = 0; u < 2; ++u) O[u][d] = mac(pf[u], uf[d], O[u][d]);
    }
    load_rest(unit);
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const Split k = AHEAD ? ke[AHEAD ? i : 0] : frag(cur, U::ke + i * 128);
#pragma unroll
      for (int d = 0; d < ND; ++d) S[i][d] = mac(k, uf[d], S[i][d] * dec[i]);
    }
    load_keys(unit);

    // the heads' norm over all waves' columns, gain and gate
    float* mine = red[c & 1][w];
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        float ss = 0.f;
#pragma unroll
        for (int d = 0; d < ND; ++d) ss += O[u][d][j] * O[u][d][j];
#pragma unroll
        for (int d = 1; d < 16; d <<= 1) ss += __shfl_xor(ss, d, 64);
        if (c16 == 0) mine[16 * u + 4 * g + j] = ss;
      }
    __syncthreads();
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      float4_ sum = float4_{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int v = 0; v < NW; ++v) sum += load4(&red[c & 1][v][16 * u + 4 * g]);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int t = at + 16 * u + 4 * g + j;
        const float r = 1.f / sqrtf(sum[j] / (float)p.vdim + p.eps);
        bf16_t* out = static_cast<bf16_t*>(p.out) + (row0 + t) * p.ldo + h * DV + col0;
        if (t < total) {
#pragma unroll
          for (int d = 0; d < ND; ++d)
            out[16 * d] = f2bf(O[u][d][j] * r * gain[d] * gate_act<true>(bf2f(z[u][j][d]), p.gate_kind));
        }
      }
    }
  }
  if (slot >= 0) {
#pragma unroll
    for (int i = 0; i < NK; ++i)
#pragma unroll
      for (int d = 0; d < ND; ++d)
#pragma unroll
        for (int j = 0; j < 4; ++j) st[(long)(16 * i + 4 * g + j) * DV + 16 * d] = S[i][d][j];
  }
}

template <int MODE, int DK, int DV, int KT>
static void prep(const RuleArgs& a, hipStream_t s) {
  constexpr int lds = 4 * (2 * kC * (DK + 4) + 3 * kC * 36 + kC + (MODE == kChannel ? kC * (DK + 4) : kC));
  (void)hipFuncSetAttribute(reinterpret_cast<const void*>(rule_prep_kernel<MODE, DK, DV, KT>),
                            hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  rule_prep_kernel<MODE, DK, DV, KT><<<dim3((a.max_q + kC - 1) / kC, a.heads, a.B), 256, lds, s>>>(a);
}

template <int MODE, int DK, int DV>
static void chunks(const RuleArgs& a, hipStream_t s) {
  if (MODE == kRetention || a.taps <= 4) prep<MODE, DK, DV, 4>(a, s);
  else prep<MODE, DK, DV, 16>(a, s);
  constexpr int ND = DV == 64 ? 1 : 2;
  rule_scan_kernel<MODE != kRetention, DK, DV, ND, (DK <= 128)><<<dim3(a.heads, a.B), DV / ND * 4, 0, s>>>(a);
}

void launch_rule_chunks(const RuleArgs& a, hipStream_t s) {
#define GO(DK, DV, MODE) chunks<MODE, DK, DV>(a, s)
  if (a.mode == kRetention) SHAI_LM_STATE(GO, kRetention);
  else if (a.mode == kHead) SHAI_LM_STATE(GO, kHead);
  else SHAI_LM_STATE(GO, kChannel);
#undef GO
  SHAI_CHECK_LAUNCH();
}

template <typename T, int MODE, int DK, int DV>
static void rows(const RuleArgs& a, hipStream_t s) {
  constexpr int NT = DK > 128 ? 1024 : 256;
  rule_rows_kernel<T, MODE, DK, DV, NT><<<dim3(a.H, a.B), NT, 0, s>>>(a);
}

template <typename T>
static void rows(const RuleArgs& a, hipStream_t s) {
#define GO(DK, DV, MODE) rows<T, MODE, DK, DV>(a, s)
  if (a.mode == kRetention) SHAI_LM_STATE(GO, kRetention);
  else if (a.mode == kHead) SHAI_LM_STATE(GO, kHead);
  else SHAI_LM_STATE(GO, kChannel);
#undef GO
}

void launch_rule_rows(const RuleArgs& a, bool f32, hipStream_t s) {
  if (f32) rows<float>(a, s);
  else rows<bf16_t>(a, s);
  SHAI_CHECK_LAUNCH();
}

}  // namespace shai_lm
