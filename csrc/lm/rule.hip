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
// chunks   bf16 prompts in chunks of 32 rows, three launches.  With B_t the product of the decays up to row t of a chunk,
//            A[t, s] = b_t sum_d k_t k_s B_t / B_s (s < t),   P[t, s] = sum_d q_t k_s B_t / B_s (s <= t),
//            U = (I + A)^-1 diag(b) (V - (B K) S),   O = (B Q) S + P U,   S' = B_end S + (K B_end / B)^T U.
//          prep (a workgroup per chunk and head of queries and keys, all at once): convolution, norms, decays per channel, the
//          two score matrices, and the operands of the scan in the order its lanes load them.
//          solve (a wave per chunk and head): the inverse, and decays per head.
//          scan (a workgroup per sequence and head): chunk after chunk, each wave 16 columns of S (registers); prepared
//          chunks are loaded to LDS one ahead.
//          Few long sequences are cut into segments.  A segment is affine in the state, S' = M S + L: a first scan starts
//          from zero for L and, without values, from the identity for M; `link` chains the segments' states; then every
//          segment is scanned from its own.
//          Quotients of decays come from differences of running logarithms.  A decay per channel enters the matrix products
//          through a reference between the two rows: the border of the 16-row halves, that of a half's 8-row blocks, or a
//          block's fourth row.  Operands of matrix products are a bf16 value plus its bf16 remainder; sums are fp32.
#include "matrix_state.h"

namespace shai_lm {

constexpr int kRetention = 0, kHead = 1, kChannel = 2;     // decay: fixed; per head; per key channel
constexpr float kLeast = -40.f;                            // base-2 logarithm of a decay that leaves nothing in fp32

__device__ __forceinline__ float softplus_exact(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
// base-2 logarithm of exp(-rate softplus(x)), limited
__device__ __forceinline__ float log_decay(float x, float rate, float least) {
  const float e = __builtin_amdgcn_exp2f(-fabsf(x) * kInvLn2);
  const float series = e * (1.f - e * (0.5f - e * (1.f / 3.f - e * (0.25f - e * 0.2f)))) * kInvLn2;
  const float sp = fmaxf(x, 0.f) * kInvLn2 + (e < 0.03f ? series : __builtin_amdgcn_logf(1.f + e));
  return fmaxf(-rate * sp, least);
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
__global__ void __launch_bounds__(NT, NT > 256 ? 4 : 3) rule_rows_kernel(const RuleArgs p) {
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
  const int ring0 = DELTA ? pos0 % p.taps : 0;
  // channel ch of row t after its convolution and silu
  auto conv = [&](long t, int ch) {
    const int row = (int)(t - t0);
    float y = p.conv[(p.taps - 1) * channels + ch] * load1(x + t * p.ldx + ch);
#pragma unroll 3
    for (int j = 1; j < p.taps; ++j) {
      const int m = ring0 + row - j;                         // before the step's first row: its place in the ring
      const bool here = row >= j;
      const T* src = here ? x + (t - j) * p.ldx + ch : ring + (m < 0 ? m + p.taps : m) * channels + ch;
      if (here || (pos0 + row >= j && slot >= 0)) y += p.conv[(p.taps - 1 - j) * channels + ch] * load1(src);
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
    float rq = 1.f, rk = 1.f, gh = MODE == kRetention ? p.rate[h] : 1.f, beta = 1.f;
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
      __builtin_amdgcn_sched_barrier(0);          // four rows of k and q in registers at a time
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
        __builtin_amdgcn_sched_barrier(0);
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
// Prepared chunks, in 16-byte units.  Rows of a chunk (time x channels) are kept in the order in which the scan reads them from LDS,
// as rows and, transposed, as columns.  Keys and queries: bf16 values and then their remainders; of every 32 channels, 4 g .. and
// 16 + 4 g .. share a 16-byte piece, and the pieces of a row are permuted by its number modulo 8.  Values: 8-byte pieces
// permuted by `turned`.  Score operands (time x time) are fragments of [64 lanes] of 16 bytes, values and remainders one after
// the other, u: rows 16 u ..; a lane holds times 4 g .. and 16 + 4 g ..
// Row units: one per head with a decay per channel (decays applied), else one per key head (the scan applies the decays).
template <int DK, bool CHANNEL>
struct RowUnit {
  static constexpr int part = DK * 8;                        // [2][32][DK]
  static constexpr int kd = 0;                               // K, or B K
  static constexpr int qd = part;                            // Q, or B Q
  static constexpr int ke = CHANNEL ? 2 * part : 0;          // K B_end / B
  static constexpr int size = CHANNEL ? 3 * part : 2 * part;
};
template <int DV>
struct HeadUnit {
  static constexpr int tf = 0;                               // (I + A)^-1 diag(b)  [u 2][2][64]
  static constexpr int pf = tf + 256;                        // P (retention starts here)
  static constexpr int vf = pf + 256;                        // V [32][DV], values only
  static constexpr int dec = vf + DV * 4;                    // floats: B_end [DK], or B [32], B_end / B [32], B_end
  static constexpr int size = dec + 64;
};
__device__ __forceinline__ int turned(int t) { return (t & 3) << 2 | (t >> 2 & 3); }
// 8 columns 8 vec .. of row t of the values
template <int DV>
__device__ __forceinline__ void put_values(uint4_* part, int t, int vec, uint4_ y) {
  const int x = turned(t);
  part[t * (DV / 8) + (vec ^ (x >> 1))] = x & 1 ? uint4_{y[2], y[3], y[0], y[1]} : y;
}
__device__ __forceinline__ uint32_t dpp_swap2(uint32_t x) {       // lanes 0 1 2 3 of every four <- 2 3 0 1
  return __builtin_amdgcn_update_dpp(0u, x, 0x4E, 0xf, 0xf, true);
}
// 8 channels 8 vec .. of row t; lanes of consecutive `vec` call it together
template <int DK>
__device__ __forceinline__ void put_row(uint4_* part, int t, int vec, const Split& f) {
  const bool second = vec & 2;                    // of the 16 channels that share pieces with 16 others
  const int piece = 4 * (vec >> 2) + 2 * (vec & 1) + second;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const uint4_ y = __builtin_bit_cast(uint4_, i ? f.lo : f.hi);
    const uint32_t a = dpp_swap2(second ? y[0] : y[2]), b = dpp_swap2(second ? y[1] : y[3]);
    part[i * 4 * DK + t * (DK / 8) + (piece ^ (t & 7))] = second ? uint4_{a, b, y[2], y[3]} : uint4_{y[0], y[1], a, b};
  }
}
// Scores before the solve, fp32 [2][32][32]: A and P (a decay per channel), or k k^T and q k^T.
constexpr int kScores = 512;
// chunks of earlier sequences never reach the next one's first
__device__ __forceinline__ long first_chunk(const RuleArgs& p, int b) { return p.q_start[b] / kC + b; }

__device__ __forceinline__ uint4_* head_unit(const RuleArgs& p, long chunk, int head, int size) {
  return static_cast<uint4_*>(p.ws) + (chunk * p.heads + head) * size;
}
// behind all head units; then the scores
__device__ __forceinline__ uint4_* row_unit(const RuleArgs& p, long chunk, int key, int keys, int size, int head_size) {
  return static_cast<uint4_*>(p.ws) + p.ws_chunks * p.heads * head_size + (chunk * keys + key) * size;
}
__device__ __forceinline__ float* score_unit(const RuleArgs& p, long chunk, int key, int keys, int size, int head_size) {
  return reinterpret_cast<float*>(static_cast<uint4_*>(p.ws) + p.ws_chunks * (p.heads * (long)head_size + keys * (long)size) +
                                  (chunk * keys + key) * kScores);
}

long rule_chunk_bytes(int dk, int dv, int heads, int keys, bool channel) {
  return 16L * ((long)keys * (dk * (channel ? 24 : 16) + kScores) + (long)heads * (512 + dv * 4 + 64));
}

// ---- inputs of 4 rows x 8 channels
// Channels ch .. of rows r0 .. r0 + 3 of a chunk after their convolution and silu; rows behind the last live one are zero.
// `x`: the chunk's first row, row `at` of the step; before the step's first row the ring's inputs count.
__device__ __forceinline__ void conv_rows(const RuleArgs& p, const bf16_t* x, int ch, int channels, int r0, int at, int live,
                                          int pos0, int slot, float (&y)[4][8]) {
  auto tap = [&](int j, float (&wt)[8]) {         // of the input j rows before
    const float* cw = p.conv + (long)(p.taps - 1 - min(j, p.taps - 1)) * channels + ch;
    const float on = j < p.taps ? 1.f : 0.f;
    *reinterpret_cast<float4_*>(wt) = load4(cw) * on;
    *reinterpret_cast<float4_*>(wt + 4) = load4(cw + 4) * on;
  };
#pragma unroll
  for (int r = 0; r < 4; ++r)
#pragma unroll
    for (int i = 0; i < 8; ++i) y[r][i] = 0.f;
  if (at > 0 && p.taps <= 4) {                    // every input is a row of the step
    uint4_ in[7];
    float wt[4][8];
#pragma unroll
    for (int i = 0; i < 7; ++i)                   // (rows behind the last one repeat it: their results are dropped)
      in[i] = *reinterpret_cast<const uint4_*>(x + (long)min(r0 + i - 3, live - 1) * p.ldx + ch);
#pragma unroll
    for (int j = 0; j < 4; ++j) tap(j, wt[j]);
#pragma unroll
    for (int i = 0; i < 7; ++i) {
      float f[8];
      unpack8(in[i], f);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = r - i + 3;
        if (j >= 0 && j < 4) {
#pragma unroll
          for (int e = 0; e < 8; ++e) y[r][e] += wt[j < 0 || j > 3 ? 0 : j][e] * f[e];
        }
      }
    }
  } else {
    const bf16_t* ring = static_cast<const bf16_t*>(p.ring) + (long)max(slot, 0) * p.taps * channels + ch;
    const int ring0 = pos0 % p.taps;
#pragma unroll 1
    for (int j = 0; j < p.taps; ++j) {
      float wt[8];
      tap(j, wt);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = min(r0 + r, live - 1) - j, m = ring0 + at + i;
        const bool here = at + i >= 0, past = pos0 + at + i >= 0 && slot >= 0;
        const bf16_t* src = here ? x + (long)i * p.ldx + ch : ring + (long)(m < 0 ? m + p.taps : m) * channels;
        float f[8];
        unpack8(here || past ? *reinterpret_cast<const uint4_*>(src) : uint4_{0u, 0u, 0u, 0u}, f);
#pragma unroll
        for (int e = 0; e < 8; ++e) y[r][e] += wt[e] * f[e];
      }
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r)
#pragma unroll
    for (int i = 0; i < 8; ++i) y[r][i] = r0 + r < live ? silu_fast(y[r][i]) : 0.f;
}

// the same without a convolution: channels d0 .. of the head at x, turned where `rope` is given
__device__ __forceinline__ void turn_rows(const RuleArgs& p, const bf16_t* x, int d0, int r0, int live, const float* rope,
                                          float (&y)[4][8]) {
  const int half = p.rot >> 1;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = r0 + r;
    const bf16_t* row = x + (long)min(t, live - 1) * p.ldx;
    unpack8(t < live ? *reinterpret_cast<const uint4_*>(row + d0) : uint4_{0u, 0u, 0u, 0u}, y[r]);
    if (rope && d0 < p.rot && t < live) {
      const float* a = rope + (long)t * p.rot;
      if ((half & 7) == 0) {                      // the partners are 8 consecutive channels too
        const bool low = d0 < half;
        const float* cs = a + 2 * (low ? d0 : d0 - half);
        float o[8];
        unpack8(*reinterpret_cast<const uint4_*>(row + (low ? d0 + half : d0 - half)), o);
#pragma unroll
        for (int i = 0; i < 8; i += 2) {
          const float4_ c = load4(cs + 2 * i);
          y[r][i] = y[r][i] * c[0] + (low ? -o[i] : o[i]) * c[1];
          y[r][i + 1] = y[r][i + 1] * c[2] + (low ? -o[i + 1] : o[i + 1]) * c[3];
        }
      } else {
        for (int i = 0; i < 8; ++i) {
          const int d = d0 + i;
          if (d < p.rot) {
            const bool low = d < half;
            const float o = bf2f(row[low ? d + half : d - half]);
            const float* cs = a + 2 * (low ? d : d - half);
            y[r][i] = y[r][i] * cs[0] + (low ? -o : o) * cs[1];
          }
        }
      }
    }
  }
}

// factor that makes a row of y (VQ lanes of 8 channels each) a unit vector, times dim^-1/2 for queries
template <int VQ>
__device__ __forceinline__ float unit_factor(const float (&y)[8], bool query, int dim) {
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) ss += y[i] * y[i];
#pragma unroll
  for (int d = 1; d < VQ; d <<= 1) ss += __shfl_xor(ss, d, 64);
  return __builtin_amdgcn_rsqf(query ? (ss + 1e-6f) * (float)dim : ss + 1e-6f);
}

// One decay per head, or a fixed one: a workgroup prepares a chunk's queries and keys, their products, and the values of the
// heads that share them.  Queries and keys lie in LDS as values and remainders, as the matrix products read them.
template <bool DELTA, int DK, int DV>
__global__ void __launch_bounds__(512, 4) rule_prep_head_kernel(const RuleArgs p) {
  using U = RowUnit<DK, false>;
  using HU = HeadUnit<DV>;
  constexpr int NT = 512, LD = DK + 8, VQ = DK / 8, VV = DV / 8;
  extern __shared__ __attribute__((aligned(16))) bf16_t planes[];
  bf16_t* sq = planes;                            // [2][32][LD] values, remainders
  bf16_t* sk = sq + 2 * kC * LD;
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int group = p.H / p.G, keys = p.heads / group;
  const int b = blockIdx.z, key = p.head0 / group + blockIdx.y, at = blockIdx.x * kC;
  const int total = p.q_lens[b];
  if (at >= total) return;
  const int live = min(kC, total - at);
  const long row0 = p.q_start[b] + at;
  const int slot = p.slots[b], pos0 = p.pos[p.q_start[b]];
  const int channels = 2 * p.G * DK + p.H * DV;
  const bf16_t* x = static_cast<const bf16_t*>(p.x) + row0 * p.ldx;
  const long chunk = first_chunk(p, b) + blockIdx.x;
  uint4_* rows = row_unit(p, chunk, blockIdx.y, keys, U::size, HU::size);
  float* scores = score_unit(p, chunk, blockIdx.y, keys, U::size, HU::size);
  auto head = [&](int j) { return head_unit(p, chunk, blockIdx.y * group + j, HU::size); };

  // ---- inputs: a task is 4 rows x 8 channels of q, k or a head's v
  for (int id = tid; id < 2 * DK + group * DV; id += NT) {
    const int what = id < DK ? 0 : id < 2 * DK ? 1 : 2, e = id - what * DK;
    const int vec = what < 2 ? e % VQ : e % VV, rg = what < 2 ? e / VQ : e / VV % 8, j = what < 2 ? 0 : e / DV;
    const int first = what < 2 ? (what * p.G + key) * DK : 2 * p.G * DK + (key * group + j) * DV;
    float y[4][8];
    if constexpr (DELTA) conv_rows(p, x, first + 8 * vec, channels, 4 * rg, at, live, pos0, slot, y);
    else turn_rows(p, x + first, 8 * vec, 4 * rg, live, what < 2 ? p.rope + row0 * p.rot : nullptr, y);
    if (what < 2) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float scale = DELTA ? unit_factor<VQ>(y[r], what == 0, p.dim) : what ? __builtin_amdgcn_rsqf((float)p.dim) : 1.f;
        const Split f = split8(float4_{y[r][0], y[r][1], y[r][2], y[r][3]} * scale,
                               float4_{y[r][4], y[r][5], y[r][6], y[r][7]} * scale);
        bf16_t* dst = (what ? sk : sq) + (4 * rg + r) * LD + 8 * vec;
        *reinterpret_cast<bf16x8*>(dst) = f.hi;
        *reinterpret_cast<bf16x8*>(dst + kC * LD) = f.lo;
        put_row<DK>(rows + (what ? U::kd : U::qd), 4 * rg + r, vec, f);
      }
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r) put_values<DV>(head(j) + HU::vf, 4 * rg + r, vec, pack8(y[r]));
    }
  }
  __syncthreads();

  // ---- k k^T and q k^T: tiles (rows 16 .., keys 0 ..), (0, 0), (16, 16) by a wave each
  const int g = lane >> 4, c16 = lane & 15;
  if (w < 6 && (DELTA || (w & 1))) {
    const int tile = w >> 1, tr = tile == 1 ? 0 : 16, tc = tile == 2 ? 16 : 0;
    const bf16_t* left = ((w & 1) ? sq : sk) + (tr + c16) * LD + 8 * g;
    const bf16_t* right = sk + (tc + c16) * LD + 8 * g;
    auto frag = [&](const bf16_t* m) {
      return Split{*reinterpret_cast<const bf16x8*>(m), *reinterpret_cast<const bf16x8*>(m + kC * LD)};
    };
    float4_ acc = float4_{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < DK / 32; ++i) acc = mac(frag(left + 32 * i), frag(right + 32 * i), acc);
#pragma unroll
    for (int j = 0; j < 4; ++j) scores[(w & 1) * 1024 + (tr + 4 * g + j) * 32 + tc + c16] = acc[j];
  }
}

// Decays per channel: a row's logarithm is kept relative to the fourth row of its 8-row block (c), so that 2^c and 2^-c stay in
// range (rows forget 2^-24 at most); what lies between two blocks, or a block and a border, is one factor per channel.  `fac`:
// [0 + j] start of the chunk to block j, [4 + j] block j to the chunk's end, [8 + j] block j to or from the border of the halves,
// [12 + j] to or from the border of the half's two blocks.
constexpr float kLeastChannel = -24.f;

template <int DK, int DV>
__global__ void __launch_bounds__(512, 4) rule_prep_channel_kernel(const RuleArgs p) {
  using U = RowUnit<DK, true>;
  using HU = HeadUnit<DV>;
  constexpr int NT = 512, LD = DK + 4, VQ = DK / 8, VV = DV / 8;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* sq = lds;                                // [32][LD] q, then q 2^c
  float* sk = sq + kC * LD;                       // [32][LD] k, then k 2^c
  float* sbeta = sk + kC * LD;                    // [32]
  float* sb = sbeta + kC;                         // [32][LD] c, then k 2^-c
  float* sref = sb + kC * LD;                     // logarithms at the blocks' fourth rows [4][DK] and ends [4][DK]
  float* fac = sref + 8 * DK;                     // [16][DK]
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int b = blockIdx.z, h = p.head0 + blockIdx.y, at = blockIdx.x * kC;
  const int total = p.q_lens[b];
  if (at >= total) return;
  const int live = min(kC, total - at);
  const long row0 = p.q_start[b] + at;
  const int slot = p.slots[b], pos0 = p.pos[p.q_start[b]];
  const int grp = h / (p.H / p.G), channels = 2 * p.G * DK + p.H * DV;
  const bf16_t* x = static_cast<const bf16_t*>(p.x) + row0 * p.ldx;
  const long chunk = first_chunk(p, b) + blockIdx.x;
  uint4_* head = head_unit(p, chunk, blockIdx.y, HU::size);
  uint4_* rows = row_unit(p, chunk, blockIdx.y, p.heads, U::size, HU::size);
  float* scores = score_unit(p, chunk, blockIdx.y, p.heads, U::size, HU::size);

  // ---- inputs: a task is 4 rows x 8 channels of q, k or v
  for (int id = tid; id < 2 * DK + DV; id += NT) {
    const int what = id < DK ? 0 : id < 2 * DK ? 1 : 2, e = id - what * DK;
    const int vec = what < 2 ? e % VQ : e % VV, rg = what < 2 ? e / VQ : e / VV;
    const int ch = 8 * vec + (what == 2 ? 2 * p.G * DK + h * DV : (what * p.G + grp) * DK);
    float y[4][8];
    conv_rows(p, x, ch, channels, 4 * rg, at, live, pos0, slot, y);
    if (what < 2) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float scale = unit_factor<VQ>(y[r], what == 0, p.dim);
        float* dst = (what ? sk : sq) + (4 * rg + r) * LD + 8 * vec;
        store4(dst, float4_{y[r][0], y[r][1], y[r][2], y[r][3]} * scale);
        store4(dst + 4, float4_{y[r][4], y[r][5], y[r][6], y[r][7]} * scale);
      }
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r) put_values<DV>(head + HU::vf, 4 * rg + r, vec, pack8(y[r]));
    }
  }

  // ---- write strengths and running logarithms of the decays (by the waves with the fewest tasks)
  if (tid < kC) sbeta[tid] = tid < live ? sigmoid_f(p.beta[(row0 + tid) * p.ldb + h]) : 0.f;
  {
    const int d = tid - (NT - DK);
    if (d >= 0) {
      const float bias = p.bias[h * DK + d], rate = p.rate[h];
      const float* z = p.decay + row0 * p.ldd + h * DK + d;
      float run = 0.f;
#pragma unroll 1
      for (int j = 0; j < 4; ++j) {
        float lg[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) lg[i] = z[(long)min(8 * j + i, live - 1) * p.ldd];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          run += 8 * j + i < live ? log_decay(lg[i] + bias, rate, kLeastChannel) : 0.f;
          lg[i] = run;
        }
        sref[j * DK + d] = lg[3];
        sref[(4 + j) * DK + d] = run;
#pragma unroll
        for (int i = 0; i < 8; ++i) sb[(8 * j + i) * LD + d] = lg[i] - lg[3];
      }
    }
  }
  __syncthreads();

  // ---- q 2^c, k 2^c, k 2^-c, and the factors between blocks
  {
#pragma unroll 2
    for (int id = tid; id < kC * DK / 4; id += NT) {
      const int o = id / (DK / 4) * LD + id % (DK / 4) * 4;
      const float4_ c = load4(sb + o), q = load4(sq + o), k = load4(sk + o);
      float4_ up, dn;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        up[j] = __builtin_amdgcn_exp2f(c[j]);
        dn[j] = __builtin_amdgcn_exp2f(-c[j]);
      }
      store4(sq + o, q * up);
      store4(sk + o, k * up);
      store4(sb + o, k * dn);
    }
    for (int id = tid; id < 16 * DK; id += NT) {
      const int kind = id / (4 * DK), j = id / DK & 3, d = id % DK;
      const float r = sref[j * DK + d];
      const float m = sref[(kind == 1 ? 7 : kind == 2 ? 5 : j < 2 ? 4 : 6) * DK + d];
      const bool to = kind == 1 || (kind == 2 ? j < 2 : !(j & 1));           // from the block to the border
      fac[id] = __builtin_amdgcn_exp2f(kind == 0 ? r : to ? m - r : r - m);
    }
    __syncthreads();
  }

  // ---- scores: tiles (rows 16 .., keys 0 ..), (0, 0), (16, 16), of k and of q by a wave each
  const int g = lane >> 4, c16 = lane & 15;
  const float4_ zero = float4_{0.f, 0.f, 0.f, 0.f};
  if (w < 6) {
    const int tile = w >> 1, tr = tile == 1 ? 0 : 16, tc = tile == 2 ? 16 : 0;
    const bool of_q = w & 1, late = c16 >= 8;
    const float* left = (of_q ? sq : sk) + (tr + c16) * LD;
    float4_ acc = zero, in = zero;
    auto frag = [&](const float* row, int d0) { return split8(load4(row + d0), load4(row + d0 + 4)); };
    auto scaled = [&](const float* row, const float* f, int d0) {
      return split8(load4(row + d0) * load4(f + d0), load4(row + d0 + 4) * load4(f + d0 + 4));
    };
#pragma unroll 2
    for (int i = 0; i < DK / 32; ++i) {
      const int d0 = 32 * i + 8 * g;
      const float* dn = sb + (tc + c16) * LD;     // k 2^-c
      if (tile == 0) {
        acc = mac(scaled(left, fac + (10 + late) * DK, d0), scaled(dn, fac + (8 + late) * DK, d0), acc);
      } else {
        const float* f = fac + (12 + (tr >> 3) + late) * DK;
        const Split keys = scaled(late ? sk + (tr + c16) * LD : dn, f, d0);
        in = mac(frag(left, d0), frag(dn, d0), in);
        if (of_q) {
          Split rows = scaled(left, f, d0);
          const bf16x8 none = __builtin_bit_cast(bf16x8, uint4_{0u, 0u, 0u, 0u});
          rows.hi = late ? rows.hi : none;
          rows.lo = late ? rows.lo : none;
          acc = mac(rows, keys, acc);
        } else {
          acc = mac(keys, keys, acc);
        }
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int t = tr + 4 * g + j, s = tc + c16;
      float y = tile && (t >> 3) == (s >> 3) ? in[j] : acc[j];
      y = of_q ? y : s < t ? y * sbeta[t] : 0.f;
      scores[of_q * 1024 + t * 32 + s] = y;
    }
  }

  // ---- operands of the scan
  for (int id = tid; id < kC * VQ; id += NT) {
    const int t = id / VQ, vec = id % VQ, o = t * LD + 8 * vec;
    const float* from = fac + (t >> 3) * DK + 8 * vec;
    const float* to = from + 4 * DK;
    const float4_ f0 = load4(from), f1 = load4(from + 4);
    put_row<DK>(rows + U::kd, t, vec, split8(load4(sk + o) * f0, load4(sk + o + 4) * f1));
    put_row<DK>(rows + U::qd, t, vec, split8(load4(sq + o) * f0, load4(sq + o + 4) * f1));
    put_row<DK>(rows + U::ke, t, vec, split8(load4(sb + o) * load4(to), load4(sb + o + 4) * load4(to + 4)));
  }
  if (tid < DK) reinterpret_cast<float*>(head + HU::dec)[tid] = fac[3 * DK + tid] * fac[7 * DK + tid];
}

// The rest of a head's chunk by one wave: (I + A)^-1 diag(b), P, and the decays of its rows.  LDS: A below the diagonal, the
// inverse's transpose above it (its diagonal is 1).
template <int MODE, int DK, int DV>
__global__ void __launch_bounds__(256, 4) rule_solve_kernel(const RuleArgs p) {
  using HU = HeadUnit<DV>;
  constexpr bool DELTA = MODE != kRetention, CHANNEL = MODE == kChannel;
  constexpr int LS = 36;
  __shared__ __attribute__((aligned(16))) float sm[4][DELTA ? kC * LS : 4], sb[4][kC], sbeta[4][kC];
  const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c16 = lane & 15, tl = lane & 31;
  const int b = blockIdx.z, h = p.head0 + blockIdx.y, at = (blockIdx.x * 4 + w) * kC;
  const int total = p.q_lens[b];
  if (at >= total) return;                        // whole waves: no barrier below
  const int live = min(kC, total - at), group = CHANNEL ? 1 : p.H / p.G;
  const long row = p.q_start[b] + at + min(tl, live - 1), chunk = first_chunk(p, b) + blockIdx.x * 4 + w;
  uint4_* unit = head_unit(p, chunk, blockIdx.y, HU::size);
  const float* scores = score_unit(p, chunk, blockIdx.y / group, p.heads / group, RowUnit<DK, CHANNEL>::size, HU::size);
  float* m = sm[w];
  float* lb = sb[w];
  float* beta = sbeta[w];
  float a[DELTA ? 16 : 1];
  if constexpr (DELTA) {
#pragma unroll
    for (int i = 0; i < 16; ++i) a[i] = scores[64 * i + lane];               // rows 2 i, 2 i + 1
  }
  float4_ pr[2][2];
#pragma unroll
  for (int u = 0; u < 2; ++u)
#pragma unroll
    for (int v = 0; v < 2; ++v) pr[u][v] = load4(scores + 1024 + (16 * u + c16) * 32 + 16 * v + 4 * g);
  float lg = 0.f, bt = 0.f;
  if constexpr (DELTA) bt = tl < live ? sigmoid_f(p.beta[row * p.ldb + h]) : 0.f;
  if constexpr (MODE == kHead) {
    lg = tl < live ? log_decay(p.decay[row * p.ldd + h] + p.bias[h], p.rate[h], kLeast) : 0.f;
#pragma unroll
    for (int d = 1; d < kC; d <<= 1) {
      const float other = __shfl_up(lg, d, 32);
      if (tl >= d) lg += other;
    }
  } else if constexpr (!CHANNEL) {
    lg = (float)min(tl + 1, live) * fmaxf(p.rate[p.H + h], kLeast);
  }
  if (lane < kC) {
    lb[tl] = lg;
    beta[tl] = bt;
  }
  if constexpr (!CHANNEL) {
    const float end = __shfl(lg, 31, 64);
    float* dec = reinterpret_cast<float*>(unit + HU::dec);
    dec[lane] = __builtin_amdgcn_exp2f(lane < kC ? lg : end - lg);
    if (lane == 0) dec[64] = __builtin_amdgcn_exp2f(end);
  }
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  auto put = [&](int place, const Split& f) {
    unit[place + lane] = __builtin_bit_cast(uint4_, f.hi);
    unit[place + 64 + lane] = __builtin_bit_cast(uint4_, f.lo);
  };
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int t = 16 * u + c16;
    const float l = lb[t];
#pragma unroll
    for (int v = 0; v < 2; ++v)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int s = 16 * v + 4 * g + i;
        const float y = CHANNEL ? pr[u][v][i] : pr[u][v][i] * __builtin_amdgcn_exp2f(fminf(l - lb[s], 0.f));
        pr[u][v][i] = s > t ? 0.f : y;            // (scores above the diagonal are not all written)
      }
    put(HU::pf + u * 128, split8(pr[u][0], pr[u][1]));
  }
  if constexpr (DELTA) {
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int t = 2 * i + (lane >> 5);
      if (tl < t) m[t * LS + tl] = CHANNEL ? a[i] : a[i] * beta[t] * __builtin_amdgcn_exp2f(lb[t] - lg);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    float col[16];
    {                                             // both 16 x 16 blocks on the diagonal by columns
      const float* blk = m + ((lane >> 5) * 16) * LS + (lane >> 5) * 16;
#pragma unroll
      for (int t = 0; t < 16; ++t) {
        if (t % 4 == 0) __builtin_amdgcn_sched_barrier(0);                  // four rows in registers at a time
        float y = t == c16 ? 1.f : 0.f, y2 = 0.f;
#pragma unroll
        for (int s = 0; s < t; ++s) {
          const float e = blk[t * LS + s] * col[s];
          if (s & 1) y2 -= e;
          else y -= e;
        }
        col[t] = y + y2;
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      float* up = m + ((lane >> 5) * 16 + c16) * LS + (lane >> 5) * 16;
#pragma unroll
      for (int t = 1; t < 16; ++t)
        if (t > c16 && !(lane & 16)) up[t] = col[t];
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    {                                             // A21 T11, kept above the diagonal
      float y[4];
#pragma unroll
      for (int s = 0; s < 16; ++s) col[s] = s == c16 ? 1.f : s > c16 ? m[c16 * LS + s] : 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        y[i] = 0.f;
#pragma unroll
        for (int s = 0; s < 16; ++s) y[i] += m[(16 + 4 * g + i) * LS + s] * col[s];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) m[(4 * g + i) * LS + 16 + c16] = y[i];
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    {                                             // -T22 of it, transposed
      float4_ y = float4_{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < 16; ++s) {
        const float e = s == c16 ? 1.f : s < c16 ? m[(16 + s) * LS + 16 + c16] : 0.f;
        y -= e * load4(m + s * LS + 16 + 4 * g);
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
#pragma unroll
      for (int i = 0; i < 4; ++i) m[(4 * g + i) * LS + 16 + c16] = y[i];
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      float4_ inv[2];
      const int t = 16 * u + c16;
#pragma unroll
      for (int v = 0; v < 2; ++v)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int s = 16 * v + 4 * g + i;
          inv[v][i] = (s < t ? m[s * LS + t] : s == t ? 1.f : 0.f) * beta[s];
        }
      put(HU::tf + u * 128, split8(inv[0], inv[1]));
    }
  }
}

// x + its neighbours, inside 8 or 16 lanes
template <int CTRL>
__device__ __forceinline__ float add_dpp(float x) {
  return x + __uint_as_float(__builtin_amdgcn_update_dpp(0u, __float_as_uint(x), CTRL, 0xf, 0xf, true));
}
template <int N>
__device__ __forceinline__ float lanes_sum(float x) {
  x = add_dpp<0xB1>(x);                           // quad_perm 1 0 3 2
  x = add_dpp<0x4E>(x);                           // quad_perm 2 3 0 1
  x = add_dpp<0x141>(x);                          // mirror of 8 lanes
  if constexpr (N >= 16) x = add_dpp<0x140>(x);   // mirror of 16 lanes
  if constexpr (N >= 32) x += __shfl_xor(x, 16, 64);
  return x;
}

typedef short s4v __attribute__((ext_vector_type(4)));

// 16 bytes a lane to LDS at the wave-uniform byte address `lds`, lane after lane.  Written out, so that the compiler does not wait
// for it before every read of LDS: the caller waits (vmcnt) before the barrier after which the data are read.
__device__ __forceinline__ void dma16_unwaited(const uint4_* src, uint32_t lds) {
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(lds), "v"(src) : "memory", "m0");
}
__device__ __forceinline__ void wait_vm() {
  __builtin_amdgcn_s_waitcnt(0x0f70);             // vmcnt(0)
  asm volatile("" ::: "memory");
}
__device__ __forceinline__ uint32_t lds_address(const void* p) {
  return (uint32_t)(uintptr_t)(__attribute__((address_space(3))) const void*)p;
}

// Segment j of sequence b: its last state L [DK][DV], after `link` the next segment's first; of the delta rule then M [DK][DK].
__device__ __forceinline__ float* segment_unit(const RuleArgs& p, int b, int j, int head, long size) {
  return p.seg_ws + (((long)p.q_start[b] / p.seg + b + j) * p.heads + head) * size;
}

// Waves of 16 columns of S each.  A prepared chunk goes to LDS by DMA, one chunk ahead where two fit (AHEAD).
// TOTALS: L and M of every segment but a sequence's last.
template <int MODE, int DK, int DV, bool AHEAD, bool TOTALS>
__global__ void __launch_bounds__(DV * 4) __attribute__((amdgpu_waves_per_eu(DV / 64, DV / 64)))
rule_scan_kernel(const RuleArgs p) {
  constexpr bool DELTA = MODE != kRetention, CHANNEL = MODE == kChannel;
  using U = RowUnit<DK, CHANNEL>;
  using HU = HeadUnit<DV>;
  constexpr int NW = DV / 16, NI = DK / 32, NK = DK / 16, LO = DV + 4, TPR = DV / 8;
  constexpr int FH = DELTA ? 0 : HU::pf;          // what retention does not use is not loaded
  constexpr int SIZE = U::size + HU::size;
  extern __shared__ __attribute__((aligned(16))) uint4_ staged[];
  // [32][LO] outputs: behind the chunks or, with one, in its place (used up by then)
  float* so = reinterpret_cast<float*>(AHEAD ? staged + 2 * SIZE : staged);
  static_assert(kC * LO * 4 <= SIZE * 16, "outputs in place of the chunk");
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int g = lane >> 4, c16 = lane & 15;
  // heads that share rows follow each other on one XCD (workgroups go round them)
  constexpr int KINDS = TOTALS && DELTA ? 1 + (DK + DV - 1) / DV : 1;     // L, then DV columns of M each
  constexpr long SEGMENT = DK * (DELTA ? DV + DK : DV);
  const int cuts = TOTALS ? p.cuts - 1 : p.cuts;
  const int jobs = p.heads * p.B * cuts * KINDS, q8 = jobs >> 3, r8 = jobs & 7, xcd = blockIdx.x & 7;
  const int job = (xcd < r8 ? xcd * (q8 + 1) : r8 * (q8 + 1) + (xcd - r8) * q8) + (blockIdx.x >> 3);
  const int unit = job / p.heads, hi = job % p.heads, h = p.head0 + hi, group = CHANNEL ? 1 : p.H / p.G;
  const int kind = unit % KINDS, j0 = unit / KINDS % cuts, b = unit / KINDS / cuts;
  const long begin = (long)j0 * p.seg, left = p.q_lens[b] - begin;
  if (left < 1 || (TOTALS && (left <= p.seg || (kind && j0 == 0)))) return;
  const int total = (int)min(left, (long)p.seg);
  const int chunks = (total + kC - 1) / kC;
  const long row0 = p.q_start[b] + begin;
  const int slot = p.slots[b];
  const bool old = slot >= 0 && p.pos[p.q_start[b]] > 0;
  float* st = p.state + ((long)max(slot, 0) * p.H + h) * DK * DV + 16 * w + c16;

  const int keys = p.heads / group;
  const long chunk0 = first_chunk(p, b) + begin / kC;
  const uint4_* head = head_unit(p, chunk0, hi, HU::size) + lane;
  const uint4_* rows = row_unit(p, chunk0, hi / group, keys, U::size, HU::size) + lane;
  const uint32_t at0 = __builtin_amdgcn_readfirstlane(lds_address(staged));
  auto stage = [&](int c) {
    const uint32_t dst = at0 + (AHEAD && (c & 1) ? SIZE * 16 : 0);
    const uint4_* su = rows + (long)c * keys * U::size;
    const uint4_* sh = head + (long)c * p.heads * HU::size;
#pragma unroll
    for (int j = 0; j < (U::size / 64 + NW - 1) / NW; ++j) {
      const int i = j * NW + w;
      if (i < U::size / 64 && !(TOTALS && 64 * i >= U::qd && 64 * i < U::qd + U::part)) dma16_unwaited(su + 64 * i, dst + 1024 * i);
    }
#pragma unroll
    for (int j = 0; j < ((HU::size - FH) / 64 + NW - 1) / NW; ++j) {
      const int i = FH / 64 + j * NW + w;
      if (i < HU::size / 64) dma16_unwaited(sh + 64 * i, dst + U::size * 16 + 1024 * i);
    }
  };
  stage(0);
  float4_ S[NK];                                  // rows 16 i + 4 g .., the wave's columns
  if (TOTALS && kind) {
#pragma unroll
    for (int i = 0; i < NK; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) S[i][j] = 16 * i + 4 * g + j == (kind - 1) * DV + 16 * w + c16 ? 1.f : 0.f;
  } else {
    const bool linked = !TOTALS && j0 > 0;
    const float* from = linked ? segment_unit(p, b, j0 - 1, hi, SEGMENT) + 16 * w + c16 : st;
    const bool some = linked || (old && j0 == 0);
#pragma unroll
    for (int i = 0; i < NK; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) S[i][j] = some ? from[(long)(16 * i + 4 * g + j) * DV] : 0.f;
  }
  // pieces of this lane: 16 bytes of row c16, 8 bytes of row 4 g + tq (channels 32 i ..: i even, odd), and of its values
  const int tq = c16 >> 2, tp = c16 & 3;
  int row_at[2], col_at[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    row_at[i] = c16 * (DK / 8) + ((4 * i + g) ^ (c16 & 7));
    col_at[i] = (4 * g + tq) * (DK / 4) + 2 * ((4 * i + tp) ^ (4 * (g & 1) + tq));
  }
  const int value_at = (4 * g + tq) * (DV / 4) + 4 * ((w & 3) ^ tq) + 16 * (w >> 2) + (tp ^ g);
  // epilogue: a thread's row of the chunk and 8 columns
  const int er = tid / TPR, ec = tid % TPR * 8;
  float gain[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) gain[i] = DELTA && !TOTALS ? p.gain[ec + i] : 1.f;
  const float inv_vdim = 1.f / (float)p.vdim;
  const bf16_t* gate = static_cast<const bf16_t*>(p.gate) + row0 * p.ldg + h * DV + ec;
  bf16_t* out = static_cast<bf16_t*>(p.out) + row0 * p.ldo + h * DV + ec;
  wait_vm();
  __syncthreads();
  for (int c = 0; c < chunks; ++c) {
    const uint4_* cur = staged + (AHEAD ? (c & 1) * SIZE : 0);
    const uint4_* curh = cur + U::size;
    const int t = c * kC + er;
    uint4_ z = {};
    if constexpr (!TOTALS) z = *reinterpret_cast<const uint4_*>(gate + (long)min(t, total - 1) * p.ldg);
    if (AHEAD && c + 1 < chunks) stage(c + 1);
    auto frag = [&](int place) {
      return Split{__builtin_bit_cast(bf16x8, curh[place + lane]), __builtin_bit_cast(bf16x8, curh[place + 64 + lane])};
    };
    // row 16 u + c16: channels 32 i + 4 g .. and 32 i + 16 + 4 g ..
    auto row = [&](int place, int u, int i) {
      const uint4_* m = cur + place + u * 2 * DK + 8 * (i >> 1) + row_at[i & 1];
      return Split{__builtin_bit_cast(bf16x8, m[0]), __builtin_bit_cast(bf16x8, m[4 * DK])};
    };
    // a column, 8-byte piece `at` in rows of n: times 4 g .. and 16 + 4 g ..
    auto column = [&](const uint4_* part, int n, int at) {
      const uint2_* m = reinterpret_cast<const uint2_*>(part) + at;
      const s4v lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4v*)(m));
      const s4v hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4v*)(m + 16 * n));
      const uint2_ a = __builtin_bit_cast(uint2_, lo), b2 = __builtin_bit_cast(uint2_, hi);
      return uint4_{a[0], a[1], b2[0], b2[1]};
    };
    auto key_column = [&](int i) {                // channel 16 i + c16
      uint4_ y[2];
#pragma unroll
      for (int v = 0; v < 2; ++v) y[v] = column(cur + U::ke + v * 4 * DK, DK / 4, col_at[i >> 1 & 1] + 16 * (i >> 2) + (i & 1));
      return Split{__builtin_bit_cast(bf16x8, y[0]), __builtin_bit_cast(bf16x8, y[1])};
    };
    // Operands are read from LDS a step ahead of the products that use them; independent sums take turns.
    auto hold = [] {
      if constexpr (AHEAD) __builtin_amdgcn_sched_barrier(0);
    };
    constexpr int NR = (DELTA ? 2 : 0) + (TOTALS ? 0 : 2);     // sums of a step: K S (rows 0 .., 16 ..), then Q S
    float4_ acc[NR + 1] = {};
    Split f[NI][NR + 1];
    auto load_rows = [&](int i) {
#pragma unroll
      for (int j = 0; j < NR; ++j) f[i][j] = row(DELTA && j < 2 ? U::kd : U::qd, j & 1, i);
    };
    if constexpr (NR > 0) load_rows(0);
#pragma unroll
    for (int i = 0; i < (NR > 0 ? NI : 0); ++i) {
      if (i + 1 < NI) load_rows(i + 1);
      hold();
      const Split sf = split8(S[2 * i], S[2 * i + 1]);
#pragma unroll
      for (int j = 0; j < NR; ++j) acc[j] = mac(f[i][j].hi, sf.hi, acc[j]);
#pragma unroll
      for (int j = 0; j < NR; ++j) acc[j] = mac(f[i][j].lo, sf.hi, acc[j]);
#pragma unroll
      for (int j = 0; j < NR; ++j) acc[j] = mac(f[i][j].hi, sf.lo, acc[j]);
    }
    float4_* O = acc + (DELTA ? 2 : 0);           // not with TOTALS
    const float* dec = reinterpret_cast<const float*>(curh + HU::dec);
    const uint4_ vr = column(curh + HU::vf, DV / 4, value_at);
    Split pf[2], tf[2];
    if constexpr (!TOTALS) {
      pf[0] = frag(HU::pf);
      pf[1] = frag(HU::pf + 128);
    }
    if constexpr (DELTA) {
      tf[0] = frag(HU::tf);
      tf[1] = frag(HU::tf + 128);
    }
    float4_ from[2], to[2];
    float all = 0.f;
    if constexpr (!CHANNEL) {
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        from[u] = load4(dec + 16 * u + 4 * g);
        to[u] = load4(dec + 32 + 16 * u + 4 * g);
      }
      all = dec[64];
    }
    Split kc[NK];
    float4_ kdec[CHANNEL ? NK : 1];
    auto load_keys = [&](int i) {
#pragma unroll
      for (int j = i; j < i + 2 && j < NK; ++j) {
        kc[j] = key_column(j);
        if constexpr (CHANNEL) kdec[j] = load4(dec + 16 * j + 4 * g);
      }
    };
    load_keys(0);
    hold();
    float4_ v[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      v[u] = float4_{__uint_as_float(vr[2 * u] << 16), __uint_as_float(vr[2 * u] & 0xffff0000u),
                     __uint_as_float(vr[2 * u + 1] << 16), __uint_as_float(vr[2 * u + 1] & 0xffff0000u)};
      if (TOTALS && kind) v[u] = float4_{0.f, 0.f, 0.f, 0.f};
      if constexpr (!CHANNEL) {                   // decays from the chunk's start
        if constexpr (DELTA) acc[u] *= from[u];
        if constexpr (!TOTALS) O[u] *= from[u];
      }
    }
    Split uf;                                     // U, its rows decayed to the chunk's end for the state
    if constexpr (DELTA) {
      const Split rf = split8(v[0] - acc[0], v[1] - acc[1]);
#pragma unroll
      for (int u = 0; u < 2; ++u) v[u] = mac(tf[u].hi, rf.hi, float4_{0.f, 0.f, 0.f, 0.f});
#pragma unroll
      for (int u = 0; u < 2; ++u) v[u] = mac(tf[u].lo, rf.hi, v[u]);
#pragma unroll
      for (int u = 0; u < 2; ++u) v[u] = mac(tf[u].hi, rf.lo, v[u]);
      uf = split8(v[0], v[1]);
      if constexpr (!TOTALS) {
#pragma unroll
        for (int u = 0; u < 2; ++u) O[u] = mac(pf[u].hi, uf.hi, O[u]);
#pragma unroll
        for (int u = 0; u < 2; ++u) O[u] = mac(pf[u].lo, uf.hi, O[u]);
#pragma unroll
        for (int u = 0; u < 2; ++u) O[u] = mac(pf[u].hi, uf.lo, O[u]);
      }
    } else if constexpr (!TOTALS) {
      const bf16x8 vf = __builtin_bit_cast(bf16x8, vr);
#pragma unroll
      for (int u = 0; u < 2; ++u) O[u] = mac(pf[u].hi, vf, O[u]);
#pragma unroll
      for (int u = 0; u < 2; ++u) O[u] = mac(pf[u].lo, vf, O[u]);
    }
    if constexpr (!CHANNEL) uf = split8(v[0] * to[0], v[1] * to[1]);
#pragma unroll
    for (int i = 0; i < NK; i += 2) {             // two tiles of the state at a time
      load_keys(i + 2);
      hold();
#pragma unroll
      for (int j = i; j < i + 2; ++j) {
        if constexpr (CHANNEL) S[j] *= kdec[j];
        else S[j] *= all;
      }
#pragma unroll
      for (int j = i; j < i + 2; ++j) S[j] = mac(kc[j].hi, uf.hi, S[j]);
#pragma unroll
      for (int j = i; j < i + 2; ++j) S[j] = mac(kc[j].lo, uf.hi, S[j]);
#pragma unroll
      for (int j = i; j < i + 2; ++j) S[j] = mac(kc[j].hi, uf.lo, S[j]);
    }

    if constexpr (TOTALS) {
      if constexpr (!AHEAD) {
        __syncthreads();
        if (c + 1 < chunks) stage(c + 1);
      }
      wait_vm();
      __syncthreads();
      continue;
    }
    __syncthreads();                              // every wave is done with the chunk and the last one's outputs
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int j = 0; j < 4; ++j) so[(16 * u + 4 * g + j) * LO + 16 * w + c16] = O[u][j];
    if constexpr (AHEAD) wait_vm();
    __syncthreads();
    // every head's norm, gain and gate
    float y[8], zf[8], ss = 0.f;
    *reinterpret_cast<float4_*>(y) = load4(so + er * LO + ec);
    *reinterpret_cast<float4_*>(y + 4) = load4(so + er * LO + ec + 4);
    if constexpr (!AHEAD) {
      __syncthreads();
      if (c + 1 < chunks) stage(c + 1);
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) ss += y[i] * y[i];
    const float r = __builtin_amdgcn_rsqf(lanes_sum<TPR>(ss) * inv_vdim + p.eps);
    unpack8(z, zf);
#pragma unroll
    for (int i = 0; i < 8; ++i) y[i] *= r * gain[i] * gate_act<true>(zf[i], p.gate_kind);
    if (t < total) *reinterpret_cast<uint4_*>(out + (long)t * p.ldo) = pack8(y);
    if constexpr (!AHEAD) {
      wait_vm();
      __syncthreads();
    }
  }
  if constexpr (TOTALS) {
    const int col = (kind ? (kind - 1) * DV : 0) + 16 * w + c16, width = kind ? DK : DV;
    float* to = segment_unit(p, b, j0, hi, SEGMENT) + (kind ? DK * DV : 0) + col;
    if (col < width) {
#pragma unroll
      for (int i = 0; i < NK; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) to[(long)(16 * i + 4 * g + j) * width] = S[i][j];
    }
  } else if (slot >= 0 && left <= p.seg) {
#pragma unroll
    for (int i = 0; i < NK; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) st[(long)(16 * i + 4 * g + j) * DV] = S[i][j];
  }
}

// The first state of every segment but a sequence's first: S = M S + L, fp32.  A workgroup per sequence, head and 16 columns, a
// wave per 16 rows.
template <bool DELTA, int DK, int DV>
__global__ void __launch_bounds__(DK * 4) rule_link_kernel(const RuleArgs p) {
  constexpr long SEGMENT = DK * (DELTA ? DV + DK : DV);
  constexpr int NQ = DELTA ? DK / 16 : 1;
  __shared__ __attribute__((aligned(16))) float x[DELTA ? 16 * (DK + 4) : 1];      // the state, a column after the other
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, g = lane >> 4, c16 = lane & 15;
  const int b = blockIdx.z, hi = blockIdx.y, col = blockIdx.x * 16 + c16;
  const int total = p.q_lens[b], links = (total - 1) / p.seg;                      // segments with one behind them
  if (links < 2) return;
  auto unit = [&](int j) { return segment_unit(p, b, j, hi, SEGMENT); };
  auto last = [&](int j) {
    float4_ y;
#pragma unroll
    for (int i = 0; i < 4; ++i) y[i] = unit(j)[(long)(16 * w + 4 * g + i) * DV + col];
    return y;
  };
  float4_ S = last(0);
  const float fixed = DELTA ? 0.f : __builtin_amdgcn_exp2f((float)p.seg * fmaxf(p.rate[p.H + p.head0 + hi], kLeast));
  for (int j = 1; j < links; ++j) {
    float4_ next = last(j);
    if constexpr (DELTA) {
      float4_ m[NQ];
#pragma unroll
      for (int q = 0; q < NQ; ++q) m[q] = load4(unit(j) + DK * DV + (16 * w + c16) * DK + 16 * q + 4 * g);
      __syncthreads();                            // the last state is read
      *reinterpret_cast<float4_*>(x + c16 * (DK + 4) + 16 * w + 4 * g) = S;
      __syncthreads();
#pragma unroll
      for (int q = 0; q < NQ; ++q) {
        const float4_ y = load4(x + c16 * (DK + 4) + 16 * q + 4 * g);
#pragma unroll
        for (int i = 0; i < 4; ++i) next = __builtin_amdgcn_mfma_f32_16x16x4f32(m[q][i], y[i], next, 0, 0, 0);
      }
    } else {
      next += fixed * S;
    }
    S = next;
#pragma unroll
    for (int i = 0; i < 4; ++i) unit(j)[(long)(16 * w + 4 * g + i) * DV + col] = S[i];
  }
}

template <int MODE, int DK, int DV, bool AHEAD>
static void scan(const RuleArgs& a, hipStream_t s) {
  constexpr bool DELTA = MODE != kRetention;
  constexpr int unit = (RowUnit<DK, MODE == kChannel>::size + HeadUnit<DV>::size) * 16;
  constexpr int lds = AHEAD ? 2 * unit + kC * (DV + 4) * 4 : unit;
  static_assert(lds <= 160 * 1024, "prepared chunks in LDS");
  if (a.cuts > 1) {
    constexpr int kinds = DELTA ? 1 + (DK + DV - 1) / DV : 1;
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(rule_scan_kernel<MODE, DK, DV, AHEAD, true>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    rule_scan_kernel<MODE, DK, DV, AHEAD, true><<<a.heads * a.B * (a.cuts - 1) * kinds, DV * 4, lds, s>>>(a);
    rule_link_kernel<DELTA, DK, DV><<<dim3(DV / 16, a.heads, a.B), DK * 4, 0, s>>>(a);
  }
  (void)hipFuncSetAttribute(reinterpret_cast<const void*>(rule_scan_kernel<MODE, DK, DV, AHEAD, false>),
                            hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  rule_scan_kernel<MODE, DK, DV, AHEAD, false><<<a.heads * a.B * a.cuts, DV * 4, lds, s>>>(a);
}

long rule_segment_bytes(int dk, int dv, int heads, bool retention) { return 4L * heads * dk * (retention ? dv : dv + dk); }

template <int MODE, int DK, int DV>
static void chunks(const RuleArgs& a, hipStream_t s) {
  const int n = (a.max_q + kC - 1) / kC;
  if constexpr (MODE == kChannel) {
    constexpr int lds = 4 * (3 * kC * (DK + 4) + kC + 24 * DK);
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(rule_prep_channel_kernel<DK, DV>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    rule_prep_channel_kernel<DK, DV><<<dim3(n, a.heads, a.B), 512, lds, s>>>(a);
  } else {
    constexpr bool DELTA = MODE == kHead;
    constexpr int lds = 2 * 4 * kC * (DK + 8);
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(rule_prep_head_kernel<DELTA, DK, DV>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    rule_prep_head_kernel<DELTA, DK, DV><<<dim3(n, a.heads / (a.H / a.G), a.B), 512, lds, s>>>(a);
  }
  rule_solve_kernel<MODE, DK, DV><<<dim3((n + 3) / 4, a.heads, a.B), 256, 0, s>>>(a);
  scan<MODE, DK, DV, (DK <= 128)>(a, s);
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
