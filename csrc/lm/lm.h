// Launchers of the decoder-block kernels (libshai_lm.so): decoders with an fp32 residual stream, mixture-of-experts
// layers, chunked and latent attention, and gated recurrences.  Every kernel takes bf16 or fp32 weights / activations
// (`f32`); norms, routing, scores, recurrent state and the residual are fp32 in both.  The model width is padded to a multiple of 64 by the caller.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace shai_lm {

struct EmbedNormArgs {
  const int* ids;
  const int* prev;         // preceding token of each row, -1 at a sequence's start
  const void* table;       // [V, Dp]
  const void* bigram;      // [buckets + 1, Dp] or null
  long mul_prev, mul_cur, buckets;
  const float* w;          // norm weight (gain - 1)
  float eps;
  int T, V, Dp, width;
  float* x;                // [T, Dp]
  void* h;                 // [T, Dp]
};
void launch_embed_norm(const EmbedNormArgs& a, bool f32, hipStream_t s);

struct AddNormArgs {
  float* x;                // [*, Dp] residual, updated in place unless `rows` is set
  const void* dense;       // [*, Dp] added, or null
  const void* ye;          // [slots, Dp] expert outputs, or null
  const int* slot_of;      // [*, top]
  const float* wts;        // [*, top]
  int top;
  const float* inject;     // [*, Dp] fp32 added, or null
  const int* rows;         // optional: normalise only these rows
  const float* w;          // norm weight (gain - 1), or null: no norm output
  float eps;
  int T, Dp, width;
  void* h;                 // [T, Dp]
};
void launch_add_norm(const AddNormArgs& a, bool f32, hipStream_t s);

// Residual add with a norm of its own, the next sublayer's norm, and its input convolution:
//   x' = x + mult * norm(delta) wb (+ bb) (+ step),   h = norm(x') w (+ b),   h += causal convolution of h over time
// Every part but the source of x may be absent.  A norm with a bias is a layer norm (mean taken off), one without is an
// RMS norm; h without w is x' itself.
struct ResidualNormArgs {
  const float* x;          // [*, Dp], or null: x = table[ids] * scale
  const int* ids;
  const void* table;       // [V, Dp]
  float scale;
  int V;
  const void* delta;       // [*, Dp] sublayer output, or [parts, *, Dp] fp32 partial sums of it, or null
  int parts;               // 0: delta is of the type of h
  long part_stride;
  const void* ye;          // [slots, Dp] expert outputs, their weighted sum added to delta, or null
  const int* slot_of;      // [*, top]
  const float* wts;        // [*, top]
  int top;
  const float* wb;         // its norm's gain, or null: added without a norm
  const float* bb;         // its norm's bias, or null
  float mult;
  const float* step;       // [Dp] added to every row, or null
  float* x_out;            // [*, Dp], or null
  const int* rows;         // optional: only these rows (no convolution)
  const float* w;          // gain, or null: no norm
  const float* b;          // bias, or null
  float eps;
  int T, Dp, width;
  void* h;                 // [T, Dp], or null
  // convolution (cw null: none)
  const float* cw;         // [taps, Dp], oldest tap first
  int taps;
  float* state;            // [slots, taps - 1, Dp]: the last inputs of every sequence, oldest first
  float* tail;             // [B, taps - 1, Dp]: this step's last inputs (prefill); null: decode, state updated in place
  const int* row_seq;      // prefill: sequence of every row
  const int* q_start;      // prefill: [B] first row
  const int* q_lens;       // prefill: [B]
  const int* pos;          // [T]
  const int* slots;        // [B] state slot, -1: none
  int B, run;              // rows per workgroup
};
void launch_residual_norm(const ResidualNormArgs& a, bool f32, hipStream_t s);   // run <= 64

struct ConvCommitArgs {    // the tails of a prefill step into the state of every layer run
  float* state;            // [runs, slots, taps - 1, Dp]
  const float* tail;       // [runs, B, taps - 1, Dp]
  const int* q_lens;
  const int* slots;
  int runs, n_slots, B, taps, Dp;
};
void launch_conv_commit(const ConvCommitArgs& a, hipStream_t s);

struct RopeRowsArgs {      // cos / sin of pos * freq, every row of a step
  const int* pos;
  const float* freq;       // [n][2]: frequency as a float and its remainder
  int T, n;
  float* out;              // [T, n, 2]
};
void launch_rope_rows(const RopeRowsArgs& a, hipStream_t s);

enum Epi : int { EPI_NONE = 0, EPI_CLAMP_GLU = 1, EPI_SOFTCAP = 2, EPI_XIELU = 3, EPI_ROTARY = 4, EPI_GELU_GLU = 5,
                 EPI_RELU2 = 6, EPI_GELU_ROWS = 7 };
constexpr __host__ __device__ bool glu_epi(int epi) { return epi == EPI_CLAMP_GLU || epi == EPI_GELU_GLU; }
// The bf16 kernels are compiled per class of epilogues: code of the others costs a kernel registers and instruction cache.
enum EpiClass : int { EC_PLAIN = 0, EC_CLAMP = 1, EC_GELU = 2, EC_OTHER = 3, EC_ANY = 4 };
constexpr __host__ __device__ int epi_class(int epi) {
  return epi == EPI_NONE || epi == EPI_RELU2 ? EC_PLAIN : epi == EPI_CLAMP_GLU ? EC_CLAMP
         : epi == EPI_GELU_GLU || epi == EPI_GELU_ROWS ? EC_GELU : EC_OTHER;
}
constexpr __host__ __device__ bool epi_in(int ec, int epi) { return ec == EC_ANY || ec == epi_class(epi); }
constexpr __host__ __device__ bool glu_class(int ec) { return ec == EC_ANY || ec == EC_CLAMP || ec == EC_GELU; }
struct GemmArgs {
  const void* A;           // [rows, K]
  const void* W;           // [N, K] or [E, N, K]
  void* C;                 // [M, N'] bf16, or fp32
  const int* tiles;        // grouped: [n_tiles][2] = (expert or -1, first slot)
  const int* offsets;      // grouped: [E + 1] first slot of every expert
  const int* gather;       // grouped, optional: A row of every slot
  int M, N, K;
  int n_tiles;
  int a_rows;              // rows of A
  int bm;                  // grouped row tile (16, 128 or 256)
  int epi;
  float param;
  int n_main;              // columns n_main .. N - 1 are a plain fp32 product, stored in side [M, N - n_main]
  float* side;
  int n_act;               // columns from n_act on are plain (EPI_RELU2 only; n_main: none)
  bool out_f32;
  long lda, ldc;           // row strides of A and C
  int splits;              // K cut into this many parts over blockIdx.z: C [splits, M, N] fp32 partial sums
  int batch;               // dense: products batched over blockIdx.z (streaming kernel only)
  long a_batch, w_batch, c_batch;
  const float* vec;        // EPI_XIELU: (alpha_p, alpha_n)
  const float* rope;       // EPI_ROTARY: [M, rot] cos / sin pairs; columns rot0 .. rot0 + rot - 1 of every `head` columns
  int head, rot0, rot;
  const int* ids;          // EPI_GELU_ROWS: [M] row of `table` (the type of A) that multiplies row m
  const void* table;       // [table_rows, N] with rows table_ld apart
  long table_ld;
  int table_rows;
  bool table_f32;
};
void launch_gemm(const GemmArgs& a, bool f32, hipStream_t s);          // streaming kernel, any M
void launch_gemm_tile(const GemmArgs& a, hipStream_t s);               // LDS-tiled bf16 kernel (gemm_tile.hip)

struct RouteArgs {
  const float* logits;     // [T, E]
  int T, E, top, groups, keep;
  int* ids;                // [T, top]
  float* wts;              // [T, top]
  const float* bias;       // [E] added to the logits, or null
  bool renorm;             // weights: softmax over the chosen logits only (else their share of all experts' softmax)
};
void launch_route(const RouteArgs& a, hipStream_t s);

struct PlanArgs {
  const int* ids;          // [P] expert of every (token, k) pair
  int P, top, E, bm, n_tiles;
  int* offsets;            // [E + 1]
  int* token_of;           // [P]
  int* slot_of;            // [P]
  int* tiles;              // [n_tiles][2]
};
void launch_plan(const PlanArgs& a, hipStream_t s);
void launch_route_plan(const RouteArgs& r, const PlanArgs& a, hipStream_t s);   // T <= 16, E <= 256

struct AttnArgs {
  const void* qkvg;        // [T, ld]: q (H dk), k (G dk), v (G dv), gate logits (H gate_w)
  long ld, ldo;            // row strides of qkvg and o
  int v_off;               // column of the values (that of the keys where those are the values)
  int gate_off, gate_w;    // column of the gate logits; 1 per head or dv of them, 0: no gate
  bool own_kv;             // rows hold k and v (else another layer's are in the cache, and the gate follows q)
  bool window;             // a position sees itself and the chunk - 1 before it (else its own chunk)
  const float* rope;       // [T, rot] cos / sin of every row, or null: q and k are used as they are.  Otherwise dimension
  int rot, dim;            // i < rot / 2 of a head is turned with i + rot / 2, and the head divided by its rms over `dim`
  float eps;
  const float* q_gain;     // [dk], or null: with gains the norm comes first, then the rotation
  const float* k_gain;
  const float* temp;       // [H] factor on a head's scores, or null
  float out_scale;         // factor on the output where there is no gate
  void* kc;                // [blocks, G, 64, dk]
  void* vc;                // [blocks, G, 64, dv]
  void* o;                 // [T, H dv]
  const int* bt;           // [B, max_blocks]
  const int* ctx;          // [B] context length incl. this step's tokens
  const int* q_lens;       // [B], null: one row per sequence (decode)
  const int* q_start;      // [B]
  const int* slots;        // [T] cache slot of every row, -1: none
  float* ws;               // decode split partials
  int B, T, max_q, H, G, dk, dv, max_blocks, splits, chunk;
  float scale;
  // latent form of the prefill kernel: q rows at `qkvg`; keys of sequence b are rows kv_start[b] ..; a key is
  // [kv[0 .. np) | lat[rank .. )], its value kv[np .. np + dv)
  const void* kv;          // [rows, H, np + dv]
  const void* lat;         // [rows, lat_ld]
  const int* kv_start;
  const float* sink;       // [H] exp(sink) is added to a head's denominator; or null (not in the latent form)
  int np, rank, lat_ld, lat_pad;   // lat_pad: the last column after `rank` from which 8 values may be read
};
void launch_kv_store(const AttnArgs& a, bool f32, hipStream_t s);
void launch_head_prep(const AttnArgs& a, bool f32, hipStream_t s);     // q in place, k (turned, normed) and v to the cache
void launch_attn_prefill(const AttnArgs& a, bool f32, hipStream_t s);
void launch_attn_decode(const AttnArgs& a, bool f32, hipStream_t s);
void launch_latent_prefill(const AttnArgs& a, hipStream_t s);          // bf16

struct LatentPrepArgs {
  const float* d;          // [parts, T, qp + rp + op], summed over parts: query latent, key/value latent, rotated key part
  const float* wq;         // [qp] gains (zero in the pads)
  const float* wkv;        // [rp]
  const float* rope;       // [T, rot]
  const int* slots;        // [T] cache slot, -1: none
  void* cache;             // [blocks, 64, rp + op]
  void* cq;                // [T, qp]
  float eps;
  int T, parts, q_rank, kv_rank, rot, qp, rp, op;
};
void launch_latent_prep(const LatentPrepArgs& a, bool f32, hipStream_t s);

struct LatentGatherArgs {  // cached rows of the listed sequences, back to back
  const void* cache;       // [blocks, 64, ld]
  void* out;               // [rows, ld]
  const int* bt;           // [B, max_blocks]
  const int* seqs;         // [n]
  const int* ctx;          // [n]
  const int* start;        // [n] first output row
  int n, max_ctx, max_blocks, ld_bytes;
};
void launch_latent_gather(const LatentGatherArgs& a, hipStream_t s);

struct LatentArgs {        // attention of single rows over the cached latents
  const void* ql;          // [n, H, rp] queries in latent space
  const void* q;           // [n, ldq]: the rotated part of head h at h * head + np
  const void* cache;       // [blocks, 64, rp + op]
  void* o;                 // [n, H, rp]
  const int* bt;           // [B, max_blocks]
  const int* seqs;         // [n] block table row of every entry, or null: entry i
  const int* ctx;          // [n] keys that an entry sees
  const float* sink;       // [H]
  float* ws;               // [n, H, splits, rp + 4]: partial output, maximum, denominator
  float scale;
  long ldq;
  int n, H, head, np, rot, rp, op, max_blocks, splits;
};
bool latent_decode_fits(int rp, int op);
void launch_latent_decode(const LatentArgs& a, hipStream_t s);         // bf16, sizes that fit
void launch_latent_rows(const LatentArgs& a, bool f32, hipStream_t s); // any size

struct ScanArgs {          // minGRU: S = (1 - z) S + z c, out = S silu(g)
  const float* zx;         // [T, 2 W]: z and u before their biases
  const void* g;           // [T, W]
  const float* bias;       // [2 W]
  float* state;            // [slots, W]
  void* out;               // [T, W]
  const int* pos;          // [T]
  const int* q_start;      // [B], null: one row per sequence (decode)
  const int* q_lens;
  const int* slots;        // [B], -1: none
  float* ws;               // [B, chunks, 2, W] when a sequence has several chunks
  int T, B, W, max_q, len, chunks;
};
void launch_mingru_scan(const ScanArgs& a, bool f32, hipStream_t s);

struct Hgrn2Args {         // S = diag(f) S + (1 - f) v^T, o = S^T silu(q), out = o / rms(o) gain, head by head
  const void* qv;          // [T, H dk + H dv]
  const float* z;          // [T, H dk] forget logits before their bias
  const float* bias;       // [H dk]
  const float* lower;      // [H dk] lower bound of f (1 in the pads)
  const float* gain;       // [dv] (0 in the pads)
  float* state;            // [slots, H, dk, dv]
  void* out;               // [T, H dv]
  const int* pos;          // [T]
  const int* q_start;      // [B], null: one row per sequence (decode)
  const int* q_lens;
  const int* slots;        // [B], -1: none
  float* ws;               // [B, segments, H, dk dv + dk] when a sequence has several segments
  int T, B, H, dk, dv, vdim, len, segments;   // len: rows of a segment, a multiple of 32
  float eps;
};
void launch_hgrn2_rows(const Hgrn2Args& a, bool f32, hipStream_t s);   // row by row
void launch_hgrn2_chunks(const Hgrn2Args& a, hipStream_t s);           // bf16, 32 rows at a time

struct RuleArgs {          // delta rule (mode 1: a decay per head, 2: per key channel) or retention (mode 0), see rule.hip
  int mode;
  const void* x;           // [T, 2 G dk + H dv]: projected q, k, v
  const void* gate;        // [T, H dv]
  const float* decay;      // [T, H] or [T, H dk] logits before their bias
  const float* beta;       // [T, H] logits
  long ldx, ldg, ldd, ldb, ldo;    // row strides
  const float* conv;       // [taps, channels of x], oldest tap first
  const float* rate;       // [H]; retention: [2, H] decays and their base-2 logarithms
  const float* bias;       // [H] or [H dk]
  const float* gain;       // [dv] (0 in the pads); retention: none
  const float* rope;       // retention: [T, rot] cos / sin
  void* ring;              // [slots, taps, channels] of the type of x
  float* state;            // [slots, H, dk, dv]
  void* out;               // [T, H dv]
  const int* pos;          // [T]
  const int* q_start;      // [B], null: one row per sequence (decode)
  const int* q_lens;
  const int* slots;        // [B], -1: none
  void* ws;                // chunks: ws_chunks = T / 32 + B prepared chunks (rule_chunk_bytes each)
  long ws_chunks;
  float* seg_ws;           // T / seg + B units (rule_segment_bytes each), if sequences are cut
  int seg, cuts;           // rows of a segment (a multiple of 32), segments of the longest sequence
  int T, B, H, G, dk, dv, dim, vdim, taps, rot, gate_kind, max_q, head0, heads;
  float eps;
};
void launch_rule_rows(const RuleArgs& a, bool f32, hipStream_t s);     // row by row
void launch_rule_chunks(const RuleArgs& a, hipStream_t s);             // bf16, 32 rows at a time; heads head0 .. of a prefill step
// workspace of one chunk of `heads` heads and `keys` heads of queries and keys (those of every head with a decay per channel)
long rule_chunk_bytes(int dk, int dv, int heads, int keys, bool channel);
// workspace of a segment of `heads` heads
long rule_segment_bytes(int dk, int dv, int heads, bool retention);

struct RingArgs {          // the last inputs of a prefill step into the rings
  const void* x;
  void* ring;
  const int* pos;
  const int* q_start;
  const int* q_lens;
  const int* slots;
  long ldx;
  int B, n_slots, taps, channels;
};
void launch_ring_commit(const RingArgs& a, bool f32, hipStream_t s);

}  // namespace shai_lm
