// Launchers of the decoder-block kernels (libshai_lm.so): decoders with an fp32 residual stream, mixture-of-experts
// layers and chunked attention.  Every kernel takes bf16 or fp32 weights / activations (`f32`); norms, routing, scores
// and the residual are fp32 in both.  The model width is padded to a multiple of 64 by the caller.
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

enum Epi : int { EPI_NONE = 0, EPI_CLAMP_GLU = 1, EPI_SOFTCAP = 2 };
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
  bool out_f32;
};
void launch_gemm(const GemmArgs& a, bool f32, hipStream_t s);          // streaming kernel, any M
void launch_gemm_tile(const GemmArgs& a, hipStream_t s);               // LDS-tiled bf16 kernel (gemm_tile.hip)

struct RouteArgs {
  const float* logits;     // [T, E]
  int T, E, top, groups, keep;
  int* ids;                // [T, top]
  float* wts;              // [T, top]
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
  const void* qkvg;        // [T, ld]: q (H dk), k (G dk), v (G dv), gate logits (H)
  long ld;
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
};
void launch_kv_store(const AttnArgs& a, bool f32, hipStream_t s);
void launch_attn_prefill(const AttnArgs& a, bool f32, hipStream_t s);
void launch_attn_decode(const AttnArgs& a, bool f32, hipStream_t s);

}  // namespace shai_lm
