// torch operator registrations of libshai_lm.so: the decoder-block kernels (csrc/lm) and the token-level ops every
// language model's step uses (sampler, token feedback).  Same rules as csrc/bindings.cpp: caller-allocated outputs, the
// current stream, no allocation or synchronisation, and every size a kernel relies on checked here before its launch.
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>
#include <torch/library.h>
#include <algorithm>

#include "kernels/launchers.h"
#include "lm/lm.h"

using at::Tensor;
using c10::optional;

namespace {
#define SHAI_CHECK(cond, ...) TORCH_CHECK(cond, "shai: ", __VA_ARGS__)

hipStream_t stream() { return c10::hip::getCurrentHIPStream().stream(); }

void check(const Tensor& t, at::ScalarType dt, const char* name) {
  SHAI_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == dt, name, " must be a contiguous GPU ", dt,
             " tensor, got ", t.scalar_type());
  SHAI_CHECK(t.numel() == 0 || reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0, name, " must be 16-byte aligned");
}
void check_f32(const Tensor& t, const char* name) {
  SHAI_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat && t.is_contiguous(), name, " must be contiguous f32 GPU");
}
void check_i32(const Tensor& t, const char* name) {
  SHAI_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::kInt, name, " must be contiguous int32 GPU");
}
// the op's element type: true for fp32, false for bf16
bool is_f32(const Tensor& t) {
  SHAI_CHECK(t.scalar_type() == at::kFloat || t.scalar_type() == at::kBFloat16, "bf16 or fp32, got ", t.scalar_type());
  return t.scalar_type() == at::kFloat;
}
void check_width(int64_t Dp, int64_t width) {
  SHAI_CHECK(Dp % 64 == 0 && Dp <= 16384 && width >= 1 && width <= Dp, "width ", width, " in rows of ", Dp,
             ": rows must be a multiple of 64 and at most 16384");
}

void embed_norm(const Tensor& ids, const optional<Tensor>& prev, const Tensor& table, const optional<Tensor>& bigram,
                int64_t mul_prev, int64_t mul_cur, const Tensor& w, double eps, int64_t width, const Tensor& x,
                const Tensor& h) {
  const auto dt = table.scalar_type();
  const bool f32 = is_f32(table);
  check_i32(ids, "ids");
  check(table, dt, "table");
  check(w, at::kFloat, "w");
  check(x, at::kFloat, "x");
  check(h, dt, "h");
  shai_lm::EmbedNormArgs a{};
  a.T = ids.numel();
  a.V = table.size(0);
  a.Dp = table.size(1);
  a.width = width;
  check_width(a.Dp, width);
  SHAI_CHECK(w.numel() == a.Dp && x.numel() == (long)a.T * a.Dp && h.numel() == x.numel(), "embed_norm shapes");
  a.ids = ids.data_ptr<int>();
  a.table = table.data_ptr();
  if (bigram) {
    check(*bigram, dt, "bigram");
    SHAI_CHECK(prev.has_value() && prev->numel() >= a.T, "the bigram embedding needs every row's preceding token");
    check_i32(*prev, "prev");
    SHAI_CHECK(bigram->dim() == 2 && bigram->size(0) >= 2 && bigram->size(1) == a.Dp && mul_prev >= 0 && mul_cur >= 0 &&
                   mul_prev < (1LL << 31) && mul_cur < (1LL << 31), "bigram table / multipliers");
    a.prev = prev->data_ptr<int>();
    a.bigram = bigram->data_ptr();
    a.buckets = bigram->size(0) - 1;
    a.mul_prev = mul_prev;
    a.mul_cur = mul_cur;
  }
  a.w = w.data_ptr<float>();
  a.eps = eps;
  a.x = x.data_ptr<float>();
  a.h = h.data_ptr();
  if (a.T > 0) shai_lm::launch_embed_norm(a, f32, stream());
}

void add_norm(const Tensor& x, const optional<Tensor>& dense, const optional<Tensor>& ye,
              const optional<Tensor>& slot_of, const optional<Tensor>& wts, const optional<Tensor>& inject,
              const optional<Tensor>& rows, const optional<Tensor>& w, double eps, int64_t width,
              const optional<Tensor>& h) {
  check(x, at::kFloat, "x");
  shai_lm::AddNormArgs a{};
  const long R = x.size(0);
  a.Dp = x.size(1);
  a.width = width;
  check_width(a.Dp, width);
  a.x = x.data_ptr<float>();
  a.T = R;
  at::ScalarType dt = h ? h->scalar_type() : dense ? dense->scalar_type() : ye ? ye->scalar_type() : at::kFloat;
  if (dense) {
    check(*dense, dt, "dense");
    SHAI_CHECK(dense->size(0) == R && dense->size(1) == a.Dp, "dense must be [rows, D]");
    a.dense = dense->data_ptr();
  }
  if (ye) {
    SHAI_CHECK(slot_of.has_value() && wts.has_value(), "expert outputs need slot_of and weights");
    check(*ye, dt, "ye");
    check_i32(*slot_of, "slot_of");
    check(*wts, at::kFloat, "wts");
    a.top = slot_of->size(1);
    SHAI_CHECK(slot_of->size(0) == R && wts->sizes() == slot_of->sizes() && ye->size(0) == R * a.top &&
                   ye->size(1) == a.Dp, "expert outputs must be [rows * top, D]");
    a.ye = ye->data_ptr();
    a.slot_of = slot_of->data_ptr<int>();
    a.wts = wts->data_ptr<float>();
  }
  if (inject) {
    check(*inject, at::kFloat, "inject");
    SHAI_CHECK(inject->sizes() == x.sizes(), "inject must have x's shape");
    a.inject = inject->data_ptr<float>();
  }
  if (rows) {
    check_i32(*rows, "rows");
    SHAI_CHECK(w.has_value(), "rows selects rows to normalise");
    a.rows = rows->data_ptr<int>();
    a.T = rows->numel();
  }
  if (w) {
    check(*w, at::kFloat, "w");
    SHAI_CHECK(h.has_value() && w->numel() == a.Dp, "w must be [D], with an output h");
    check(*h, dt, "h");
    SHAI_CHECK(h->numel() == (long)a.T * a.Dp, "h must be [rows, D]");
    a.w = w->data_ptr<float>();
    a.h = h->data_ptr();
  }
  a.eps = eps;
  const bool f32 = dt == at::kFloat;
  SHAI_CHECK(f32 || dt == at::kBFloat16, "bf16 or fp32");
  if (a.T > 0) shai_lm::launch_add_norm(a, f32, stream());
}

void lm_gemm(const Tensor& A, const Tensor& W, const Tensor& C, const optional<Tensor>& tiles,
             const optional<Tensor>& offsets, const optional<Tensor>& gather, int64_t bm, int64_t epi, double param,
             const optional<Tensor>& side) {
  const bool f32 = is_f32(A);
  check(A, A.scalar_type(), "A");
  check(W, A.scalar_type(), "W");
  check(C, f32 || C.scalar_type() == at::kFloat ? at::kFloat : at::kBFloat16, "C");
  shai_lm::GemmArgs g{};
  SHAI_CHECK(A.dim() == 2 && C.dim() == 2 && (W.dim() == 2 || W.dim() == 3), "lm_gemm ranks");
  g.a_rows = A.size(0);
  g.M = C.size(0);
  g.N = W.size(-2);
  g.K = W.size(-1);
  g.epi = epi;
  g.param = param;
  g.out_f32 = C.scalar_type() == at::kFloat;
  SHAI_CHECK(A.size(1) == g.K && g.K % 64 == 0 && g.N >= 1, "lm_gemm: K must match and be a multiple of 64");
  SHAI_CHECK(epi >= 0 && epi <= 2, "lm_gemm epilogue");
  g.n_main = g.N;
  if (side) {  // the last rows of W are a plain product, stored in fp32
    check(*side, at::kFloat, "side");
    SHAI_CHECK(!tiles && epi == shai_lm::EPI_CLAMP_GLU && side->dim() == 2 && side->size(0) == g.M && side->size(1) >= 1 &&
                   side->size(1) < g.N, "side output: dense GLU products, [M, last rows of W]");
    g.n_main = g.N - side->size(1);
    SHAI_CHECK(g.n_main % 4 == 0, "side output: the GLU rows of W must be a multiple of 4");
    g.side = side->data_ptr<float>();
  }
  SHAI_CHECK(epi != shai_lm::EPI_CLAMP_GLU || g.n_main % 2 == 0, "GLU products need (gate, up) row pairs");
  SHAI_CHECK(C.size(1) == (epi == shai_lm::EPI_CLAMP_GLU ? g.n_main / 2 : g.N), "lm_gemm output columns");
  g.A = A.data_ptr();
  g.W = W.data_ptr();
  g.C = C.data_ptr();
  if (tiles) {
    SHAI_CHECK(offsets.has_value() && W.dim() == 3, "grouped lm_gemm: W [E, N, K], tiles and offsets");
    check_i32(*tiles, "tiles");
    check_i32(*offsets, "offsets");
    SHAI_CHECK(offsets->numel() == W.size(0) + 1 && (bm == 16 || bm == 128 || bm == 256), "grouped lm_gemm: offsets [E + 1], bm");
    g.tiles = tiles->data_ptr<int>();
    g.offsets = offsets->data_ptr<int>();
    g.n_tiles = tiles->size(0);
    g.bm = bm;
    if (gather) {
      check_i32(*gather, "gather");
      SHAI_CHECK(gather->numel() == g.M, "gather: one A row per output row");
      g.gather = gather->data_ptr<int>();
    } else {
      SHAI_CHECK(g.a_rows == g.M, "grouped lm_gemm without gather: A rows are the slots");
    }
  } else {
    SHAI_CHECK(W.dim() == 2 && g.a_rows == g.M, "dense lm_gemm: W [N, K], A [M, K]");
  }
  if (g.M == 0) return;
  const long lim = 0x7fffffffL;
  const bool tile = !f32 && (g.tiles ? bm >= 128 : g.M > 64) && (long)g.a_rows * g.K * 2 < lim &&
                    (long)g.N * g.K * 2 < lim;
  if (tile) shai_lm::launch_gemm_tile(g, stream());
  else shai_lm::launch_gemm(g, f32, stream());
}

void moe_route(const Tensor& logits, int64_t groups, int64_t keep, const Tensor& ids, const Tensor& wts) {
  check(logits, at::kFloat, "logits");
  check_i32(ids, "ids");
  check(wts, at::kFloat, "wts");
  shai_lm::RouteArgs a{};
  a.T = logits.size(0);
  a.E = logits.size(1);
  a.top = ids.size(1);
  a.groups = groups;
  a.keep = keep;
  SHAI_CHECK(ids.size(0) == a.T && wts.sizes() == ids.sizes(), "route outputs must be [T, top]");
  SHAI_CHECK(a.E <= 1024 && groups >= 1 && a.E % groups == 0 && keep >= 1 && keep <= groups && a.top >= 1 &&
                 a.top <= keep * (a.E / groups), "route: up to 1024 experts in equal groups, top within the kept ones");
  a.logits = logits.data_ptr<float>();
  a.ids = ids.data_ptr<int>();
  a.wts = wts.data_ptr<float>();
  if (a.T > 0) shai_lm::launch_route(a, stream());
}

// logits -> picks -> slots for up to 16 tokens in one launch (moe_route + moe_plan with 16-row tiles)
void moe_route_plan(const Tensor& logits, int64_t groups, int64_t keep, const Tensor& ids, const Tensor& wts,
                    const Tensor& offsets, const Tensor& token_of, const Tensor& slot_of, const Tensor& tiles) {
  check(logits, at::kFloat, "logits");
  check(wts, at::kFloat, "wts");
  for (auto* t : {&ids, &offsets, &token_of, &slot_of, &tiles}) check_i32(*t, "moe_route_plan tensor");
  shai_lm::RouteArgs r{};
  r.T = logits.size(0);
  r.E = logits.size(1);
  r.top = ids.size(1);
  r.groups = groups;
  r.keep = keep;
  SHAI_CHECK(r.T >= 1 && r.T <= 16 && r.E <= 256, "moe_route_plan: up to 16 tokens and 256 experts");
  SHAI_CHECK(ids.size(0) == r.T && wts.sizes() == ids.sizes(), "route outputs must be [T, top]");
  SHAI_CHECK(reinterpret_cast<uintptr_t>(ids.data_ptr()) % 16 == 0, "moe_route_plan: ids must be 16-byte aligned");
  SHAI_CHECK(groups >= 1 && r.E % groups == 0 && keep >= 1 && keep <= groups && r.top >= 1 &&
                 r.top <= keep * (r.E / groups), "route: experts in equal groups, top within the kept ones");
  r.logits = logits.data_ptr<float>();
  r.ids = ids.data_ptr<int>();
  r.wts = wts.data_ptr<float>();
  shai_lm::PlanArgs a{};
  a.P = ids.numel();
  a.top = r.top;
  a.E = r.E;
  a.bm = 16;
  a.n_tiles = tiles.size(0);
  SHAI_CHECK(offsets.numel() == a.E + 1 && token_of.numel() == a.P && slot_of.numel() == a.P && tiles.size(1) == 2 &&
                 a.n_tiles >= std::min<long>(a.P, a.E + a.P / 16), "moe_route_plan outputs");
  a.ids = r.ids;
  a.offsets = offsets.data_ptr<int>();
  a.token_of = token_of.data_ptr<int>();
  a.slot_of = slot_of.data_ptr<int>();
  a.tiles = tiles.data_ptr<int>();
  shai_lm::launch_route_plan(r, a, stream());
}

// `ids` comes from moe_route (every entry in 0 .. E - 1)
void moe_plan(const Tensor& ids, int64_t bm, const Tensor& offsets, const Tensor& token_of, const Tensor& slot_of,
              const Tensor& tiles) {
  for (auto* t : {&ids, &offsets, &token_of, &slot_of, &tiles}) check_i32(*t, "moe_plan tensor");
  shai_lm::PlanArgs a{};
  a.P = ids.numel();
  a.top = ids.size(1);
  a.E = offsets.numel() - 1;
  a.bm = bm;
  a.n_tiles = tiles.size(0);
  SHAI_CHECK(reinterpret_cast<uintptr_t>(ids.data_ptr()) % 16 == 0, "moe_plan: ids must be 16-byte aligned");
  SHAI_CHECK(a.E >= 1 && a.E <= 1024 && (bm == 16 || bm == 128 || bm == 256), "moe_plan: up to 1024 experts, bm 16 / 128 / 256");
  SHAI_CHECK(token_of.numel() == a.P && slot_of.numel() == a.P && tiles.size(1) == 2 &&
                 a.n_tiles >= std::min<long>(a.P, a.E + a.P / bm), "moe_plan outputs");
  a.ids = ids.data_ptr<int>();
  a.offsets = offsets.data_ptr<int>();
  a.token_of = token_of.data_ptr<int>();
  a.slot_of = slot_of.data_ptr<int>();
  a.tiles = tiles.data_ptr<int>();
  if (a.P > 0) shai_lm::launch_plan(a, stream());
}

shai_lm::AttnArgs attn_args(const Tensor& qkvg, const Tensor& kc, const Tensor& vc, const Tensor* o, int64_t heads) {
  const auto dt = qkvg.scalar_type();
  is_f32(qkvg);
  check(qkvg, dt, "qkvg");
  check(kc, dt, "k_cache");
  check(vc, dt, "v_cache");
  SHAI_CHECK(qkvg.dim() == 2 && kc.dim() == 4 && vc.dim() == 4 && kc.size(0) == vc.size(0) && kc.size(1) == vc.size(1) &&
                 kc.size(2) == 64 && vc.size(2) == 64, "caches must be [blocks, G, 64, dk | dv]");
  shai_lm::AttnArgs a{};
  a.T = qkvg.size(0);
  a.ld = qkvg.size(1);
  a.H = heads;
  a.G = kc.size(1);
  a.dk = kc.size(3);
  a.dv = vc.size(3);
  SHAI_CHECK(a.dk % 64 == 0 && a.dv % 64 == 0 && ((a.dk <= 128 && a.dv <= 128) || (a.dk == 256 && a.dv == 256)),
             "stored head sizes: 64 / 128 each, or 256 / 256");
  SHAI_CHECK(a.H >= 1 && a.G >= 1 && a.H % a.G == 0, "query heads must be a multiple of kv heads");
  SHAI_CHECK(a.ld % 8 == 0 && a.ld >= (long)a.H * a.dk + (long)a.G * (a.dk + a.dv) + a.H, "qkvg row too short");
  a.qkvg = qkvg.data_ptr();
  a.kc = kc.data_ptr();
  a.vc = vc.data_ptr();
  if (o) {
    check(*o, dt, "o");
    SHAI_CHECK(o->dim() == 2 && o->size(0) == a.T && o->size(1) == (long)a.H * a.dv, "o must be [T, H dv]");
    a.o = o->data_ptr();
  }
  return a;
}

void kv_store(const Tensor& qkvg, const Tensor& kc, const Tensor& vc, const Tensor& slots, int64_t heads) {
  shai_lm::AttnArgs a = attn_args(qkvg, kc, vc, nullptr, heads);
  check_i32(slots, "slots");
  SHAI_CHECK(slots.numel() >= a.T, "one slot per row");
  a.slots = slots.data_ptr<int>();
  if (a.T > 0) shai_lm::launch_kv_store(a, is_f32(qkvg), stream());
}

void chunk_attn_prefill(const Tensor& qkvg, const Tensor& kc, const Tensor& vc, const Tensor& o, const Tensor& bt,
                        const Tensor& ctx, const Tensor& q_lens, const Tensor& q_start, int64_t max_q, int64_t heads,
                        int64_t chunk, double scale) {
  shai_lm::AttnArgs a = attn_args(qkvg, kc, vc, &o, heads);
  for (auto* t : {&bt, &ctx, &q_lens, &q_start}) check_i32(*t, "batch tensor");
  a.B = bt.size(0);
  a.max_blocks = bt.size(1);
  SHAI_CHECK(ctx.numel() == a.B && q_lens.numel() == a.B && q_start.numel() == a.B && max_q >= 1 && chunk >= 1 &&
                 a.B <= 65535 && a.H <= 65535, "per-sequence [B] tensors, max_q and chunk >= 1");
  a.bt = bt.data_ptr<int>();
  a.ctx = ctx.data_ptr<int>();
  a.q_lens = q_lens.data_ptr<int>();
  a.q_start = q_start.data_ptr<int>();
  a.max_q = max_q;
  a.chunk = chunk;
  a.scale = scale;
  shai_lm::launch_attn_prefill(a, is_f32(qkvg), stream());
}

void chunk_attn_decode(const Tensor& qkvg, const Tensor& kc, const Tensor& vc, const Tensor& o, const Tensor& bt,
                       const Tensor& ctx, const Tensor& slots, const Tensor& ws, int64_t heads, int64_t splits,
                       int64_t chunk, double scale) {
  shai_lm::AttnArgs a = attn_args(qkvg, kc, vc, &o, heads);
  for (auto* t : {&bt, &ctx, &slots}) check_i32(*t, "batch tensor");
  a.B = bt.size(0);
  a.max_blocks = bt.size(1);
  SHAI_CHECK(a.B == a.T && ctx.numel() >= a.B && slots.numel() >= a.B && chunk >= 1 && a.B <= 65535,
             "decode: one row per sequence");
  SHAI_CHECK(splits >= 1 && splits <= 64 &&
                 (splits == 1 || (ws.scalar_type() == at::kFloat && ws.is_contiguous() &&
                                  ws.numel() >= (long)a.B * a.H * splits * (a.dv + 2))), "decode split workspace");
  a.bt = bt.data_ptr<int>();
  a.ctx = ctx.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.ws = splits > 1 ? ws.data_ptr<float>() : nullptr;
  a.splits = splits;
  a.max_q = 1;
  a.chunk = chunk;
  a.scale = scale;
  shai_lm::launch_attn_decode(a, is_f32(qkvg), stream());
}

void sample(const Tensor& logits, const Tensor& temps, const Tensor& top_k, const Tensor& top_p,
            const Tensor& uniforms, const Tensor& out) {
  SHAI_CHECK(logits.is_cuda() && logits.dim() == 2 && logits.stride(1) == 1, "logits must be a 2D GPU tensor");
  const bool bf16 = logits.scalar_type() == at::kBFloat16;
  SHAI_CHECK(bf16 || logits.scalar_type() == at::kFloat, "logits must be bf16 or fp32");
  const int B = logits.size(0);
  check_f32(temps, "temps");
  check_f32(top_p, "top_p");
  check_f32(uniforms, "uniforms");
  check_i32(top_k, "top_k");
  check_i32(out, "out");
  SHAI_CHECK(temps.numel() == B && top_p.numel() == B && uniforms.numel() == B && top_k.numel() == B &&
                 out.numel() == B,
             "per-row parameter sizes");
  shai::launch_sample(logits.data_ptr(), bf16, logits.stride(0), B, logits.size(1), temps.data_ptr<float>(),
                      top_k.data_ptr<int>(), top_p.data_ptr<float>(), uniforms.data_ptr<float>(),
                      out.data_ptr<int>(), stream());
}

void token_feedback(const Tensor& ids, const Tensor& rowmap, const Tensor& prev) {
  SHAI_CHECK(ids.scalar_type() == at::kInt && rowmap.scalar_type() == at::kInt && prev.scalar_type() == at::kInt &&
                 ids.is_contiguous() && rowmap.is_contiguous() && prev.is_contiguous() && rowmap.numel() == ids.numel(),
             "token_feedback: int32 contiguous ids / rowmap of one length");
  shai::launch_token_feedback(ids.data_ptr<int>(), rowmap.data_ptr<int>(), prev.data_ptr<int>(), (int)ids.numel(),
                              stream());
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(shai, m) {
  m.def("embed_norm(Tensor ids, Tensor? prev, Tensor table, Tensor? bigram, int mul_prev, int mul_cur, Tensor w, float eps, int width, Tensor(a!) x, Tensor(b!) h) -> ()");
  m.def("add_norm(Tensor(a!) x, Tensor? dense, Tensor? ye, Tensor? slot_of, Tensor? wts, Tensor? inject, Tensor? rows, Tensor? w, float eps, int width, Tensor(b!)? h) -> ()");
  m.def("lm_gemm(Tensor a, Tensor w, Tensor(a!) c, Tensor? tiles, Tensor? offsets, Tensor? gather, int bm, int epi, float param, Tensor(b!)? side=None) -> ()");
  m.def("moe_route(Tensor logits, int groups, int keep, Tensor(a!) ids, Tensor(b!) wts) -> ()");
  m.def("moe_route_plan(Tensor logits, int groups, int keep, Tensor(a!) ids, Tensor(b!) wts, Tensor(c!) offsets, Tensor(d!) token_of, Tensor(e!) slot_of, Tensor(f!) tiles) -> ()");
  m.def("moe_plan(Tensor ids, int bm, Tensor(a!) offsets, Tensor(b!) token_of, Tensor(c!) slot_of, Tensor(d!) tiles) -> ()");
  m.def("kv_store(Tensor qkvg, Tensor(a!) k_cache, Tensor(b!) v_cache, Tensor slots, int heads) -> ()");
  m.def("chunk_attn_prefill(Tensor qkvg, Tensor k_cache, Tensor v_cache, Tensor(a!) o, Tensor block_table, Tensor ctx_lens, Tensor q_lens, Tensor q_start, int max_q, int heads, int chunk, float scale) -> ()");
  m.def("chunk_attn_decode(Tensor qkvg, Tensor(a!) k_cache, Tensor(b!) v_cache, Tensor(c!) o, Tensor block_table, Tensor ctx_lens, Tensor slots, Tensor(d!) ws, int heads, int splits, int chunk, float scale) -> ()");
  m.def("sample(Tensor logits, Tensor temps, Tensor top_k, Tensor top_p, Tensor uniforms, Tensor(a!) out) -> ()");
  m.def("token_feedback(Tensor(a!) ids, Tensor rowmap, Tensor prev) -> ()");
}

TORCH_LIBRARY_IMPL(shai, CUDA, m) {
  m.impl("embed_norm", &embed_norm);
  m.impl("add_norm", &add_norm);
  m.impl("lm_gemm", &lm_gemm);
  m.impl("moe_route", &moe_route);
  m.impl("moe_route_plan", &moe_route_plan);
  m.impl("moe_plan", &moe_plan);
  m.impl("kv_store", &kv_store);
  m.impl("chunk_attn_prefill", &chunk_attn_prefill);
  m.impl("chunk_attn_decode", &chunk_attn_decode);
  m.impl("sample", &sample);
  m.impl("token_feedback", &token_feedback);
}
