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
// a matrix of contiguous rows that may lie apart
void check_rows(const Tensor& t, at::ScalarType dt, const char* name) {
  SHAI_CHECK(t.is_cuda() && t.dim() == 2 && t.scalar_type() == dt && (t.size(1) <= 1 || t.stride(1) == 1) &&
                 (t.size(0) <= 1 || t.stride(0) >= t.size(1)), name, " must be a GPU ", dt, " matrix of contiguous rows");
}
// the same, read or written 16 bytes at a time
void check_rows16(const Tensor& t, at::ScalarType dt, const char* name) {
  check_rows(t, dt, name);
  SHAI_CHECK(t.stride(0) * t.element_size() % 16 == 0 && reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0, name,
             " rows must be 16-byte aligned");
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
             const optional<Tensor>& side, const optional<Tensor>& vec, const optional<Tensor>& rope, int64_t head,
             int64_t rot0, const optional<Tensor>& ids, const optional<Tensor>& table, int64_t act) {
  const bool f32 = is_f32(A);
  SHAI_CHECK(A.is_cuda() && A.dim() == 2 && A.stride(1) == 1 && A.stride(0) % 8 == 0 && A.stride(0) >= A.size(1) &&
                 reinterpret_cast<uintptr_t>(A.data_ptr()) % 16 == 0, "A rows must be contiguous and 16-byte aligned");
  check(W, A.scalar_type(), "W");
  SHAI_CHECK(C.scalar_type() == at::kFloat || (!f32 && C.scalar_type() == at::kBFloat16), "C: fp32, or bf16 as A");
  check_rows(C, C.scalar_type(), "C");
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
  SHAI_CHECK(epi >= 0 && epi <= 7, "lm_gemm epilogue");
  const bool glu = shai_lm::glu_epi(epi);
  g.n_main = g.N;
  g.lda = A.stride(0);
  g.batch = 1;
  if (side) {  // the last rows of W are a plain product, stored in fp32
    check(*side, at::kFloat, "side");
    SHAI_CHECK(!tiles && (glu || epi == shai_lm::EPI_NONE || epi == shai_lm::EPI_RELU2) && side->dim() == 2 &&
                   side->size(0) == g.M && side->size(1) >= 1 && side->size(1) < g.N,
               "side output: dense plain, squared ReLU or GLU products, [M, last rows of W]");
    g.n_main = g.N - side->size(1);
    SHAI_CHECK(g.n_main % 4 == 0, "side output: the other rows of W must be a multiple of 4");
    g.side = side->data_ptr<float>();
  }
  SHAI_CHECK(!glu || g.n_main % 2 == 0, "GLU products need (gate, up) row pairs");
  SHAI_CHECK(reinterpret_cast<uintptr_t>(C.data_ptr()) % 16 == 0, "C must be 16-byte aligned");
  SHAI_CHECK(C.size(1) == (glu ? g.n_main / 2 : g.n_main), "lm_gemm output columns");
  g.ldc = g.M > 1 ? C.stride(0) : std::max<int64_t>(C.stride(0), C.size(1));
  g.n_act = act > 0 ? act : g.n_main;
  SHAI_CHECK(act == 0 || (epi == shai_lm::EPI_RELU2 && act % 4 == 0 && act <= g.n_main), "act: leading columns, a multiple of 4");
  if (epi == shai_lm::EPI_XIELU) {
    SHAI_CHECK(vec.has_value() && vec->numel() == 2, "the xIELU epilogue needs its two coefficients");
    check_f32(*vec, "vec");
    g.vec = vec->data_ptr<float>();
  }
  if (epi == shai_lm::EPI_ROTARY) {
    SHAI_CHECK(rope.has_value() && rope->dim() == 2 && rope->size(0) == g.M && !tiles, "rotary epilogue: rope [M, dims]");
    check_f32(*rope, "rope");
    g.rope = rope->data_ptr<float>();
    g.rot = rope->size(1);
    g.head = head;
    g.rot0 = rot0;
    SHAI_CHECK(g.rot % 2 == 0 && rot0 % 4 == 0 && rot0 >= 0 && head % 4 == 0 && rot0 + g.rot <= head && g.N % head == 0,
               "rotary epilogue: heads of ", head, " columns, the rotated ones from a multiple of 4");
  }
  if (epi == shai_lm::EPI_GELU_ROWS) {
    SHAI_CHECK(ids.has_value() && table.has_value() && !tiles && ids->numel() >= g.M && table->is_cuda() &&
                   table->scalar_type() == A.scalar_type() && table->dim() == 2 && table->size(0) >= 1 && table->size(1) == g.N &&
                   table->stride(1) == 1 && table->stride(0) % 4 == 0 && g.N % 4 == 0 &&
                   reinterpret_cast<uintptr_t>(table->data_ptr()) % 16 == 0,
               "table rows: ids [M] and a table [rows, N] of the type of A, rows 4-element aligned");
    check_i32(*ids, "ids");
    g.ids = ids->data_ptr<int>();
    g.table = table->data_ptr();
    g.table_ld = table->stride(0);
    g.table_rows = table->size(0);
    g.table_f32 = f32;
  }
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
  const long lim = 0x7fffffffL, esize = f32 ? 4 : 2, osize = g.out_f32 ? 4 : 2;
  const bool tile = !f32 && (g.tiles ? bm >= 128 && (long)g.a_rows * g.lda * 2 < lim : g.M > 64) && (long)g.N * g.K * 2 < lim;
  if (!tile) return shai_lm::launch_gemm(g, f32, stream());
  // the tiled kernel addresses A with 32-bit offsets: a longer A runs in equal parts
  const int total = g.M;
  const long most = std::max<long>(256, (lim / (g.lda * 2)) / 256 * 256), parts = (total + most - 1) / most;
  const int rows = g.tiles ? total : (int)std::min<long>(total, ((total + parts - 1) / parts + 255) / 256 * 256);
  SHAI_CHECK(g.tiles || (long)rows * g.lda * 2 < lim, "lm_gemm: rows of A are too long");
  for (int at = 0; at < total; at += rows) {
    shai_lm::GemmArgs part = g;
    if (!g.tiles) {
      part.M = part.a_rows = std::min(rows, total - at);
      part.A = static_cast<const char*>(g.A) + at * g.lda * esize;
      part.C = static_cast<char*>(g.C) + at * g.ldc * osize;
      if (g.side) part.side = g.side + (long)at * (g.N - g.n_main);
      if (g.rope) part.rope = g.rope + (long)at * g.rot;
      if (g.ids) part.ids = g.ids + at;
    }
    shai_lm::launch_gemm_tile(part, stream());
  }
}

// c[t, h] = a[t, h] w[h]^T for every head h: a [T, H, K], w [H, N, K], c [T, H, N], any strides between rows and heads
void lm_gemm_heads(const Tensor& A, const Tensor& W, const Tensor& C) {
  const bool f32 = is_f32(A);
  SHAI_CHECK(A.dim() == 3 && W.dim() == 3 && C.dim() == 3 && W.scalar_type() == A.scalar_type() &&
                 C.scalar_type() == A.scalar_type(), "lm_gemm_heads: three [.., .., ..] tensors of one type");
  for (auto* t : {&A, &W, &C})
    SHAI_CHECK(t->is_cuda() && t->stride(2) == 1 && t->stride(0) % 8 == 0 && t->stride(1) % 8 == 0 && t->stride(0) >= 0 &&
                   t->stride(1) >= 0 && reinterpret_cast<uintptr_t>(t->data_ptr()) % 16 == 0,
               "lm_gemm_heads: rows must be contiguous and 16-byte aligned");
  shai_lm::GemmArgs g{};
  g.M = g.a_rows = A.size(0);
  g.batch = A.size(1);
  g.K = A.size(2);
  g.N = g.n_main = g.n_act = W.size(1);
  SHAI_CHECK(W.size(0) == g.batch && W.size(2) == g.K && W.stride(1) == g.K && g.K % 64 == 0 && g.N % 4 == 0 &&
                 C.size(0) == g.M && C.size(1) == g.batch && C.size(2) == g.N && g.batch <= 65535, "lm_gemm_heads shapes");
  g.A = A.data_ptr();
  g.W = W.data_ptr();
  g.C = C.data_ptr();
  g.lda = A.stride(0);
  g.a_batch = A.stride(1);
  g.w_batch = W.stride(0);
  g.ldc = C.stride(0);
  g.c_batch = C.stride(1);
  g.out_f32 = f32;
  if (g.M > 0) shai_lm::launch_gemm(g, f32, stream());
}

// partial sums of a w^T over equal parts of K: c [splits, M, N] fp32
void lm_gemm_parts(const Tensor& A, const Tensor& W, const Tensor& C) {
  const bool f32 = is_f32(A);
  check_rows16(A, A.scalar_type(), "A");
  check(W, A.scalar_type(), "W");
  check(C, at::kFloat, "C");
  shai_lm::GemmArgs g{};
  SHAI_CHECK(A.dim() == 2 && W.dim() == 2 && C.dim() == 3, "lm_gemm_parts ranks");
  g.M = g.a_rows = A.size(0);
  g.N = g.n_main = g.n_act = g.ldc = W.size(0);
  g.K = A.size(1);
  g.lda = A.stride(0);
  g.splits = C.size(0);
  g.batch = 1;
  g.out_f32 = true;
  SHAI_CHECK(W.size(1) == g.K && g.K % 64 == 0 && C.size(1) == g.M && C.size(2) == g.N && g.splits >= 1 &&
                 g.splits <= g.K / 64, "lm_gemm_parts shapes");
  g.A = A.data_ptr();
  g.W = W.data_ptr();
  g.C = C.data_ptr();
  if (g.M == 0) return;
  const long lim = 0x7fffffffL;
  const bool tile = !f32 && g.M > 64 && (long)g.M * g.lda * 2 < lim && (long)g.N * g.K * 2 < lim;
  if (tile) shai_lm::launch_gemm_tile(g, stream());
  else shai_lm::launch_gemm(g, f32, stream());
}

void residual_norm(const optional<Tensor>& x, const optional<Tensor>& ids, const optional<Tensor>& table, double scale,
                   const optional<Tensor>& delta, const optional<Tensor>& wb, double mult, const optional<Tensor>& step,
                   const optional<Tensor>& x_out, const optional<Tensor>& rows, const optional<Tensor>& w, double eps,
                   int64_t width, const optional<Tensor>& h, const optional<Tensor>& cw, const optional<Tensor>& state,
                   const optional<Tensor>& tail, const optional<Tensor>& row_seq, const optional<Tensor>& q_start,
                   const optional<Tensor>& q_lens, const optional<Tensor>& pos, const optional<Tensor>& slots,
                   const optional<Tensor>& bb, const optional<Tensor>& b, const optional<Tensor>& ye,
                   const optional<Tensor>& slot_of, const optional<Tensor>& wts) {
  shai_lm::ResidualNormArgs a{};
  a.width = width;
  a.eps = eps;
  long R;
  at::ScalarType dt = at::kFloat;               // of every tensor but the residual and partial sums
  for (auto* t : {&delta, &table, &ye, &h})
    if (*t) dt = (*t)->scalar_type();
  SHAI_CHECK(dt == at::kFloat || dt == at::kBFloat16, "bf16 or fp32");
  SHAI_CHECK(x.has_value() != ids.has_value(), "residual_norm: a residual or token ids");
  if (x) {
    check(*x, at::kFloat, "x");
    R = x->size(0);
    a.Dp = x->size(1);
    a.x = x->data_ptr<float>();
  } else {
    check_i32(*ids, "ids");
    SHAI_CHECK(table.has_value(), "token ids need a table");
    check(*table, dt, "table");
    R = ids->numel();
    a.V = table->size(0);
    a.Dp = table->size(1);
    a.ids = ids->data_ptr<int>();
    a.table = table->data_ptr();
    a.scale = scale;
  }
  a.T = R;
  check_width(a.Dp, width);
  auto row_vec = [&](const optional<Tensor>& t, const char* name) -> const float* {
    if (!t) return nullptr;
    check(*t, at::kFloat, name);
    SHAI_CHECK(t->numel() == a.Dp, name, " must be [D]");
    return t->data_ptr<float>();
  };
  if (delta) {
    const bool many = delta->dim() == 3;
    check(*delta, many ? at::kFloat : dt, "delta");
    SHAI_CHECK((many || delta->dim() == 2) && delta->size(-2) == R && delta->size(-1) == a.Dp && (wb.has_value() || !bb),
               "delta must be [rows, D] or [parts, rows, D]; a norm's bias comes with its gain");
    a.delta = delta->data_ptr();
    a.parts = many ? delta->size(0) : 0;
    a.part_stride = R * a.Dp;
  }
  if (ye) {  // the weighted outputs of a token's experts
    check(*ye, dt, "ye");
    SHAI_CHECK(!delta && wb.has_value() && slot_of.has_value() && wts.has_value(),
               "expert outputs: the only delta, with slot_of, weights and gain");
    check_i32(*slot_of, "slot_of");
    check(*wts, at::kFloat, "wts");
    a.top = slot_of->size(1);
    SHAI_CHECK(slot_of->size(0) == R && wts->sizes() == slot_of->sizes() && ye->size(0) == R * a.top && ye->size(1) == a.Dp,
               "expert outputs must be [rows * top, D]");
    a.ye = ye->data_ptr();
    a.slot_of = slot_of->data_ptr<int>();
    a.wts = wts->data_ptr<float>();
  }
  a.wb = row_vec(wb, "wb");
  a.bb = row_vec(bb, "bb");
  a.mult = mult;
  a.step = row_vec(step, "step");
  a.w = row_vec(w, "w");
  a.b = row_vec(b, "b");
  SHAI_CHECK(!b || w.has_value(), "a norm's bias comes with its gain");
  if (x_out) {
    check(*x_out, at::kFloat, "x_out");
    SHAI_CHECK(x_out->size(0) == R && x_out->size(1) == a.Dp, "x_out must be [rows, D]");
    a.x_out = x_out->data_ptr<float>();
  }
  if (rows) {
    check_i32(*rows, "rows");
    SHAI_CHECK(!cw && h.has_value(), "rows selects rows of h");
    a.rows = rows->data_ptr<int>();
    a.T = rows->numel();
  }
  SHAI_CHECK(!w || h.has_value(), "a norm needs an output h");
  if (h) {
    check(*h, dt, "h");
    SHAI_CHECK(h->numel() == (long)a.T * a.Dp, "h must be [rows, D]");
    a.h = h->data_ptr();
  }
  if (cw) {
    check(*cw, at::kFloat, "cw");
    SHAI_CHECK(!(delta || ye) || wb, "convolution: a delta has a norm");
    SHAI_CHECK(cw->dim() == 2 && cw->size(1) == a.Dp && cw->size(0) >= 1 && cw->size(0) <= 16, "convolution: 1 to 16 taps");
    a.taps = cw->size(0);
    SHAI_CHECK(h.has_value() && x_out.has_value() && (!x || x->data_ptr() != x_out->data_ptr()),
               "convolution: needs an output h, and x_out apart from x");
    SHAI_CHECK(state.has_value() && pos.has_value() && slots.has_value() && pos->numel() >= R, "convolution: state, pos, slots");
    check(*state, at::kFloat, "state");
    check_i32(*pos, "pos");
    check_i32(*slots, "slots");
    SHAI_CHECK(state->dim() == 3 && state->size(1) == a.taps - 1 && state->size(2) == a.Dp, "state must be [slots, taps - 1, D]");
    a.cw = cw->data_ptr<float>();
    a.state = state->data_ptr<float>();
    a.pos = pos->data_ptr<int>();
    a.slots = slots->data_ptr<int>();
    a.B = R;
    a.run = 1;
    if (tail) {
      SHAI_CHECK(row_seq.has_value() && q_start.has_value() && q_lens.has_value(), "prefill convolution: row_seq, q_start, q_lens");
      check(*tail, at::kFloat, "tail");
      check_i32(*row_seq, "row_seq");
      check_i32(*q_start, "q_start");
      check_i32(*q_lens, "q_lens");
      a.B = q_lens->numel();
      SHAI_CHECK(tail->dim() == 3 && tail->size(0) == a.B && tail->size(1) == a.taps - 1 && tail->size(2) == a.Dp &&
                     row_seq->numel() == R && q_start->numel() == a.B, "tail must be [B, taps - 1, D]");
      a.tail = tail->data_ptr<float>();
      a.row_seq = row_seq->data_ptr<int>();
      a.q_start = q_start->data_ptr<int>();
      a.q_lens = q_lens->data_ptr<int>();
      a.run = R >= 32768 ? 32 : R >= 8192 ? 16 : R >= 4096 ? 8 : R >= 2048 ? 4 : 2;
    }
    SHAI_CHECK(slots->numel() >= a.B, "one state slot per sequence");
  }
  if (a.T > 0) shai_lm::launch_residual_norm(a, dt == at::kFloat, stream());
}

void conv_commit(const Tensor& state, const Tensor& tail, const Tensor& q_lens, const Tensor& slots) {
  check(state, at::kFloat, "state");
  check(tail, at::kFloat, "tail");
  check_i32(q_lens, "q_lens");
  check_i32(slots, "slots");
  SHAI_CHECK(state.dim() == 4 && tail.dim() == 4 && state.size(0) == tail.size(0) && state.size(2) == tail.size(2) &&
                 state.size(3) == tail.size(3) && state.size(3) % 4 == 0, "state [runs, slots, taps - 1, D], tail [runs, B, taps - 1, D]");
  shai_lm::ConvCommitArgs a{};
  a.runs = state.size(0);
  a.n_slots = state.size(1);
  a.B = tail.size(1);
  a.taps = state.size(2) + 1;
  a.Dp = state.size(3);
  SHAI_CHECK(q_lens.numel() == a.B && slots.numel() == a.B && a.B <= 65535 && a.runs <= 65535, "one length and slot per sequence");
  a.state = state.data_ptr<float>();
  a.tail = tail.data_ptr<float>();
  a.q_lens = q_lens.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  if (tail.numel() > 0) shai_lm::launch_conv_commit(a, stream());
}

void rope_rows(const Tensor& pos, const Tensor& freq, const Tensor& out) {
  check_i32(pos, "pos");
  check_f32(freq, "freq");
  check_f32(out, "out");
  SHAI_CHECK(freq.dim() == 2 && freq.size(1) == 2 && out.dim() == 2 && out.size(0) <= pos.numel() &&
                 out.size(1) == 2 * freq.size(0), "rope_rows: freq [n, 2], out [T, 2 n]");
  shai_lm::RopeRowsArgs a{pos.data_ptr<int>(), freq.data_ptr<float>(), (int)out.size(0), (int)freq.size(0),
                          out.data_ptr<float>()};
  if (out.numel() > 0) shai_lm::launch_rope_rows(a, stream());
}

void latent_prep(const Tensor& d, const Tensor& wq, const Tensor& wkv, const Tensor& rope, const Tensor& slots,
                 const Tensor& cache, const Tensor& cq, double eps, int64_t q_rank, int64_t kv_rank) {
  const auto dt = cq.scalar_type();
  const bool f32 = is_f32(cq);
  check(d, at::kFloat, "d");
  check(wq, at::kFloat, "wq");
  check(wkv, at::kFloat, "wkv");
  check(rope, at::kFloat, "rope");
  check_i32(slots, "slots");
  check(cache, dt, "cache");
  check(cq, dt, "cq");
  shai_lm::LatentPrepArgs a{};
  SHAI_CHECK((d.dim() == 2 || d.dim() == 3) && cq.dim() == 2 && cache.dim() == 3 && cache.size(1) == 64 && rope.dim() == 2, "latent_prep ranks");
  a.T = d.size(-2);
  a.parts = d.dim() == 3 ? d.size(0) : 1;
  a.qp = cq.size(1);
  a.rp = wkv.numel();
  a.op = cache.size(2) - a.rp;
  a.rot = rope.size(1);
  a.q_rank = q_rank;
  a.kv_rank = kv_rank;
  a.eps = eps;
  SHAI_CHECK(a.qp % 64 == 0 && a.rp % 64 == 0 && a.op % 2 == 0 && a.op >= a.rot && a.rot % 2 == 0 && wq.numel() == a.qp &&
                 d.size(-1) == a.qp + a.rp + a.op && (a.parts == 1 || (a.qp + a.rp + a.op) * 4 <= 65536 - 64) && cq.size(0) == a.T && rope.size(0) == a.T && slots.numel() >= a.T &&
                 q_rank >= 1 && q_rank <= a.qp && kv_rank >= 1 && kv_rank <= a.rp, "latent_prep shapes");
  a.d = d.data_ptr<float>();
  a.wq = wq.data_ptr<float>();
  a.wkv = wkv.data_ptr<float>();
  a.rope = rope.data_ptr<float>();
  a.slots = slots.data_ptr<int>();
  a.cache = cache.data_ptr();
  a.cq = cq.data_ptr();
  if (a.T > 0) shai_lm::launch_latent_prep(a, f32, stream());
}

// start: first output row of every listed sequence; the caller sized `out` for all of them
void latent_gather(const Tensor& cache, const Tensor& bt, const Tensor& seqs, const Tensor& ctx, const Tensor& start,
                   int64_t max_ctx, const Tensor& out) {
  check(cache, out.scalar_type(), "cache");
  check(out, out.scalar_type(), "out");
  for (auto* t : {&bt, &seqs, &ctx, &start}) check_i32(*t, "latent_gather tensor");
  shai_lm::LatentGatherArgs a{};
  a.n = seqs.numel();
  a.max_ctx = max_ctx;
  a.max_blocks = bt.size(1);
  a.ld_bytes = cache.size(2) * cache.element_size();
  SHAI_CHECK(cache.dim() == 3 && cache.size(1) == 64 && out.dim() == 2 && out.size(1) == cache.size(2) && a.ld_bytes % 16 == 0 &&
                 ctx.numel() == a.n && start.numel() == a.n && a.n <= 65535 && max_ctx <= (int64_t)a.max_blocks * 64,
             "latent_gather shapes");
  a.cache = cache.data_ptr();
  a.out = out.data_ptr();
  a.bt = bt.data_ptr<int>();
  a.seqs = seqs.data_ptr<int>();
  a.ctx = ctx.data_ptr<int>();
  a.start = start.data_ptr<int>();
  if (a.n > 0 && max_ctx > 0) shai_lm::launch_latent_gather(a, stream());
}

void latent_attn_prefill(const Tensor& q, const Tensor& kv, const Tensor& lat, const Tensor& o, const Tensor& ctx,
                         const Tensor& q_lens, const Tensor& q_start, const Tensor& kv_start, const Tensor& sink,
                         int64_t max_q, int64_t heads, int64_t np, int64_t rot, int64_t rank, double scale) {
  for (auto* t : {&q, &kv, &lat, &o}) check(*t, at::kBFloat16, "latent prefill tensor");
  for (auto* t : {&ctx, &q_lens, &q_start, &kv_start}) check_i32(*t, "batch tensor");
  check_f32(sink, "sink");
  shai_lm::AttnArgs a{};
  a.B = ctx.numel();
  a.H = a.G = heads;
  SHAI_CHECK(heads >= 1 && q.dim() == 2 && o.dim() == 2 && kv.dim() == 2 && lat.dim() == 2 && q.size(1) % heads == 0 &&
                 o.size(1) % heads == 0 && q.size(0) == o.size(0), "latent prefill: q [T, H dk], o [T, H dv]");
  a.T = q.size(0);
  a.ld = q.size(1);
  a.ldo = o.size(1);
  a.dk = q.size(1) / heads;
  a.dv = o.size(1) / heads;
  SHAI_CHECK((a.dk == 64 && a.dv == 64) || (a.dk == 128 && (a.dv == 64 || a.dv == 128)) || (a.dk == 192 && a.dv == 128) ||
                 (a.dk == 256 && a.dv == 256), "latent prefill head sizes: 64/64, 128/64, 128/128, 192/128 or 256/256");
  a.np = np;
  const int rp8 = (rot + 7) / 8 * 8;
  a.rank = rank;
  a.lat_ld = lat.size(1);
  a.lat_pad = a.lat_ld - a.rank - 8;   // the queries are zero past the rotated part: any finite value will do there
  SHAI_CHECK(np >= 0 && np % 8 == 0 && np + rp8 <= a.dk && rank % 8 == 0 && rank + rp8 <= a.lat_ld && a.lat_ld % 8 == 0 &&
                 kv.size(1) == heads * (np + a.dv) && kv.size(0) == lat.size(0), "latent prefill: kv [rows, H (np + dv)]");
  SHAI_CHECK(q_lens.numel() == a.B && q_start.numel() == a.B && kv_start.numel() == a.B && sink.numel() == heads && max_q >= 1 &&
                 a.B <= 65535 && a.H <= 65535, "per-sequence [B] tensors");
  a.qkvg = q.data_ptr();
  a.kv = kv.data_ptr();
  a.lat = lat.data_ptr();
  a.o = o.data_ptr();
  a.ctx = ctx.data_ptr<int>();
  a.q_lens = q_lens.data_ptr<int>();
  a.q_start = q_start.data_ptr<int>();
  a.kv_start = kv_start.data_ptr<int>();
  a.sink = sink.data_ptr<float>();
  a.max_q = max_q;
  a.chunk = 1;
  a.scale = scale;
  if (a.T > 0 && a.B > 0) shai_lm::launch_latent_prefill(a, stream());
}

void latent_attn_rows(const Tensor& ql, const Tensor& q, const Tensor& cache, const Tensor& o, const Tensor& bt,
                      const optional<Tensor>& seqs, const Tensor& ctx, const Tensor& sink, const Tensor& ws, int64_t splits,
                      int64_t np, int64_t rot, double scale) {
  const auto dt = q.scalar_type();
  const bool f32 = is_f32(q);
  check(ql, dt, "ql");
  check(q, dt, "q");
  check(cache, dt, "cache");
  check(o, dt, "o");
  check_i32(bt, "block table");
  check_i32(ctx, "ctx");
  check_f32(sink, "sink");
  shai_lm::LatentArgs a{};
  SHAI_CHECK(ql.dim() == 3 && q.dim() == 2 && cache.dim() == 3 && cache.size(1) == 64 && bt.dim() == 2, "latent_attn_rows ranks");
  a.n = ql.size(0);
  a.H = ql.size(1);
  a.rp = ql.size(2);
  a.op = cache.size(2) - a.rp;
  a.ldq = q.size(1);
  a.head = q.size(1) / a.H;
  a.np = np;
  a.rot = rot;
  a.max_blocks = bt.size(1);
  a.splits = splits;
  a.scale = scale;
  SHAI_CHECK(q.size(0) == a.n && q.size(1) % a.H == 0 && a.rp % 64 == 0 && a.rp <= 1024 && a.op >= (rot + 7) / 8 * 8 &&
                 a.op % 4 == 0 && np % 8 == 0 && np + (rot + 7) / 8 * 8 <= a.head && o.sizes() == ql.sizes() &&
                 ctx.numel() >= a.n && sink.numel() == a.H && a.n <= 65535, "latent_attn_rows shapes");
  if (seqs) {
    check_i32(*seqs, "seqs");
    SHAI_CHECK(seqs->numel() == a.n, "seqs: one per row");
    a.seqs = seqs->data_ptr<int>();
  } else {
    SHAI_CHECK(bt.size(0) >= a.n, "one block table row per entry");
  }
  a.ql = ql.data_ptr();
  a.q = q.data_ptr();
  a.cache = cache.data_ptr();
  a.o = o.data_ptr();
  a.bt = bt.data_ptr<int>();
  a.ctx = ctx.data_ptr<int>();
  a.sink = sink.data_ptr<float>();
  if (a.n == 0) return;
  if (f32 || !shai_lm::latent_decode_fits(a.rp, a.op)) {
    SHAI_CHECK((a.rp + a.op + 64) * 16 <= 65536, "latent rows of up to 4032 values");
    shai_lm::launch_latent_rows(a, f32, stream());
    return;
  }
  SHAI_CHECK(splits >= 1 && splits <= 64 &&
                 (splits == 1 || (ws.scalar_type() == at::kFloat && ws.is_contiguous() &&
                                  ws.numel() >= (long)a.n * a.H * splits * (a.rp + 4))), "split workspace");
  a.ws = splits > 1 ? ws.data_ptr<float>() : nullptr;
  shai_lm::launch_latent_decode(a, stream());
}

void mingru_scan(const Tensor& zx, const Tensor& g, const Tensor& bias, const Tensor& state, const Tensor& out,
                 const Tensor& pos, const optional<Tensor>& q_start, const optional<Tensor>& q_lens, const Tensor& slots,
                 const Tensor& ws, int64_t max_q, int64_t len) {
  const bool f32 = is_f32(g);
  check(zx, at::kFloat, "zx");
  check(g, g.scalar_type(), "g");
  check(bias, at::kFloat, "bias");
  check(state, at::kFloat, "state");
  check(out, g.scalar_type(), "out");
  check_i32(pos, "pos");
  check_i32(slots, "slots");
  shai_lm::ScanArgs a{};
  SHAI_CHECK(g.dim() == 2 && zx.dim() == 2 && state.dim() == 2 && len >= 1 && max_q >= 1, "mingru_scan ranks");
  a.T = g.size(0);
  a.W = g.size(1);
  SHAI_CHECK(zx.size(0) == a.T && zx.size(1) == 2 * a.W && bias.numel() == 2 * a.W && state.size(1) == a.W &&
                 out.sizes() == g.sizes() && pos.numel() >= a.T, "mingru_scan shapes");
  a.B = a.T;
  a.len = len;
  a.max_q = max_q;
  a.chunks = (max_q + len - 1) / len;
  if (q_lens) {
    SHAI_CHECK(q_start.has_value(), "prefill scan: q_start");
    check_i32(*q_lens, "q_lens");
    check_i32(*q_start, "q_start");
    a.B = q_lens->numel();
    SHAI_CHECK(q_start->numel() == a.B, "one start per sequence");
    a.q_lens = q_lens->data_ptr<int>();
    a.q_start = q_start->data_ptr<int>();
  } else {
    SHAI_CHECK(a.chunks == 1, "decode scan: one row per sequence");
  }
  SHAI_CHECK(slots.numel() >= a.B && a.B <= 65535 && a.chunks <= 65535, "one state slot per sequence");
  SHAI_CHECK(a.chunks == 1 || (ws.scalar_type() == at::kFloat && ws.is_contiguous() &&
                               ws.numel() >= (long)a.B * a.chunks * 2 * a.W), "scan workspace");
  a.zx = zx.data_ptr<float>();
  a.g = g.data_ptr();
  a.bias = bias.data_ptr<float>();
  a.state = state.data_ptr<float>();
  a.out = out.data_ptr();
  a.pos = pos.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.ws = a.chunks > 1 ? ws.data_ptr<float>() : nullptr;
  if (a.T > 0) shai_lm::launch_mingru_scan(a, f32, stream());
}

void hgrn2(const Tensor& qv, const Tensor& z, const Tensor& bias, const Tensor& lower, const Tensor& gain,
           const Tensor& state, const Tensor& out, const Tensor& pos, const optional<Tensor>& q_start,
           const optional<Tensor>& q_lens, const Tensor& slots, const Tensor& ws, int64_t max_q, int64_t len, int64_t vdim,
           double eps) {
  const bool f32 = is_f32(qv);
  check(qv, qv.scalar_type(), "qv");
  check(out, qv.scalar_type(), "out");
  for (auto* t : {&z, &bias, &lower, &gain, &state}) check(*t, at::kFloat, "hgrn2 fp32 tensor");
  check_i32(pos, "pos");
  check_i32(slots, "slots");
  shai_lm::Hgrn2Args a{};
  SHAI_CHECK(qv.dim() == 2 && z.dim() == 2 && out.dim() == 2 && state.dim() == 4 && max_q >= 1 && len >= 32 && len % 32 == 0,
             "hgrn2 ranks");
  a.T = qv.size(0);
  a.H = state.size(1);
  a.dk = state.size(2);
  a.dv = state.size(3);
  SHAI_CHECK((a.dk == 64 && a.dv == 64) || (a.dk == 64 && a.dv == 128) || (a.dk == 128 && a.dv == 64) ||
                 (a.dk == 128 && a.dv == 128) || (a.dk == 256 && a.dv == 256), "stored head sizes: 64 / 128 each, or 256 / 256");
  SHAI_CHECK(a.H >= 1 && a.H <= 65535 && qv.size(1) == (long)a.H * (a.dk + a.dv) && z.size(0) == a.T &&
                 z.size(1) == (long)a.H * a.dk && bias.numel() == (long)a.H * a.dk && lower.numel() == bias.numel() && gain.numel() == a.dv &&
                 out.size(0) == a.T && out.size(1) == (long)a.H * a.dv && pos.numel() >= a.T && vdim >= 1 && vdim <= a.dv,
             "hgrn2 shapes");
  a.B = a.T;
  a.vdim = vdim;
  a.eps = eps;
  a.len = len;
  a.segments = 1;
  if (q_lens) {
    SHAI_CHECK(q_start.has_value(), "prefill: q_start");
    check_i32(*q_lens, "q_lens");
    check_i32(*q_start, "q_start");
    a.B = q_lens->numel();
    SHAI_CHECK(q_start->numel() == a.B, "one start per sequence");
    a.q_lens = q_lens->data_ptr<int>();
    a.q_start = q_start->data_ptr<int>();
    if (!f32) a.segments = (max_q + len - 1) / len;
  }
  SHAI_CHECK(slots.numel() >= a.B && a.B <= 65535 && a.segments <= 65535, "one state slot per sequence");
  SHAI_CHECK(a.segments == 1 || (ws.scalar_type() == at::kFloat && ws.is_contiguous() &&
                                 ws.numel() >= (long)a.B * a.segments * a.H * a.dk * (a.dv + 1)), "hgrn2 workspace");
  a.qv = qv.data_ptr();
  a.z = z.data_ptr<float>();
  a.bias = bias.data_ptr<float>();
  a.lower = lower.data_ptr<float>();
  a.gain = gain.data_ptr<float>();
  a.state = state.data_ptr<float>();
  a.out = out.data_ptr();
  a.pos = pos.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.ws = a.segments > 1 ? ws.data_ptr<float>() : nullptr;
  if (a.T == 0) return;
  if (f32 || !a.q_lens) shai_lm::launch_hgrn2_rows(a, f32, stream());
  else shai_lm::launch_hgrn2_chunks(a, stream());
}

// Delta rule (conv, beta, ring given) or retention (rope given): sizes checked, everything but the workspace filled in
shai_lm::RuleArgs rule_args(const Tensor& x, const Tensor& gate, const Tensor& state, const Tensor& out, const Tensor& pos,
                            const Tensor& slots, int64_t kv_heads, int64_t dim, int64_t vdim, int64_t gate_kind, double eps,
                            const Tensor& rate, const optional<Tensor>& decay, const optional<Tensor>& beta,
                            const optional<Tensor>& conv, const optional<Tensor>& bias, const optional<Tensor>& gain,
                            const optional<Tensor>& ring, const optional<Tensor>& rope, const optional<Tensor>& q_start,
                            const optional<Tensor>& q_lens) {
  const auto dt = x.scalar_type();
  is_f32(x);
  check_rows16(x, dt, "x");
  check_rows(gate, dt, "gate");
  check_rows(out, dt, "out");
  check(state, at::kFloat, "state");
  check(rate, at::kFloat, "rate");
  check_i32(pos, "pos");
  check_i32(slots, "slots");
  shai_lm::RuleArgs a{};
  SHAI_CHECK(state.dim() == 4, "state must be [slots, H, dk, dv]");
  a.T = x.size(0);
  a.H = state.size(1);
  a.dk = state.size(2);
  a.dv = state.size(3);
  a.G = kv_heads;
  SHAI_CHECK((a.dk == 64 && a.dv == 64) || (a.dk == 64 && a.dv == 128) || (a.dk == 128 && a.dv == 64) ||
                 (a.dk == 128 && a.dv == 128) || (a.dk == 256 && a.dv == 256), "stored head sizes: 64 / 128 each, or 256 / 256");
  const long channels = 2L * a.G * a.dk + (long)a.H * a.dv;
  SHAI_CHECK(a.H >= 1 && a.H <= 65535 && a.G >= 1 && a.H % a.G == 0 && x.size(1) == channels && gate.size(0) == a.T &&
                 gate.size(1) == (long)a.H * a.dv && out.size(0) == a.T && out.size(1) == gate.size(1) && pos.numel() >= a.T &&
                 dim >= 1 && dim <= a.dk && vdim >= 1 && vdim <= a.dv && (gate_kind == 0 || gate_kind == 1), "rule shapes");
  a.dim = dim;
  a.vdim = vdim;
  a.gate_kind = gate_kind;
  a.eps = eps;
  a.x = x.data_ptr();
  a.gate = gate.data_ptr();
  a.state = state.data_ptr<float>();
  a.out = out.data_ptr();
  a.rate = rate.data_ptr<float>();
  a.pos = pos.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.ldx = x.stride(0);
  a.ldg = gate.stride(0);
  a.ldo = out.stride(0);
  a.taps = 1;
  if (conv) {
    SHAI_CHECK(decay.has_value() && beta.has_value() && bias.has_value() && gain.has_value() && ring.has_value(),
               "delta rule: decay, beta, bias, gain and ring");
    check(*conv, at::kFloat, "conv");
    check_rows(*decay, at::kFloat, "decay");
    check_rows(*beta, at::kFloat, "beta");
    check(*bias, at::kFloat, "bias");
    check(*gain, at::kFloat, "gain");
    check(*ring, dt, "ring");
    a.taps = conv->size(0);
    a.mode = decay->size(1) == a.H && bias->numel() == a.H ? 1 : 2;
    SHAI_CHECK(conv->dim() == 2 && a.taps >= 1 && a.taps <= 16 && conv->size(1) == channels && ring->dim() == 3 &&
                   ring->size(0) == state.size(0) && ring->size(1) == a.taps && ring->size(2) == channels && rate.numel() == a.H &&
                   gain->numel() == a.dv && beta->size(0) == a.T && beta->size(1) == a.H && decay->size(0) == a.T &&
                   (a.mode == 1 || decay->size(1) == (long)a.H * a.dk) && bias->numel() == decay->size(1), "delta rule shapes");
    a.conv = conv->data_ptr<float>();
    a.decay = decay->data_ptr<float>();
    a.beta = beta->data_ptr<float>();
    a.bias = bias->data_ptr<float>();
    a.gain = gain->data_ptr<float>();
    a.ring = ring->data_ptr();
    a.ldd = decay->stride(0);
    a.ldb = beta->stride(0);
  } else {
    SHAI_CHECK(rope.has_value(), "retention: rope");
    check(*rope, at::kFloat, "rope");
    SHAI_CHECK(a.G == a.H && rope->dim() == 2 && rope->size(0) >= a.T && rope->size(1) % 2 == 0 && rope->size(1) <= dim &&
                   rate.numel() == 2L * a.H, "retention shapes");
    a.rope = rope->data_ptr<float>();
    a.rot = rope->size(1);
  }
  a.B = a.T;
  if (q_lens) {
    SHAI_CHECK(q_start.has_value(), "prefill: q_start");
    check_i32(*q_lens, "q_lens");
    check_i32(*q_start, "q_start");
    a.B = q_lens->numel();
    SHAI_CHECK(q_start->numel() == a.B, "one start per sequence");
    a.q_lens = q_lens->data_ptr<int>();
    a.q_start = q_start->data_ptr<int>();
  }
  SHAI_CHECK(slots.numel() >= a.B && a.B <= 65535, "one state slot per sequence");
  return a;
}

void rule_rows(const Tensor& x, const Tensor& gate, const Tensor& state, const Tensor& out, const Tensor& pos,
               const Tensor& slots, int64_t kv_heads, int64_t dim, int64_t vdim, int64_t gate_kind, double eps,
               const Tensor& rate, const optional<Tensor>& decay, const optional<Tensor>& beta, const optional<Tensor>& conv,
               const optional<Tensor>& bias, const optional<Tensor>& gain, const optional<Tensor>& ring,
               const optional<Tensor>& rope, const optional<Tensor>& q_start, const optional<Tensor>& q_lens) {
  const shai_lm::RuleArgs a = rule_args(x, gate, state, out, pos, slots, kv_heads, dim, vdim, gate_kind, eps, rate, decay,
                                        beta, conv, bias, gain, ring, rope, q_start, q_lens);
  if (a.T > 0) shai_lm::launch_rule_rows(a, is_f32(x), stream());
}

// q_start / q_lens describe the packed rows of x (their sum is T); max_q: the largest of q_lens
void rule_chunks(const Tensor& x, const Tensor& gate, const Tensor& state, const Tensor& out, const Tensor& pos,
                 const Tensor& slots, int64_t kv_heads, int64_t dim, int64_t vdim, int64_t gate_kind, double eps,
                 const Tensor& rate, const optional<Tensor>& decay, const optional<Tensor>& beta, const optional<Tensor>& conv,
                 const optional<Tensor>& bias, const optional<Tensor>& gain, const optional<Tensor>& ring,
                 const optional<Tensor>& rope, const Tensor& q_start, const Tensor& q_lens, const Tensor& ws, int64_t max_q,
                 int64_t head0, int64_t heads, int64_t seg, const optional<Tensor>& seg_ws) {
  shai_lm::RuleArgs a = rule_args(x, gate, state, out, pos, slots, kv_heads, dim, vdim, gate_kind, eps, rate, decay, beta,
                                  conv, bias, gain, ring, rope, q_start, q_lens);
  SHAI_CHECK(x.scalar_type() == at::kBFloat16, "chunks: bf16 rows");
  check_rows16(gate, at::kBFloat16, "gate");
  check_rows16(out, at::kBFloat16, "out");
  check(ws, at::kByte, "ws");
  const int group = a.H / a.G;
  a.ws_chunks = (long)a.T / 32 + a.B;
  SHAI_CHECK(head0 >= 0 && heads >= 1 && head0 + heads <= a.H && head0 % group == 0 && heads % group == 0 && max_q >= 1 &&
                 ws.numel() >= a.ws_chunks * shai_lm::rule_chunk_bytes(a.dk, a.dv, heads, a.mode == 2 ? heads : heads / group, a.mode == 2),
             "rule_chunks: whole groups of heads, workspace");
  a.ws = ws.data_ptr();
  a.head0 = head0;
  a.heads = heads;
  a.max_q = std::min<int64_t>(max_q, a.T);
  a.seg = (a.max_q + 31) / 32 * 32;
  a.cuts = 1;
  if (seg > 0 && seg < a.max_q) {
    SHAI_CHECK(seg % 32 == 0 && seg_ws, "rule_chunks: segments are whole chunks and have a workspace");
    check(*seg_ws, at::kByte, "seg_ws");
    a.seg = seg;
    a.cuts = (a.max_q + a.seg - 1) / a.seg;
    SHAI_CHECK(seg_ws->numel() >= ((long)a.T / seg + a.B) * shai_lm::rule_segment_bytes(a.dk, a.dv, heads, a.mode == 0) &&
                   (long)heads * a.B * a.cuts * 8 < 0x7fffffffL, "rule_chunks: workspace of segments");
    a.seg_ws = static_cast<float*>(seg_ws->data_ptr());
  }
  if (a.T > 0) shai_lm::launch_rule_chunks(a, stream());
}

int64_t rule_segment_bytes(int64_t dk, int64_t dv, int64_t heads, bool retention) {
  return shai_lm::rule_segment_bytes(dk, dv, heads, retention);
}

int64_t rule_chunk_bytes(int64_t dk, int64_t dv, int64_t heads, int64_t keys, bool channel) {
  return shai_lm::rule_chunk_bytes(dk, dv, heads, keys, channel);
}

void ring_commit(const Tensor& x, const Tensor& ring, const Tensor& pos, const Tensor& q_start, const Tensor& q_lens,
                 const Tensor& slots) {
  check_rows(x, ring.scalar_type(), "x");
  check(ring, ring.scalar_type(), "ring");
  for (auto* t : {&pos, &q_start, &q_lens, &slots}) check_i32(*t, "ring_commit tensor");
  shai_lm::RingArgs a{};
  SHAI_CHECK(ring.dim() == 3 && x.size(1) == ring.size(2), "ring must be [slots, taps, columns of x]");
  a.B = q_lens.numel();
  a.n_slots = ring.size(0);
  a.taps = ring.size(1);
  a.channels = ring.size(2);
  a.ldx = x.stride(0);
  SHAI_CHECK(a.taps >= 1 && q_start.numel() == a.B && slots.numel() >= a.B && pos.numel() >= x.size(0) && a.B <= 65535, "ring_commit shapes");
  a.x = x.data_ptr();
  a.ring = ring.data_ptr();
  a.pos = pos.data_ptr<int>();
  a.q_start = q_start.data_ptr<int>();
  a.q_lens = q_lens.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  if (a.B > 0) shai_lm::launch_ring_commit(a, is_f32(ring), stream());
}

const float* route_bias(const optional<Tensor>& bias, int E) {
  if (!bias) return nullptr;
  check(*bias, at::kFloat, "bias");
  SHAI_CHECK(bias->numel() == E, "router bias must be [E]");
  return bias->data_ptr<float>();
}

void moe_route(const Tensor& logits, int64_t groups, int64_t keep, const Tensor& ids, const Tensor& wts,
               const optional<Tensor>& bias, bool renorm) {
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
  SHAI_CHECK(!renorm || a.top <= 64, "route: up to 64 renormalised picks");
  a.bias = route_bias(bias, a.E);
  a.renorm = renorm;
  a.logits = logits.data_ptr<float>();
  a.ids = ids.data_ptr<int>();
  a.wts = wts.data_ptr<float>();
  if (a.T > 0) shai_lm::launch_route(a, stream());
}

// logits -> picks -> slots for up to 16 tokens in one launch (moe_route + moe_plan with 16-row tiles)
void moe_route_plan(const Tensor& logits, int64_t groups, int64_t keep, const Tensor& ids, const Tensor& wts,
                    const Tensor& offsets, const Tensor& token_of, const Tensor& slot_of, const Tensor& tiles,
                    const optional<Tensor>& bias, bool renorm) {
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
  SHAI_CHECK(!renorm || r.top <= 64, "route: up to 64 renormalised picks");
  r.bias = route_bias(bias, r.E);
  r.renorm = renorm;
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

// gate_w: gate logits per head (1 or dv).  own_kv false: rows are [q | gate], the cache holds another layer's keys and values
shai_lm::AttnArgs attn_args(const Tensor& qkvg, const Tensor& kc, const Tensor& vc, const Tensor* o, int64_t heads,
                            bool per_element = false, bool own_kv = true, bool tied = false) {
  const auto dt = qkvg.scalar_type();
  is_f32(qkvg);
  check_rows16(qkvg, dt, "qkvg");
  check(kc, dt, "k_cache");
  check(vc, dt, "v_cache");
  SHAI_CHECK(kc.dim() == 4 && vc.dim() == 4 && kc.size(0) == vc.size(0) && kc.size(1) == vc.size(1) &&
                 kc.size(2) == 64 && vc.size(2) == 64, "caches must be [blocks, G, 64, dk | dv]");
  shai_lm::AttnArgs a{};
  a.T = qkvg.size(0);
  a.ld = qkvg.stride(0);
  a.H = heads;
  a.G = kc.size(1);
  a.dk = kc.size(3);
  a.dv = vc.size(3);
  SHAI_CHECK(a.dk % 64 == 0 && a.dv % 64 == 0 && ((a.dk <= 128 && a.dv <= 128) || (a.dk == 256 && a.dv == 256)),
             "stored head sizes: 64 / 128 each, or 256 / 256");
  SHAI_CHECK(a.H >= 1 && a.G >= 1 && a.H % a.G == 0, "query heads must be a multiple of kv heads");
  a.own_kv = own_kv;
  a.out_scale = 1.f;
  if (tied) {  // [q | k]: the values are the keys, no gate
    SHAI_CHECK(own_kv && !per_element && a.dk == a.dv, "keys as values: one head size");
    a.v_off = a.H * a.dk;
    SHAI_CHECK(qkvg.size(1) >= (long)(a.H + a.G) * a.dk, "qk row too short");
  } else {
    a.v_off = (a.H + a.G) * a.dk;
    a.gate_w = per_element ? a.dv : 1;
    a.gate_off = a.H * a.dk + (own_kv ? a.G * (a.dk + a.dv) : 0);
    SHAI_CHECK(qkvg.size(1) % 8 == 0 && qkvg.size(1) >= (long)a.gate_off + (long)a.H * a.gate_w, "qkvg row too short");
  }
  a.qkvg = qkvg.data_ptr();
  a.kc = kc.data_ptr();
  a.vc = vc.data_ptr();
  if (o) {
    check_rows16(*o, dt, "o");
    SHAI_CHECK(o->size(0) == a.T && o->size(1) == (long)a.H * a.dv, "o must be [T, H dv]");
    a.o = o->data_ptr();
    a.ldo = o->stride(0);
  }
  return a;
}

// rotation and norm of q and k: angles of every row, the head size before padding
void set_turn(shai_lm::AttnArgs& a, const optional<Tensor>& rope, int64_t dim, double eps, const optional<Tensor>& q_gain,
              const optional<Tensor>& k_gain) {
  if (!rope) return;
  SHAI_CHECK(q_gain.has_value() == k_gain.has_value(), "gains of both queries and keys, or none");
  if (q_gain) {
    check(*q_gain, at::kFloat, "q_gain");
    check(*k_gain, at::kFloat, "k_gain");
    SHAI_CHECK(q_gain->numel() == a.dk && k_gain->numel() == a.dk, "gains must be [dk]");
    a.q_gain = q_gain->data_ptr<float>();
    a.k_gain = k_gain->data_ptr<float>();
  }
  check(*rope, at::kFloat, "rope");
  SHAI_CHECK(rope->dim() == 2 && rope->size(0) >= a.T && rope->size(1) % 2 == 0 && dim >= 1 && dim <= a.dk &&
                 rope->size(1) <= dim, "rope must be [T, rotated dimensions of a head]");
  a.rope = rope->data_ptr<float>();
  a.rot = rope->size(1);
  a.dim = dim;
  a.eps = eps;
}

// attention without gates: factors on the scores, sinks, factor on the output
void set_ungated(shai_lm::AttnArgs& a, const optional<Tensor>& temp, const optional<Tensor>& sink, double out_scale) {
  if (!sink) return;
  SHAI_CHECK(temp.has_value(), "attention without gates: temp and sink");
  check_f32(*temp, "temp");
  check_f32(*sink, "sink");
  SHAI_CHECK(temp->numel() == a.H && sink->numel() == a.H, "temp and sink must be [H]");
  a.temp = temp->data_ptr<float>();
  a.sink = sink->data_ptr<float>();
  a.out_scale = out_scale;
}

// q of the step in place and, with own keys, k and v into the cache
void head_prep(const Tensor& qkvg, const Tensor& kc, const Tensor& vc, const Tensor& slots, int64_t heads, const Tensor& rope,
               int64_t dim, double eps, bool own_kv, bool tied, const optional<Tensor>& q_gain, const optional<Tensor>& k_gain) {
  shai_lm::AttnArgs a = attn_args(qkvg, kc, vc, nullptr, heads, false, own_kv, tied);
  set_turn(a, rope, dim, eps, q_gain, k_gain);
  check_i32(slots, "slots");
  SHAI_CHECK(slots.numel() >= a.T, "one slot per row");
  a.slots = slots.data_ptr<int>();
  if (a.T > 0) shai_lm::launch_head_prep(a, is_f32(qkvg), stream());
}

void kv_store(const Tensor& qkvg, const Tensor& kc, const Tensor& vc, const Tensor& slots, int64_t heads, bool tied) {
  shai_lm::AttnArgs a = attn_args(qkvg, kc, vc, nullptr, heads, false, true, tied);
  check_i32(slots, "slots");
  SHAI_CHECK(slots.numel() >= a.T, "one slot per row");
  a.slots = slots.data_ptr<int>();
  if (a.T > 0) shai_lm::launch_kv_store(a, is_f32(qkvg), stream());
}

// `chunk`: the size of the chunks or, with `window`, of the sliding window
void gated_attn_prefill(const Tensor& qkvg, const Tensor& kc, const Tensor& vc, const Tensor& o, const Tensor& bt,
                        const Tensor& ctx, const Tensor& q_lens, const Tensor& q_start, int64_t max_q, int64_t heads,
                        int64_t chunk, double scale, bool window, bool per_element, bool own_kv, const optional<Tensor>& temp,
                        const optional<Tensor>& sink, double out_scale) {
  shai_lm::AttnArgs a = attn_args(qkvg, kc, vc, &o, heads, per_element, own_kv, sink.has_value());
  set_ungated(a, temp, sink, out_scale);
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
  a.chunk = std::min<int64_t>(chunk, 1 << 30);
  a.window = window;
  a.scale = scale;
  shai_lm::launch_attn_prefill(a, is_f32(qkvg), stream());
}

void gated_attn_decode(const Tensor& qkvg, const Tensor& kc, const Tensor& vc, const Tensor& o, const Tensor& bt,
                       const Tensor& ctx, const Tensor& slots, const Tensor& ws, int64_t heads, int64_t splits,
                       int64_t chunk, double scale, bool window, bool per_element, bool own_kv,
                       const optional<Tensor>& rope, int64_t dim, double eps, const optional<Tensor>& q_gain,
                       const optional<Tensor>& k_gain, const optional<Tensor>& temp, const optional<Tensor>& sink,
                       double out_scale) {
  shai_lm::AttnArgs a = attn_args(qkvg, kc, vc, &o, heads, per_element, own_kv, sink.has_value());
  set_turn(a, rope, dim, eps, q_gain, k_gain);
  set_ungated(a, temp, sink, out_scale);
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
  a.chunk = std::min<int64_t>(chunk, 1 << 30);
  a.window = window;
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
  m.def("lm_gemm(Tensor a, Tensor w, Tensor(a!) c, Tensor? tiles, Tensor? offsets, Tensor? gather, int bm, int epi, float param, Tensor(b!)? side=None, Tensor? vec=None, Tensor? rope=None, int head=0, int rot0=0, Tensor? ids=None, Tensor? table=None, int act=0) -> ()");
  m.def("lm_gemm_heads(Tensor a, Tensor w, Tensor(a!) c) -> ()");
  m.def("lm_gemm_parts(Tensor a, Tensor w, Tensor(a!) c) -> ()");
  m.def("residual_norm(Tensor? x, Tensor? ids, Tensor? table, float scale, Tensor? delta, Tensor? wb, float mult, Tensor? step, Tensor(a!)? x_out, Tensor? rows, Tensor? w, float eps, int width, Tensor(b!)? h, Tensor? cw=None, Tensor(c!)? state=None, Tensor(d!)? tail=None, Tensor? row_seq=None, Tensor? q_start=None, Tensor? q_lens=None, Tensor? pos=None, Tensor? slots=None, Tensor? bb=None, Tensor? b=None, Tensor? ye=None, Tensor? slot_of=None, Tensor? wts=None) -> ()");
  m.def("conv_commit(Tensor(a!) state, Tensor tail, Tensor q_lens, Tensor slots) -> ()");
  m.def("rope_rows(Tensor pos, Tensor freq, Tensor(a!) out) -> ()");
  m.def("latent_prep(Tensor d, Tensor wq, Tensor wkv, Tensor rope, Tensor slots, Tensor(a!) cache, Tensor(b!) cq, float eps, int q_rank, int kv_rank) -> ()");
  m.def("latent_gather(Tensor cache, Tensor block_table, Tensor seqs, Tensor ctx, Tensor start, int max_ctx, Tensor(a!) out) -> ()");
  m.def("latent_attn_prefill(Tensor q, Tensor kv, Tensor lat, Tensor(a!) o, Tensor ctx, Tensor q_lens, Tensor q_start, Tensor kv_start, Tensor sink, int max_q, int heads, int np, int rot, int rank, float scale) -> ()");
  m.def("latent_attn_rows(Tensor ql, Tensor q, Tensor cache, Tensor(a!) o, Tensor block_table, Tensor? seqs, Tensor ctx, Tensor sink, Tensor(b!) ws, int splits, int np, int rot, float scale) -> ()");
  m.def("mingru_scan(Tensor zx, Tensor g, Tensor bias, Tensor(a!) state, Tensor(b!) out, Tensor pos, Tensor? q_start, Tensor? q_lens, Tensor slots, Tensor(c!) ws, int max_q, int len) -> ()");
  m.def("moe_route(Tensor logits, int groups, int keep, Tensor(a!) ids, Tensor(b!) wts, Tensor? bias=None, bool renorm=False) -> ()");
  m.def("moe_route_plan(Tensor logits, int groups, int keep, Tensor(a!) ids, Tensor(b!) wts, Tensor(c!) offsets, Tensor(d!) token_of, Tensor(e!) slot_of, Tensor(f!) tiles, Tensor? bias=None, bool renorm=False) -> ()");
  m.def("moe_plan(Tensor ids, int bm, Tensor(a!) offsets, Tensor(b!) token_of, Tensor(c!) slot_of, Tensor(d!) tiles) -> ()");
  m.def("kv_store(Tensor qkvg, Tensor(a!) k_cache, Tensor(b!) v_cache, Tensor slots, int heads, bool tied=False) -> ()");
  m.def("head_prep(Tensor(a!) qkvg, Tensor(b!) k_cache, Tensor(c!) v_cache, Tensor slots, int heads, Tensor rope, int dim, float eps, bool own_kv, bool tied=False, Tensor? q_gain=None, Tensor? k_gain=None) -> ()");
  m.def("hgrn2(Tensor qv, Tensor z, Tensor bias, Tensor lower, Tensor gain, Tensor(a!) state, Tensor(b!) out, Tensor pos, Tensor? q_start, Tensor? q_lens, Tensor slots, Tensor(c!) ws, int max_q, int len, int vdim, float eps) -> ()");
  m.def("rule_rows(Tensor x, Tensor gate, Tensor(a!) state, Tensor(b!) out, Tensor pos, Tensor slots, int kv_heads, int dim, int vdim, int gate_kind, float eps, Tensor rate, Tensor? decay=None, Tensor? beta=None, Tensor? conv=None, Tensor? bias=None, Tensor? gain=None, Tensor(c!)? ring=None, Tensor? rope=None, Tensor? q_start=None, Tensor? q_lens=None) -> ()");
  m.def("rule_chunks(Tensor x, Tensor gate, Tensor(a!) state, Tensor(b!) out, Tensor pos, Tensor slots, int kv_heads, int dim, int vdim, int gate_kind, float eps, Tensor rate, Tensor? decay=None, Tensor? beta=None, Tensor? conv=None, Tensor? bias=None, Tensor? gain=None, Tensor? ring=None, Tensor? rope=None, *, Tensor q_start, Tensor q_lens, Tensor(c!) ws, int max_q, int head0, int heads, int seg=0, Tensor(d!)? seg_ws=None) -> ()");
  m.def("rule_segment_bytes(int dk, int dv, int heads, bool retention) -> int", &rule_segment_bytes);
  m.def("rule_chunk_bytes(int dk, int dv, int heads, int keys, bool channel) -> int", &rule_chunk_bytes);
  m.def("ring_commit(Tensor x, Tensor(a!) ring, Tensor pos, Tensor q_start, Tensor q_lens, Tensor slots) -> ()");
  m.def("gated_attn_prefill(Tensor qkvg, Tensor k_cache, Tensor v_cache, Tensor(a!) o, Tensor block_table, Tensor ctx_lens, Tensor q_lens, Tensor q_start, int max_q, int heads, int chunk, float scale, bool window=False, bool per_element=False, bool own_kv=True, Tensor? temp=None, Tensor? sink=None, float out_scale=1.) -> ()");
  m.def("gated_attn_decode(Tensor qkvg, Tensor(a!) k_cache, Tensor(b!) v_cache, Tensor(c!) o, Tensor block_table, Tensor ctx_lens, Tensor slots, Tensor(d!) ws, int heads, int splits, int chunk, float scale, bool window=False, bool per_element=False, bool own_kv=True, Tensor? rope=None, int dim=0, float eps=0., Tensor? q_gain=None, Tensor? k_gain=None, Tensor? temp=None, Tensor? sink=None, float out_scale=1.) -> ()");
  m.def("sample(Tensor logits, Tensor temps, Tensor top_k, Tensor top_p, Tensor uniforms, Tensor(a!) out) -> ()");
  m.def("token_feedback(Tensor(a!) ids, Tensor rowmap, Tensor prev) -> ()");
}

TORCH_LIBRARY_IMPL(shai, CUDA, m) {
  m.impl("embed_norm", &embed_norm);
  m.impl("add_norm", &add_norm);
  m.impl("lm_gemm", &lm_gemm);
  m.impl("lm_gemm_heads", &lm_gemm_heads);
  m.impl("lm_gemm_parts", &lm_gemm_parts);
  m.impl("residual_norm", &residual_norm);
  m.impl("conv_commit", &conv_commit);
  m.impl("rope_rows", &rope_rows);
  m.impl("latent_prep", &latent_prep);
  m.impl("latent_gather", &latent_gather);
  m.impl("latent_attn_prefill", &latent_attn_prefill);
  m.impl("latent_attn_rows", &latent_attn_rows);
  m.impl("mingru_scan", &mingru_scan);
  m.impl("moe_route", &moe_route);
  m.impl("moe_route_plan", &moe_route_plan);
  m.impl("moe_plan", &moe_plan);
  m.impl("kv_store", &kv_store);
  m.impl("head_prep", &head_prep);
  m.impl("hgrn2", &hgrn2);
  m.impl("rule_rows", &rule_rows);
  m.impl("rule_chunks", &rule_chunks);
  m.impl("ring_commit", &ring_commit);
  m.impl("gated_attn_prefill", &gated_attn_prefill);
  m.impl("gated_attn_decode", &gated_attn_decode);
  m.impl("sample", &sample);
  m.impl("token_feedback", &token_feedback);
}
