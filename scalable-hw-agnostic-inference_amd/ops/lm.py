"""Decoder-block operators with an fp32 residual stream (``csrc/lm``, ``libshai_lm.so``).

What a layer-list decoder needs beyond the Llama path of :mod:`shai_amd.ops`: an n-gram embedding, a residual-add +
RMSNorm with the residual kept in fp32, one GEMM for dense and expert-grouped products, mixture-of-experts routing,
and attention restricted to fixed-size chunks of the sequence with a per-head output gate.  Every op takes bf16 or fp32
weights and activations; norms, routing, attention scores and the residual are fp32 in both.

Layout rules shared by all of them: the model width is padded to a multiple of 64 (``pad64``; the pad columns of
activations and weights are zero), so a GEMM's K is always a multiple of 64.

GPU tensors run the native kernels (raising if the library is missing); CPU tensors run
:mod:`shai_amd.ops.lm_reference` (tests).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch

from .. import native
from . import lm_reference as ref

EPI_NONE, EPI_CLAMP_GLU, EPI_SOFTCAP = 0, 1, 2
MAX_EXPERTS, MAX_TOP = 1024, 64


def pad64(n: int) -> int:
    return (n + 63) // 64 * 64


def head_pad(dim: int, vdim: int) -> tuple:
    """Stored (query/key, value) head sizes: the next of 64 / 128 each, 256 for both when either is larger."""
    if max(dim, vdim) > 256:
        raise ValueError(f"attention head sizes up to 256 are supported, got {dim} / {vdim}")
    if max(dim, vdim) > 128:
        return 256, 256
    return pad64(dim), pad64(vdim)


def _K():
    return native.lm_ops()


@dataclass
class Experts:
    """Routed rows of one mixture-of-experts layer: expert outputs ``y`` [T * top, D] in slot order, ``slot_of``
    [T, top] (the slot of each token's k-th expert), combine weights [T, top], and the dense (shared expert) output."""
    y: torch.Tensor
    slot_of: torch.Tensor
    weights: torch.Tensor
    dense: Optional[torch.Tensor] = None


@dataclass
class Plan:
    """Rows of a step sorted by expert: slots offsets[e] .. offsets[e + 1] - 1 belong to expert e; ``token_of`` is each
    slot's token.  ``tiles`` [n, 2] lists (expert, first slot) of every ``bm``-row tile (expert -1: unused entry)."""
    offsets: torch.Tensor
    token_of: torch.Tensor
    slot_of: torch.Tensor
    tiles: torch.Tensor
    bm: int


def embed_norm(ids, prev, table, bigram, mul_prev: int, mul_cur: int, w, eps: float, width: int):
    """x = table[id] (+ bigram[row(prev, id)]) in fp32 and h = RMSNorm(x) (1 + w) in the tables' dtype.
    ``prev`` is -1 for a sequence's first token (the bigram table's last row).  Returns (x, h)."""
    if not table.is_cuda:
        return ref.embed_norm(ids, prev, table, bigram, mul_prev, mul_cur, w, eps, width)
    T, D = ids.shape[0], table.shape[1]
    x = torch.empty(T, D, dtype=torch.float32, device=table.device)
    h = torch.empty(T, D, dtype=table.dtype, device=table.device)
    _K().embed_norm(ids, prev, table, bigram, int(mul_prev), int(mul_cur), w, float(eps), int(width), x, h)
    return x, h


def add_norm(x, delta, inject, w, eps: float, width: int, dtype, rows=None):
    """x += delta (+ inject) in place and h = RMSNorm(x) (1 + w) in ``dtype`` (``w`` None: no norm, returns None).
    delta: None, a [T, D] tensor, or :class:`Experts` (weighted expert outputs + shared expert).  With ``rows`` (int32)
    only those rows are normalised, h [len(rows), D], and x is left as it was."""
    if not x.is_cuda:
        return ref.add_norm(x, delta, inject, w, eps, width, dtype, rows)
    n = x.shape[0] if rows is None else rows.shape[0]
    h = torch.empty(n, x.shape[1], dtype=dtype, device=x.device) if w is not None else None
    moe = isinstance(delta, Experts)
    dense = delta.dense if moe else delta
    _K().add_norm(x, dense, delta.y if moe else None, delta.slot_of if moe else None, delta.weights if moe else None,
                  inject, rows, w, float(eps), int(width), h)
    return h


def matmul(a, w, out_dtype=None, epi: int = EPI_NONE, param: float = 0.0, plan: Optional[Plan] = None,
           gather: bool = False):
    """c = epi(a w^T).  Dense: a [M, K], w [N, K].  Grouped (``plan``): w [E, N, K], row s of c belongs to the expert of
    slot s and reads a[token_of[s]] (``gather``) or a[s].

    EPI_CLAMP_GLU: w rows are (gate_i, up_i) pairs; with g = min(gate, param), u = clamp(up, +-param) the N / 2 outputs
    are g sigmoid(1.702 g) (u + 1).  EPI_SOFTCAP: param * tanh(c / param)."""
    out_dtype = out_dtype or a.dtype
    if not a.is_cuda:
        return ref.matmul(a, w, out_dtype, epi, param, plan, gather)
    N = w.shape[-2]
    M = plan.token_of.shape[0] if plan is not None else a.shape[0]
    c = torch.empty(M, N // 2 if epi == EPI_CLAMP_GLU else N, dtype=out_dtype, device=a.device)
    if plan is None:
        _K().lm_gemm(a, w, c, None, None, None, 0, int(epi), float(param))
    else:
        _K().lm_gemm(a, w, c, plan.tiles, plan.offsets, plan.token_of if gather else None, plan.bm, int(epi),
                     float(param))
    return c


def glu_with_side(a, w, side: int, param: float):
    """One product for two consumers of ``a``: the rows of w but the last ``side`` are (gate, up) pairs of a clamped GLU
    (:func:`matmul` EPI_CLAMP_GLU), the last ``side`` rows a plain product in fp32.  Returns (glu, side product)."""
    if not a.is_cuda:
        return ref.matmul(a, w[:-side], a.dtype, EPI_CLAMP_GLU, param), ref.matmul(a, w[-side:], torch.float32, 0, 0.0)
    M, N = a.shape[0], w.shape[0]
    c = torch.empty(M, (N - side) // 2, dtype=a.dtype, device=a.device)
    s = torch.empty(M, side, dtype=torch.float32, device=a.device)
    _K().lm_gemm(a, w, c, None, None, None, 0, EPI_CLAMP_GLU, float(param), s)
    return c, s


def grouped_bm(rows: int, experts: int) -> int:
    """Row tile of a grouped product over ``rows`` slots: 16-row streaming tiles while an expert sees few rows, LDS
    tiles of 128 rows once it sees enough of them to be compute-bound, of 256 when those fill up."""
    return 16 if rows < 48 * experts else 128 if rows < 512 * experts else 256


def route(logits, top: int, groups: int, keep: int):
    """Group-limited top-k routing from fp32 logits [T, E]: (expert ids int32 [T, top], softmax scores fp32 [T, top]).
    The E experts form ``groups`` equal runs; only the ``keep`` runs with the largest best score are eligible."""
    if not logits.is_cuda:
        return ref.route(logits, top, groups, keep)
    T = logits.shape[0]
    ids = torch.empty(T, top, dtype=torch.int32, device=logits.device)
    wts = torch.empty(T, top, dtype=torch.float32, device=logits.device)
    _K().moe_route(logits, int(groups), int(keep), ids, wts)
    return ids, wts


def plan_experts(ids, experts: int) -> Plan:
    """Sort the (token, k) pairs of ``ids`` [T, top] by expert."""
    T, top = ids.shape
    P = T * top
    bm = grouped_bm(P, experts)
    if not ids.is_cuda:
        return ref.plan_experts(ids, experts, bm)
    i32 = lambda *s: torch.empty(*s, dtype=torch.int32, device=ids.device)
    plan = Plan(i32(experts + 1), i32(P), i32(T, top), i32(min(P, experts + P // bm), 2), bm)
    _K().moe_plan(ids, int(bm), plan.offsets, plan.token_of, plan.slot_of, plan.tiles)
    return plan


def route_experts(logits, top: int, groups: int, keep: int):
    """:func:`route` and :func:`plan_experts` -> (combine weights [T, top], plan); one launch for a few tokens."""
    T, E = logits.shape
    if not logits.is_cuda or T > 16 or E > 256 or grouped_bm(T * top, E) != 16:
        ids, wts = route(logits, top, groups, keep)
        return wts, plan_experts(ids, E)
    P = T * top
    i32 = lambda *s: torch.empty(*s, dtype=torch.int32, device=logits.device)
    ids, wts = i32(T, top), torch.empty(T, top, dtype=torch.float32, device=logits.device)
    plan = Plan(i32(E + 1), i32(P), i32(T, top), i32(min(P, E + P // 16), 2), 16)
    _K().moe_route_plan(logits, int(groups), int(keep), ids, wts, plan.offsets, plan.token_of, plan.slot_of, plan.tiles)
    return wts, plan


def chunk_attention(qkvg, k_cache, v_cache, batch, heads: int, chunk: int, scale: float):
    """Attention of one step over a paged cache: softmax over the keys j <= i of position i's own chunk (positions
    chunk * n .. chunk * (n + 1) - 1), each head's output times sigmoid(its gate).

    ``qkvg`` [T, >= H dk + G (dk + dv) + H] holds q, k, v and the gate logits of the step's rows; k / v are written to
    the caches [blocks, G, 64, dk | dv] at ``batch.slots`` (-1: padding row).  Returns [T, H dv]."""
    if not qkvg.is_cuda:
        return ref.chunk_attention(qkvg, k_cache, v_cache, batch, heads, chunk, scale)
    dv = v_cache.shape[3]
    T = qkvg.shape[0]
    o = torch.empty(T, heads * dv, dtype=qkvg.dtype, device=qkvg.device)
    if batch.is_prefill:
        _K().kv_store(qkvg, k_cache, v_cache, batch.slots, int(heads))
        _K().chunk_attn_prefill(qkvg, k_cache, v_cache, o, batch.block_table, batch.ctx_lens, batch.q_lens,
                                batch.q_start, int(batch.S), int(heads), int(chunk), float(scale))
        return o
    ns = max(1, min(int(batch.num_splits or 1), (chunk + 63) // 64, 64))
    ws = torch.empty(T * heads * ns * (dv + 2) if ns > 1 else 0, dtype=torch.float32, device=qkvg.device)
    _K().chunk_attn_decode(qkvg, k_cache, v_cache, o, batch.block_table, batch.ctx_lens, batch.slots, ws, int(heads),
                           ns, int(chunk), float(scale))
    return o
