"""Decoder-block operators with an fp32 residual stream (``csrc/lm``, ``libshai_lm.so``).

What a layer-list decoder needs beyond the Llama path of :mod:`shai_amd.ops`: an n-gram embedding, residual-add + norm
(RMS or layer norm) with the residual kept in fp32 (optionally a norm on the added output and a short causal convolution
on the sum or its norm), one GEMM for dense, per-head and expert-grouped products, mixture-of-experts routing, attention
restricted to fixed-size chunks of the sequence or a sliding window with an output gate or causal with a sink per head,
attention over cached latents with a sink per head, a gated linear recurrence, and linear attention with a matrix state (gated,
written by the delta rule, or with a fixed decay).  Every op takes bf16 or fp32 weights and activations; norms, routing,
attention scores, rotation angles, recurrent state and the residual are fp32 in both.

Layout rules shared by all of them: the model width is padded to a multiple of 64 (``pad64``; the pad columns of
activations and weights are zero), so a GEMM's K is always a multiple of 64.

GPU tensors run the native kernels (raising if the library is missing); CPU tensors run
:mod:`shai_amd.ops.lm_reference` (tests).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, NamedTuple, Optional

import numpy as np
import torch

from .. import native
from . import lm_reference as ref

EPI_NONE, EPI_CLAMP_GLU, EPI_SOFTCAP, EPI_XIELU, EPI_ROTARY, EPI_GELU_GLU, EPI_RELU2, EPI_GELU_ROWS = range(8)
GLU_EPIS = (EPI_CLAMP_GLU, EPI_GELU_GLU)
MAX_EXPERTS, MAX_TOP = 1024, 64
MAX_TAPS = 16                # convolution taps
MAX_LATENT = 1024            # columns of a cached latent
LATENT_SHORT = 16            # portions up to this many rows attend in latent space, longer ones expand keys and values
LATENT_GROUP_ROWS = 1 << 18  # context rows that are expanded at a time
PARTS, PARTS_COLUMNS = 4, 8192   # partial sums: at most so many, of products up to so wide in a decode step
SCAN_CHUNK, SCAN_MAX_CHUNKS = 64, 64
STATE_SEGMENT, STATE_MAX_SEGMENTS = 128, 32      # rows of a matrix-state segment at least; segments at most
WHOLE = 1 << 30              # window that holds any sequence
RULE_CHUNK = 32              # rows of a chunk of the delta rule and of retention
RULE_WORKSPACE = 1 << 32     # bytes of prepared chunks at a time (more heads take several rounds)


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
           gather: bool = False, vec=None, rope=None, head: int = 0, rot0: int = 0, ids=None, table=None):
    """c = epi(a w^T).  Dense: a [M, K], w [N, K].  Grouped (``plan``): w [E, N, K], row s of c belongs to the expert of
    slot s and reads a[token_of[s]] (``gather``) or a[s].

    EPI_CLAMP_GLU: w rows are (gate_i, up_i) pairs; with g = min(gate, param), u = clamp(up, +-param) the N / 2 outputs
    are g sigmoid(1.702 g) (u + 1).  EPI_SOFTCAP: param * tanh(c / param).  EPI_XIELU: vec[0] c^2 + c / 2 above zero,
    vec[1] (exp(c) - 1 - c) + c / 2 below.  EPI_ROTARY: columns rot0 .. rot0 + dims - 1 of every ``head`` columns are
    interleaved pairs turned by the row's angles ``rope`` [M, dims] (:func:`rope_rows`).  EPI_GELU_GLU: w rows in pairs,
    gelu_tanh(gate) up.  EPI_RELU2: max(c, 0)^2.  EPI_GELU_ROWS: gelu_tanh(c) times row ids[m] of ``table`` [rows, N] (a
    view with any row stride)."""
    out_dtype = out_dtype or a.dtype
    if not a.is_cuda:
        return ref.matmul(a, w, out_dtype, epi, param, plan, gather, vec, rope, head, rot0, ids, table)
    N = w.shape[-2]
    M = plan.token_of.shape[0] if plan is not None else a.shape[0]
    c = torch.empty(M, N // 2 if epi in GLU_EPIS else N, dtype=out_dtype, device=a.device)
    if plan is None:
        _K().lm_gemm(a, w, c, None, None, None, 0, int(epi), float(param), None, vec, rope, int(head), int(rot0),
                     ids, table)
    else:
        _K().lm_gemm(a, w, c, plan.tiles, plan.offsets, plan.token_of if gather else None, plan.bm, int(epi),
                     float(param))
    return c


def matmul_with_side(a, w, side: int, epi: int = EPI_NONE, param: float = 0.0):
    """One product for two consumers of ``a``: the rows of w but the last ``side`` as in :func:`matmul` (EPI_NONE or
    EPI_CLAMP_GLU), the last ``side`` rows a plain product in fp32.  Returns (product, side product)."""
    if not a.is_cuda:
        return ref.matmul(a, w[:-side], a.dtype, epi, param), ref.matmul(a, w[-side:], torch.float32, 0, 0.0)
    M, N = a.shape[0], w.shape[0]
    c = torch.empty(M, (N - side) // (2 if epi in GLU_EPIS else 1), dtype=a.dtype, device=a.device)
    s = torch.empty(M, side, dtype=torch.float32, device=a.device)
    _K().lm_gemm(a, w, c, None, None, None, 0, int(epi), float(param), s)
    return c, s


def matmul_joint(a, w, out, act: int, side: int):
    """One product for several consumers of ``a``, into ``out`` [M, n] (a view with any row stride): its first ``act``
    columns are max(c, 0)^2, the others plain.  The last ``side`` rows of w ([n + side, K]) are a plain product in fp32,
    which is returned (None without any)."""
    n = out.shape[1]
    if not a.is_cuda:
        c = a.float() @ w.float().T
        out[:, :act] = (torch.relu(c[:, :act]) ** 2).to(out.dtype)
        out[:, act:] = c[:, act:n].to(out.dtype)
        return c[:, n:].contiguous() if side else None
    s = torch.empty(a.shape[0], side, dtype=torch.float32, device=a.device) if side else None
    _K().lm_gemm(a, w, out, None, None, None, 0, EPI_RELU2 if act else EPI_NONE, 0.0, s, act=int(act))
    return s


def matmul_parts(a, w, out_dtype=None):
    """a w^T for a consumer that adds partial sums (:func:`residual_norm`, :func:`latent_prep`): [parts, M, N] fp32
    where the product needs K cut up to fill the chip (few rows, few columns); else :func:`matmul`."""
    M, K, N = a.shape[0], a.shape[1], w.shape[0]
    if M <= 64:
        parts = PARTS if N <= PARTS_COLUMNS and K >= PARTS * 128 else 1
    else:   # tiles of 128 x 128: two for each of the 256 CUs
        tiles = -(-M // 128) * (-(-N // 128))
        parts = min(PARTS, 512 // tiles, K // 512) if tiles < 256 else 1
    if not a.is_cuda or a.dtype != torch.bfloat16 or parts <= 1:
        return matmul(a, w, out_dtype)
    c = torch.empty(parts, M, N, dtype=torch.float32, device=a.device)
    _K().lm_gemm_parts(a, w, c)
    return c


def glu_with_side(a, w, side: int, param: float):
    """:func:`matmul_with_side` with a clamped GLU."""
    return matmul_with_side(a, w, side, EPI_CLAMP_GLU, param)


def matmul_heads(a, w):
    """c[t, h] = a[t, h] w[h]^T: a [T, H, K] and w [H, N, K] (any strides between rows and heads) -> [T, H, N]."""
    if not a.is_cuda:
        return torch.einsum("thk,hnk->thn", a.float(), w.float()).to(a.dtype).contiguous()
    c = torch.empty(a.shape[0], a.shape[1], w.shape[1], dtype=a.dtype, device=a.device)
    _K().lm_gemm_heads(a, w, c)
    return c


def grouped_bm(rows: int, experts: int) -> int:
    """Row tile of a grouped product over ``rows`` slots: 16-row streaming tiles while an expert sees few rows, LDS
    tiles of 128 rows once it sees enough of them to be compute-bound, of 256 when those fill up."""
    return 16 if rows < 48 * experts else 128 if rows < 512 * experts else 256


def route(logits, top: int, groups: int, keep: int, bias=None, renorm: bool = False):
    """Group-limited top-k routing from fp32 logits [T, E]: (expert ids int32 [T, top], softmax scores fp32 [T, top]).
    The E experts form ``groups`` equal runs; only the ``keep`` runs with the largest best score are eligible.  ``bias``
    [E] (fp32) is added to the logits; ``renorm``: the scores are a softmax over the chosen logits only."""
    if not logits.is_cuda:
        return ref.route(logits, top, groups, keep, bias, renorm)
    T = logits.shape[0]
    ids = torch.empty(T, top, dtype=torch.int32, device=logits.device)
    wts = torch.empty(T, top, dtype=torch.float32, device=logits.device)
    _K().moe_route(logits, int(groups), int(keep), ids, wts, bias, bool(renorm))
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


def route_experts(logits, top: int, groups: int = 1, keep: int = 1, bias=None, renorm: bool = False):
    """:func:`route` and :func:`plan_experts` -> (combine weights [T, top], plan); one launch for a few tokens."""
    T, E = logits.shape
    if not logits.is_cuda or T > 16 or E > 256 or grouped_bm(T * top, E) != 16:
        ids, wts = route(logits, top, groups, keep, bias, renorm)
        return wts, plan_experts(ids, E)
    P = T * top
    i32 = lambda *s: torch.empty(*s, dtype=torch.int32, device=logits.device)
    ids, wts = i32(T, top), torch.empty(T, top, dtype=torch.float32, device=logits.device)
    plan = Plan(i32(E + 1), i32(P), i32(T, top), i32(min(P, E + P // 16), 2), 16)
    _K().moe_route_plan(logits, int(groups), int(keep), ids, wts, plan.offsets, plan.token_of, plan.slot_of, plan.tiles,
                        bias, bool(renorm))
    return wts, plan


class HeadTurn(NamedTuple):
    """Rotation and norm of queries and keys before they meet: dimension i < rot / 2 of a head is turned with i + rot / 2 by
    the row's angles ``rope`` [T, rot] (:func:`rope_rows`), then the head is divided by its rms over ``dim``.  With gains
    (fp32, stored head size, zero in the pads) the norm comes first, with them, and the rotation after it."""
    rope: torch.Tensor
    dim: int
    eps: float
    q_gain: Optional[torch.Tensor] = None
    k_gain: Optional[torch.Tensor] = None


@dataclass
class Ungated:
    """Attention without an output gate: the values are the projected keys (rows are [q | k]), each head's scores times
    ``temp`` [H], exp(``sink`` [H]) in its denominator, its output times ``out_scale`` (into ``out`` [T, H dv], a view with
    any row stride)."""
    temp: torch.Tensor
    sink: torch.Tensor
    out: torch.Tensor
    out_scale: float = 1.0


def gated_attention(qkvg, k_cache, v_cache, batch, heads: int, size: int, scale: float, window: bool = False,
                    per_element: bool = False, own_kv: bool = True, turn: Optional[HeadTurn] = None,
                    plain: Optional[Ungated] = None):
    """Attention of one step over a paged cache: softmax over the keys j <= i of position i's own chunk (positions
    size * n .. size * (n + 1) - 1) or, with ``window``, of the size positions that end with i; the output times
    sigmoid(gate logits), one per head or (``per_element``) per output element.

    ``qkvg`` [T, >= H dk + G (dk + dv) + gates] holds q, k, v and the gate logits of the step's rows; k / v are written to
    the caches [blocks, G, 64, dk | dv] at ``batch.slots`` (-1: padding row), with ``turn`` as the turned keys (and q may
    be prepared in place).  ``own_kv`` False: rows are [q | gates], and the cache is another layer's, which has written
    this step's rows.  ``plain``: no gates, another form of keys, values and scores (:class:`Ungated`).  Returns [T, H dv]."""
    if not qkvg.is_cuda:
        return ref.gated_attention(qkvg, k_cache, v_cache, batch, heads, size, scale, window, per_element, own_kv, turn, plain)
    dv = v_cache.shape[3]
    T = qkvg.shape[0]
    more, gains = {}, {}
    if plain is not None:
        o, more = plain.out, dict(temp=plain.temp, sink=plain.sink, out_scale=float(plain.out_scale))
    else:
        o = torch.empty(T, heads * dv, dtype=qkvg.dtype, device=qkvg.device)
    if turn is not None and turn.q_gain is not None:
        gains = dict(q_gain=turn.q_gain, k_gain=turn.k_gain)
    if batch.is_prefill:
        if turn is not None:
            _K().head_prep(qkvg, k_cache, v_cache, batch.slots, int(heads), turn.rope, int(turn.dim), float(turn.eps), own_kv,
                           tied=plain is not None, **gains)
        elif own_kv:
            _K().kv_store(qkvg, k_cache, v_cache, batch.slots, int(heads), tied=plain is not None)
        _K().gated_attn_prefill(qkvg, k_cache, v_cache, o, batch.block_table, batch.ctx_lens, batch.q_lens,
                                batch.q_start, int(batch.S), int(heads), int(size), float(scale), window, per_element, own_kv,
                                **more)
        return o
    ns = max(1, min(int(batch.num_splits or 1), (size + 63) // 64, 64))
    ws = torch.empty(T * heads * ns * (dv + 2) if ns > 1 else 0, dtype=torch.float32, device=qkvg.device)
    _K().gated_attn_decode(qkvg, k_cache, v_cache, o, batch.block_table, batch.ctx_lens, batch.slots, ws, int(heads),
                           ns, int(size), float(scale), window, per_element, own_kv,
                           *(turn and (turn.rope, int(turn.dim), float(turn.eps)) or ()), **gains, **more)
    return o


def chunk_attention(qkvg, k_cache, v_cache, batch, heads: int, chunk: int, scale: float):
    """:func:`gated_attention` inside chunks, a gate per head."""
    return gated_attention(qkvg, k_cache, v_cache, batch, heads, chunk, scale)


# ------------------------------------------------------------------------------------------- normed residual, convolution
class Embedding(NamedTuple):
    """Residual source of a model's first norm: rows table[ids] * scale."""
    ids: torch.Tensor
    table: torch.Tensor
    scale: float = 1.0


class Affine(NamedTuple):
    """Gain and bias of a layer norm ((x - mean) / sqrt(variance + eps) gain + bias), where a gain alone means an RMS norm."""
    gain: Optional[torch.Tensor]
    bias: Optional[torch.Tensor]


PLAIN = Affine(None, None)   # no norm: the residual itself


def _gain_bias(w):
    return w if isinstance(w, Affine) else (w, None)


@dataclass
class Conv:
    """Causal convolution over time on each channel of a norm's output (or of the plain residual), added to it: weight
    [taps, D] (fp32, oldest tap first), state [slots, taps - 1, D] (fp32: the last inputs of every sequence).  ``tail``
    [B, taps - 1, D] receives a prefill step's last inputs (:func:`conv_commit` moves them into the state); None: a decode
    step, state updated here."""
    weight: torch.Tensor
    state: torch.Tensor
    tail: Optional[torch.Tensor] = None


def residual_norm(source, delta, wb, mult: float, step, w, eps: float, width: int, dtype, conv: Optional[Conv] = None,
                  batch=None, rows=None, keep: bool = True):
    """x = source (+ mult * norm(delta)) (+ step); h = norm(x), plus its convolution with ``conv``.

    source: the fp32 residual [T, D] or an :class:`Embedding`.  delta: [T, D], partial sums [parts, T, D] fp32, or
    :class:`Experts` without a dense part.  wb, w: the norms' gains (RMS norm) or :class:`Affine` (layer norm); wb PLAIN:
    delta is added as it is; w PLAIN: h = x.  Returns (x, h); the residual may be updated in place.  ``w`` None: no h.  ``rows`` (int32): h of these rows
    only, and with ``keep`` False x is None."""
    emb = isinstance(source, Embedding)
    if not (source.ids if emb else source).is_cuda:
        return ref.residual_norm(source, delta, wb, mult, step, w, eps, width, dtype, conv, batch, rows, keep)
    ids, table, scale = source if emb else (None, None, 1.0)
    T, D = (ids.shape[0], table.shape[1]) if emb else source.shape
    dev = ids.device if emb else source.device
    (wb, bb), no_h, (w, b) = _gain_bias(wb), w is None, _gain_bias(w)
    ye = {}
    if isinstance(delta, Experts):
        assert delta.dense is None
        ye = dict(ye=delta.y, slot_of=delta.slot_of, wts=delta.weights)
        delta = None
    x = None
    if keep:
        x = torch.empty(T, D, dtype=torch.float32, device=dev) if emb or conv is not None else source
    h = torch.empty(T if rows is None else rows.shape[0], D, dtype=dtype, device=dev) if not no_h else None
    ye.update(bb=bb, b=b)
    args = (None if emb else source, ids, table, float(scale), delta, wb, float(mult), step, x, rows, w, float(eps),
            int(width), h)
    if conv is None:
        _K().residual_norm(*args, **ye)
    elif conv.tail is None:
        _K().residual_norm(*args, conv.weight, conv.state, None, None, None, None, batch.positions, batch.state_slots,
                           **ye)
    else:
        _K().residual_norm(*args, conv.weight, conv.state, conv.tail, batch.row_seq, batch.q_start, batch.q_lens,
                           batch.positions, batch.state_slots, **ye)
    return x, h


def conv_commit(state, tail, batch) -> None:
    """The last convolution inputs of a prefill step (tail [runs, B, taps - 1, D]) into state [runs, slots, taps - 1, D]."""
    if not state.is_cuda:
        ref.conv_commit(state, tail, batch)
    else:
        _K().conv_commit(state, tail, batch.q_lens, batch.state_slots)


# ---------------------------------------------------------------------------------------------- rotary angles
class RopeScaling(NamedTuple):
    """Frequency scaling by wavelength: those up to original / high stay, those from original / low on are divided by
    ``factor``, and between the two the scaled and the unscaled frequency are blended."""
    factor: float
    low: float
    high: float
    original: float


def rope_freq(base: float, dims: int, scaling: Optional[RopeScaling] = None) -> torch.Tensor:
    """base^(-2 i / dims), i < dims / 2, scaled, as (float, remainder) pairs [dims / 2, 2]: angles of far positions keep
    their 32-bit accuracy."""
    f = np.power(float(base), -2.0 * np.arange(dims // 2) / dims)
    if scaling is not None:
        turns = scaling.original * f / (2.0 * np.pi)         # full turns within the original length
        s = np.clip((turns - scaling.low) / max(scaling.high - scaling.low, 1e-30), 0.0, 1.0)
        f = np.where(turns > scaling.high, f, np.where(turns < scaling.low, f / scaling.factor,
                                                       (1.0 - s) * f / scaling.factor + s * f))
    hi = f.astype(np.float32)
    return torch.tensor(np.stack([hi, (f - hi).astype(np.float32)], 1))


def rope_rows(positions, freq):
    """(cos, sin) of every row's angles, [T, dims] fp32; computed once per step for all layers that rotate alike."""
    if not positions.is_cuda:
        return ref.rope_rows(positions, freq)
    out = torch.empty(positions.shape[0], 2 * freq.shape[0], dtype=torch.float32, device=positions.device)
    _K().rope_rows(positions, freq, out)
    return out


# ---------------------------------------------------------------------------------------------- latent attention
def latent_head_pad(dk: int, dv: int) -> Optional[tuple]:
    """Head sizes of the prefill kernel that hold (dk, dv), or None."""
    for k, v in ((64, 64), (128, 64), (128, 128), (192, 128), (256, 256)):
        if dk <= k and dv <= v:
            return k, v
    return None


def latent_head_groups(heads: int) -> int:
    """Workgroups that share a row's heads in a decode step: 16 heads each, 32 from 17 heads on."""
    return 1 if heads <= 16 else -(-heads // 32)


@dataclass
class LatentGroup:
    """Sequences of a prefill step whose keys and values are expanded together (device int32 tensors, [n] each)."""
    seqs: torch.Tensor
    ctx: torch.Tensor
    q_lens: torch.Tensor
    q_start: torch.Tensor
    kv_start: torch.Tensor
    rows: int
    max_ctx: int
    max_q: int


@dataclass
class LatentPlan:
    """How a step's rows attend.  ``rows`` (None: all) attend one by one in latent space, as entries of block table row
    ``seqs`` (None: entry i is sequence i) with ``ctx`` keys; the sequences of ``groups`` run as portions."""
    n: int
    rows: Optional[torch.Tensor]
    seqs: Optional[torch.Tensor]
    ctx: torch.Tensor
    splits: int
    groups: List[LatentGroup]


def latent_plan(batch, expand: bool) -> LatentPlan:
    """``expand``: portions longer than LATENT_SHORT rows run on expanded keys and values."""
    if not batch.is_prefill:
        return LatentPlan(batch.input_ids.shape[0], None, None, batch.ctx_lens, max(1, int(batch.num_splits or 1)), [])
    dev = batch.input_ids.device
    to = lambda a: torch.from_numpy(np.ascontiguousarray(a, dtype=np.int32)).to(dev, non_blocking=True)
    q_lens, ctx = (np.asarray(a, dtype=np.int64) for a in (batch.q_lens_host, batch.ctx_lens_host))
    start = np.concatenate([[0], np.cumsum(q_lens)])[:-1]
    long = (q_lens > LATENT_SHORT) & expand
    groups, at = [], 0
    ids = np.nonzero(long)[0]
    while at < len(ids):
        n = max(1, int(np.searchsorted(np.cumsum(ctx[ids[at:]]), LATENT_GROUP_ROWS, side="right")))
        g = ids[at:at + n]
        at += n
        pack = to(np.stack([g, ctx[g], q_lens[g], start[g], np.cumsum(ctx[g]) - ctx[g]]))
        groups.append(LatentGroup(*pack.unbind(0), rows=int(ctx[g].sum()), max_ctx=int(ctx[g].max()),
                                  max_q=int(q_lens[g].max())))
    seq = np.repeat(np.arange(len(q_lens)), q_lens)
    pos = np.arange(len(seq)) - start[seq] + (ctx - q_lens)[seq]
    rows = np.nonzero(~long[seq])[0]
    pack = to(np.stack([rows, seq[rows], pos[rows] + 1]))
    splits = 1
    if len(rows):
        from . import decode_splits
        splits = decode_splits(len(rows), 1, int(pos[rows].max()) + 1)
    return LatentPlan(len(rows), pack[0] if groups else None, pack[1], pack[2], splits, groups)


def latent_prep(d, wq, wkv, rope, batch, cache, eps: float, q_rank: int, kv_rank: int):
    """The down projection's fp32 rows [q latent | kv latent | rotated key part] (each padded; or partial sums):
    norms both latents, turns the key part, writes [kv latent | key part] to ``cache`` [blocks, 64, ..] at batch.slots.  Returns the normed q latent
    in the cache's dtype."""
    if not d.is_cuda:
        return ref.latent_prep(d, wq, wkv, rope, batch, cache, eps, q_rank, kv_rank)
    cq = torch.empty(d.shape[-2], wq.shape[0], dtype=cache.dtype, device=d.device)
    _K().latent_prep(d, wq, wkv, rope, batch.slots, cache, cq, float(eps), int(q_rank), int(kv_rank))
    return cq


def latent_rows(ql, q, cache, block_table, plan: LatentPlan, sink, np_: int, rot: int, scale: float):
    """Softmax over the cached rows j < ctx of every entry, with exp(sink) in the denominator.  ql [n, H, rank]: queries
    in latent space; the rotated part of head h is q[:, h, np_ : np_ + rot] (q [n, H * head]).  -> [n, H, rank]."""
    if not q.is_cuda:
        return ref.latent_rows(ql, q, cache, block_table, plan, sink, np_, rot, scale)
    n, H, rp = ql.shape
    o = torch.empty_like(ql)
    ns = plan.splits
    ws = torch.empty(n * H * ns * (rp + 4) if ns > 1 else 0, dtype=torch.float32, device=q.device)
    _K().latent_attn_rows(ql, q, cache, o, block_table, plan.seqs, plan.ctx, sink, ws, ns, int(np_), int(rot), float(scale))
    return o


def latent_gather(cache, block_table, g: LatentGroup):
    """The cached rows of a group's sequences back to back, [g.rows, ..]."""
    if not cache.is_cuda:
        return ref.latent_gather(cache, block_table, g)
    out = torch.empty(g.rows, cache.shape[2], dtype=cache.dtype, device=cache.device)
    _K().latent_gather(cache, block_table, g.seqs, g.ctx, g.kv_start, g.max_ctx, out)
    return out


def latent_prefill(q, kv, lat, o, g: LatentGroup, sink, heads: int, np_: int, rot: int, rank: int, scale: float) -> None:
    """Causal attention of a group's portions: key j of head h is [kv[j, h, :np_] | lat[j, rank : rank + rot]], its value
    kv[j, h, np_:]; writes the portions' rows of ``o`` [T, H dv]."""
    if not q.is_cuda:
        ref.latent_prefill(q, kv, lat, o, g, sink, heads, np_, rot, rank, scale)
        return
    _K().latent_attn_prefill(q, kv, lat, o, g.ctx, g.q_lens, g.q_start, g.kv_start, sink, g.max_q, int(heads), int(np_),
                             int(rot), int(rank), float(scale))


# ---------------------------------------------------------------------------------------------- gated recurrence
def mingru_scan(zx, g, bias, state, batch):
    """S_t = (1 - z) S_(t-1) + z c per channel and sequence, z = sigmoid(zx[:, :W] + bias), c = u + 1/2 (u >= 0) or
    sigmoid(u), u = zx[:, W:] + bias; returns S silu(g).  ``state`` [slots, W] carries S (fp32); a sequence's first token
    starts from zero."""
    if not g.is_cuda:
        return ref.mingru_scan(zx, g, bias, state, batch)
    out = torch.empty_like(g)
    max_q = int(batch.S) if batch.is_prefill else 1
    least = SCAN_CHUNK if g.shape[0] > 4096 else SCAN_CHUNK // 2
    n = -(-max_q // (least * SCAN_MAX_CHUNKS)) * least
    chunks = -(-max_q // n)
    ws = torch.empty(batch.B * chunks * 2 * g.shape[1] if chunks > 1 else 0, dtype=torch.float32, device=g.device)
    _K().mingru_scan(zx, g, bias, state, out, batch.positions, batch.q_start, batch.q_lens, batch.state_slots, ws, max_q, n)
    return out


# ---------------------------------------------------------------------------------------------- matrix state
def hgrn2(qv, z, bias, lower, gain, state, batch, vdim: int, eps: float):
    """Linear attention whose forget gate also decides what is written: per head, with f = lower + (1 - lower)
    sigmoid(z + bias), S = diag(f) S + (1 - f) v^T and o = S^T silu(q); returns o / rms(o over vdim) gain, [T, H dv].

    qv [T, H dk + H dv]: queries and values; z [T, H dk] fp32 forget logits; bias, lower [H dk] (pads: lower 1); gain [dv].
    ``state`` [slots, H, dk, dv] carries S (fp32); a sequence's first token starts from zero."""
    if not qv.is_cuda:
        return ref.hgrn2(qv, z, bias, lower, gain, state, batch, vdim, eps)
    T, (_, H, dk, dv) = qv.shape[0], state.shape
    out = torch.empty(T, H * dv, dtype=qv.dtype, device=qv.device)
    max_q, n, unit = (int(batch.S) if batch.is_prefill else 1), STATE_SEGMENT, H * dk * (dv + 1)
    segments = 1
    if max_q > n and qv.dtype == torch.bfloat16:
        # enough workgroups for the chip where few long sequences would not give them, in at most 256 MB of totals
        want = min(-(-512 // (H * max(1, T // max_q))), STATE_MAX_SEGMENTS, max(1, (1 << 26) // (batch.B * unit)))
        n = max(n, -(-max_q // (32 * want)) * 32)
        segments = -(-max_q // n)
    else:
        n = -(-max_q // 32) * 32
    ws = torch.empty(batch.B * segments * unit if segments > 1 else 0, dtype=torch.float32, device=qv.device)
    _K().hgrn2(qv, z, bias, lower, gain, state, out, batch.positions, batch.q_start, batch.q_lens, batch.state_slots, ws,
               max_q, n, int(vdim), float(eps))
    return out


# ---------------------------------------------------------------------------------------------- delta rule, retention
GATE_SILU, GATE_SIGMOID = 0, 1


@dataclass
class RuleShape:
    """Sizes of a matrix-state mixer: ``dim`` / ``vdim`` before padding, ``kv_heads`` heads of queries and keys for the
    state's heads, and what its output gate is passed through."""
    kv_heads: int
    dim: int
    vdim: int
    gate: int = GATE_SILU


def rule_segment(rows: int, scans: int, retention: bool) -> int:
    """Rows of the segments that sequences of up to ``rows`` rows are cut into, 0: not cut.  ``scans``: sequences times heads,
    a workgroup each when uncut.  A first scan over the segments takes one workgroup each for retention and two for the delta
    rule; both scans together must be shorter than one over the whole sequence."""
    chunks, per = -(-rows // RULE_CHUNK), 1 if retention else 2
    n = min((256 // scans + 2 * per - 1) // per, chunks // 4)
    return -(-chunks // n) * RULE_CHUNK if n >= 3 else 0


def _rule_run(x, gate, state, out, batch, shape: RuleShape, eps: float, commit, **args):
    """The launches of one step: decode and fp32 rows one by one; bf16 portions in chunks, as many heads at a time as the
    workspace holds."""
    T, (_, H, dk, dv) = x.shape[0], state.shape
    args = dict(pos=batch.positions, slots=batch.state_slots, kv_heads=int(shape.kv_heads), dim=int(shape.dim),
                vdim=int(shape.vdim), gate_kind=int(shape.gate), eps=float(eps), **args)
    if not batch.is_prefill:
        _K().rule_rows(x, gate, state, out, **args)
        return
    args.update(q_start=batch.q_start, q_lens=batch.q_lens)
    if x.dtype == torch.float32:
        _K().rule_rows(x, gate, state, out, **args)
    else:
        # whole groups of heads with common queries and keys; rounds of equal size
        groups, per_channel = int(shape.kv_heads), "decay" in args and args["decay"].shape[1] != H
        size = H // groups
        need = lambda n: (T // RULE_CHUNK + batch.B) * _K().rule_chunk_bytes(dk, dv, n * size, n * (size if per_channel else 1), per_channel)
        rounds = -(-groups // max(1, min(groups, RULE_WORKSPACE // need(1))))
        n = -(-groups // rounds)
        ws = torch.empty(need(n), dtype=torch.uint8, device=x.device)
        seg = rule_segment(int(batch.S), -(-T // int(batch.S)) * n * size, "decay" not in args)
        seg_ws = torch.empty((T // seg + batch.B) * _K().rule_segment_bytes(dk, dv, n * size, "decay" not in args),
                             dtype=torch.uint8, device=x.device) if seg else None
        for g in range(0, groups, n):
            _K().rule_chunks(x, gate, state, out, ws=ws, max_q=int(batch.S), head0=g * size, heads=min(n, groups - g) * size,
                             seg=seg, seg_ws=seg_ws, **args)
    if commit is not None:
        _K().ring_commit(x, commit, batch.positions, batch.q_start, batch.q_lens, batch.state_slots)


def delta_rule(x, gate, decay, beta, conv, rate, bias, gain, state, ring, batch, out, shape: RuleShape, eps: float) -> None:
    """Linear attention whose matrix state S [dk, dv] per head is written by the delta rule: S = diag(g) S,
    u = sigmoid(beta) (v - S^T k), S = S + k u^T, o = S^T q; out = o / rms(o over vdim) gain act(gate).

    x [T, G dk + G dk + H dv] holds the projected queries, keys and values.  Each of their channels passes a causal
    convolution over time (``conv`` [taps, channels], oldest tap first) and silu; queries and keys are then made unit vectors
    (queries also times dim^-1/2), head h using those of head h / (H / G).  g = exp(-rate softplus(decay + bias)) with
    ``decay`` fp32 [T, H] (bias [H]: one decay per head) or [T, H dk] (bias [H dk]: one per key channel); rate [H]; beta
    logits fp32 [T, H]; gate [T, H dv]; gain [dv] (zero in the pads).  ``state`` [slots, H, dk, dv] (fp32) and ``ring``
    [slots, taps, channels] (the last inputs, each at its position modulo taps) carry a sequence; its first token starts from
    zero.  x, gate, decay, beta and out may be views with any row stride."""
    if not x.is_cuda:
        ref.delta_rule(x, gate, decay, beta, conv, rate, bias, gain, state, ring, batch, out, shape, eps)
        return
    _rule_run(x, gate, state, out, batch, shape, eps, ring, decay=decay, beta=beta, conv=conv, rate=rate, bias=bias, gain=gain,
              ring=ring)


def decay_rates(decay) -> torch.Tensor:
    """Decays in [0, 1] and their base-2 logarithms, [2, H] fp32 (2^-40 leaves nothing of a state)."""
    d = np.asarray(decay, dtype=np.float64)
    return torch.tensor(np.stack([d, np.log2(np.maximum(d, 2.0 ** -40))]), dtype=torch.float32)


def retention(x, gate, decay, rope, state, batch, out, shape: RuleShape, eps: float) -> None:
    """Linear attention with a fixed decay per head: S = decay S + k v^T, o = S^T q; out = o / rms(o over vdim) act(gate).

    x [T, H (2 dk + dv)]: projected queries, keys and values; dimension i < rot / 2 of queries and keys is turned with
    i + rot / 2 by the row's angles ``rope`` [T, rot], keys are then multiplied by dim^-1/2.  ``decay`` [2, H] fp32: the decays
    and their base-2 logarithms.  ``state`` [slots, H, dk, dv] as in :func:`delta_rule`."""
    if not x.is_cuda:
        ref.retention(x, gate, decay, rope, state, batch, out, shape, eps)
        return
    _rule_run(x, gate, state, out, batch, shape, eps, None, rate=decay, rope=rope)
