"""Building blocks of decoders that are described layer by layer in their config (fp32 residual stream).

Each block keeps its weights in the layout of :mod:`shai_amd.ops.lm` (width padded to 64, head sizes to kernel sizes,
gate / up rows interleaved, experts stacked) and packs them from checkpoint tensors in ``pack``: ``pack(get)`` maps the
block's own tensor names (``get("q")``) to its parameters, so a model only supplies the prefix.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Callable, Dict, Optional, Union

import torch
import torch.nn as nn

from ..ops import lm


def _param(*shape, dtype):
    return nn.Parameter(torch.zeros(*shape, dtype=dtype), requires_grad=False)


def _padded(t: torch.Tensor, *shape) -> torch.Tensor:
    """``t`` in the leading corner of a zero tensor of ``shape``."""
    if tuple(t.shape) == tuple(shape):
        return t
    out = t.new_zeros(shape)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


def _head_rows(t: torch.Tensor, heads: int, dim: int, pad: int, width: int) -> torch.Tensor:
    """[heads * dim, D] -> [heads * pad, width], every head's rows padded by zero rows."""
    return _padded(t.reshape(heads, dim, t.shape[1]), heads, pad, width).reshape(heads * pad, width)


def _head_columns(t: torch.Tensor, heads: int, dim: int, pad: int, width: int) -> torch.Tensor:
    """[D, heads * dim] -> [width, heads * pad], every head's columns padded by zero columns."""
    return _padded(t.reshape(t.shape[0], heads, dim), width, heads, pad).reshape(width, heads * pad)


def check_checkpoint(sd: Dict[str, torch.Tensor], want: Dict[str, tuple]) -> None:
    """A missing, unknown or misshapen tensor is an error."""
    bad = ([k for k in want if k not in sd] + [k for k in sd if k not in want]
           + [k for k in want if k in sd and tuple(sd[k].shape) != want[k]])
    if bad:
        raise ValueError(f"checkpoint does not fit config.json: {len(bad)} tensors missing, unknown or misshapen, "
                         f"e.g. {bad[:5]}")


class OffsetNorm(nn.Module):
    """RMSNorm whose stored weight is the gain minus one (applied by ``ops.lm.add_norm`` / ``embed_norm``)."""

    def __init__(self, width: int, eps: float):
        super().__init__()
        self.width, self.eps = width, eps
        self.weight = _param(lm.pad64(width), dtype=torch.float32)

    def pack(self, t: torch.Tensor) -> torch.Tensor:
        return _padded(t, lm.pad64(self.width))

    def init_random_(self, gen):
        self.weight.zero_()


class BigramEmbedding(nn.Module):
    """Token embedding plus a hashed embedding of (previous token, token): row (prev * mul_prev + cur * mul_cur) mod
    buckets; a sequence's first token takes the extra last row."""

    def __init__(self, vocab: int, width: int, buckets: Optional[int] = None, mul_prev: int = 0, mul_cur: int = 0,
                 dtype=torch.bfloat16):
        super().__init__()
        self.width, self.buckets, self.mul_prev, self.mul_cur = width, buckets, mul_prev, mul_cur
        self.weight = _param(vocab, lm.pad64(width), dtype=dtype)
        self.bigram = _param(buckets + 1, lm.pad64(width), dtype=dtype) if buckets else None

    def forward(self, ids, prev, norm: OffsetNorm):
        return lm.embed_norm(ids, prev, self.weight, self.bigram, self.mul_prev, self.mul_cur, norm.weight, norm.eps,
                             self.width)

    def init_random_(self, gen):
        for p in (self.weight, self.bigram):
            if p is not None:
                p[:, :self.width].normal_(0, 1.0, generator=gen)


@dataclass
class ChunkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int

    def __post_init__(self):
        if self.heads % self.kv_heads or self.chunk < 1:
            raise ValueError(f"bad attention sizes: {self}")


class ChunkAttention(nn.Module):
    """Attention without positions inside fixed-size chunks of the sequence, a sigmoid gate per head on its output.
    q, k, v and the gate logits come from one GEMM."""

    def __init__(self, width: int, c: ChunkAttentionConfig, dtype=torch.bfloat16):
        super().__init__()
        self.c, self.width = c, width
        self.dk, self.dv = lm.head_pad(c.dim, c.vdim)
        n = c.heads * self.dk + c.kv_heads * (self.dk + self.dv) + c.heads
        self.qkvg = _param((n + 7) // 8 * 8, lm.pad64(width), dtype=dtype)
        self.o = _param(lm.pad64(width), c.heads * self.dv, dtype=dtype)

    def shapes(self) -> Dict[str, tuple]:
        c, D = self.c, self.width
        return {"q": (c.heads * c.dim, D), "k": (c.kv_heads * c.dim, D), "v": (c.kv_heads * c.vdim, D),
                "g": (c.heads, D), "o": (D, c.heads * c.vdim)}

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        c, (n, W) = self.c, self.qkvg.shape
        rows = torch.cat([_head_rows(get("q"), c.heads, c.dim, self.dk, W),
                          _head_rows(get("k"), c.kv_heads, c.dim, self.dk, W),
                          _head_rows(get("v"), c.kv_heads, c.vdim, self.dv, W), _padded(get("g"), c.heads, W)])
        o = get("o").reshape(self.width, c.heads, c.vdim)
        return {"qkvg": _padded(rows, n, W), "o": _padded(o, W, c.heads, self.dv).reshape(W, c.heads * self.dv)}

    def forward(self, h, batch, k_cache, v_cache):
        o = lm.chunk_attention(lm.matmul(h, self.qkvg), k_cache, v_cache, batch, self.c.heads, self.c.chunk,
                               self.c.scale)
        return lm.matmul(o, self.o)

    def cache_shapes(self, blocks: int, block: int):
        g = self.c.kv_heads
        return (blocks, g, block, self.dk), (blocks, g, block, self.dv)

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


@dataclass
class ClampedGLUConfig:
    ff: int
    limit: float


@dataclass
class ReLU2Config:
    """Feed-forward without a gate: down max(up h, 0)^2."""
    ff: int


@dataclass
class MoEConfig:
    experts: int
    top: int
    expert: Union[ClampedGLUConfig, ReLU2Config]
    groups: int = 1
    keep: int = 1
    shared: Optional[ClampedGLUConfig] = None
    bias: bool = False       # the router's logits have one
    renorm: bool = False     # weights are a softmax over the chosen logits only

    def __post_init__(self):
        if (self.experts % self.groups or not 1 <= self.keep <= self.groups
                or not 1 <= self.top <= self.keep * (self.experts // self.groups)
                or self.experts > lm.MAX_EXPERTS or self.top > lm.MAX_TOP):
            raise ValueError(f"bad router sizes: {self}")


def _interleave(gate: torch.Tensor, up: torch.Tensor, ff: int, width: int) -> torch.Tensor:
    """(gate_i, up_i) row pairs, [2 ff, width]."""
    return torch.stack([_padded(gate, ff, width), _padded(up, ff, width)], 1).reshape(2 * ff, width)


class MoE(nn.Module):
    """Softmax-scored experts chosen inside the best expert groups, clamped-GLU or squared-ReLU experts, and an optional
    shared expert.  Returns :class:`ops.lm.Experts` for the next residual add to combine."""

    def __init__(self, width: int, c: MoEConfig, dtype=torch.bfloat16):
        super().__init__()
        self.c, self.width = c, width
        W, F = lm.pad64(width), lm.pad64(c.expert.ff)
        # the shared expert's gate / up rows and the router's rows: one product
        S = lm.pad64(c.shared.ff) if c.shared is not None else 0
        self.front = _param(2 * S + c.experts, W, dtype=dtype)
        self.gated = isinstance(c.expert, ClampedGLUConfig)
        if self.gated:
            self.gate_up = _param(c.experts, 2 * F, W, dtype=dtype)
        else:
            self.up = _param(c.experts, F, W, dtype=dtype)
        self.down = _param(c.experts, W, F, dtype=dtype)
        self.bias = _param(c.experts, dtype=torch.float32) if c.bias else None
        if c.shared is not None:
            self.shared_down = _param(W, S, dtype=dtype)

    def shapes(self) -> Dict[str, tuple]:
        c, D = self.c, self.width
        s = {"router": (c.experts, D)}
        if c.bias:
            s["router.b"] = (c.experts,)
        named = [(f"e{i}", c.expert) for i in range(c.experts)] + ([("shared", c.shared)] if c.shared else [])
        for name, e in named:
            s.update({f"{name}.up": (e.ff, D), f"{name}.down": (D, e.ff)})
            if isinstance(e, ClampedGLUConfig):
                s[f"{name}.gate"] = (e.ff, D)
        return s

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        c, W, F = self.c, self.front.shape[1], self.down.shape[2]
        each = lambda fn: torch.stack([fn(f"e{i}.") for i in range(c.experts)])
        out = {"front": _padded(get("router"), c.experts, W),
               **({"gate_up": each(lambda e: _interleave(get(e + "gate"), get(e + "up"), F, W))} if self.gated
                  else {"up": each(lambda e: _padded(get(e + "up"), F, W))}),
               "down": torch.stack([_padded(get(f"e{i}.down"), W, F) for i in range(c.experts)])}
        if c.bias:
            out["bias"] = get("router.b")
        if c.shared is not None:
            S = self.shared_down.shape[1]
            out["front"] = torch.cat([_interleave(get("shared.gate"), get("shared.up"), S, W), out["front"]])
            out["shared_down"] = _padded(get("shared.down"), W, S)
        return out

    def forward(self, h) -> lm.Experts:
        c = self.c
        if c.shared is not None:
            s, z = lm.glu_with_side(h, self.front, c.experts, c.shared.limit)
        else:
            z = lm.matmul(h, self.front, torch.float32)
        wts, plan = lm.route_experts(z, c.top, c.groups, c.keep, self.bias, c.renorm)
        if self.gated:
            a = lm.matmul(h, self.gate_up, epi=lm.EPI_CLAMP_GLU, param=c.expert.limit, plan=plan, gather=True)
        else:
            a = lm.matmul(h, self.up, epi=lm.EPI_RELU2, plan=plan, gather=True)
        y = lm.matmul(a, self.down, plan=plan)
        dense = lm.matmul(s, self.shared_down) if c.shared is not None else None
        return lm.Experts(y, plan.slot_of, wts, dense)

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


class SoftcapHead(nn.Module):
    """fp32 logits = cap * tanh(h W^T / cap); no cap: h W^T."""

    def __init__(self, vocab: int, width: int, cap: Optional[float], dtype=torch.bfloat16):
        super().__init__()
        self.cap, self.width = cap, width
        self.weight = _param(vocab, lm.pad64(width), dtype=dtype)

    def forward(self, h):
        return lm.matmul(h, self.weight, torch.float32, lm.EPI_SOFTCAP if self.cap else lm.EPI_NONE, self.cap or 0.0)

    def init_random_(self, gen):
        self.weight[:, :self.width].normal_(0, self.width ** -0.5, generator=gen)


class GainNorm(nn.Module):
    """RMSNorm gains as stored (applied by ``ops.lm.residual_norm``)."""

    def __init__(self, width: int):
        super().__init__()
        self.width = width
        self.weight = _param(lm.pad64(width), dtype=torch.float32)

    def pack(self, t: torch.Tensor) -> torch.Tensor:
        return _padded(t, lm.pad64(self.width))

    def init_random_(self, gen):
        self.weight[:self.width] = 1.0


class InputConv(nn.Module):
    """Causal convolution over time on each channel of a sublayer's normed input, added to it."""

    def __init__(self, width: int, taps: int):
        super().__init__()
        if not 1 <= taps <= lm.MAX_TAPS:
            raise ValueError(f"input convolutions of 1 to {lm.MAX_TAPS} taps are supported, got {taps}")
        self.width, self.taps = width, taps
        self.weight = _param(taps, lm.pad64(width), dtype=torch.float32)

    def pack(self, t: torch.Tensor) -> torch.Tensor:
        return _padded(t.T, self.taps, lm.pad64(self.width))

    def init_random_(self, gen):
        self.weight[:, :self.width].normal_(0, self.taps ** -0.5, generator=gen)


@dataclass
class LatentAttentionConfig:
    heads: int
    dim: int            # unrotated query / key size of a head
    rot_dim: int        # rotated size
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float = 10000.0

    def __post_init__(self):
        if min(self.heads, self.dim, self.vdim, self.q_rank, self.kv_rank) < 1 or self.rot_dim < 2 or self.rot_dim % 2:
            raise ValueError(f"bad attention sizes: {self}")
        if self.kv_rank > lm.MAX_LATENT:
            raise ValueError(f"latents of up to {lm.MAX_LATENT} values are supported, got {self.kv_rank}")


class LatentAttention(nn.Module):
    """Attention whose cache is one latent row and one rotated key part per token, shared by all heads; queries go through
    a latent of their own; a learned sink per head in the denominator.

    Decode steps and short portions attend in latent space: the queries go through W_uk, the attended latent through
    W_uv (one small product per head each), and keys and values are never built.  Longer portions expand them per head
    from the cached latents and run the flash kernel."""

    def __init__(self, width: int, c: LatentAttentionConfig, eps: float, dtype=torch.bfloat16):
        super().__init__()
        self.c, self.width, self.eps, self.dtype = c, width, eps, dtype
        pad8 = lambda n: (n + 7) // 8 * 8
        self.np, self.kn = pad8(c.dim), lm.pad64(c.dim)          # unrotated part in a head's row; as a product's depth
        self.qp, self.op = lm.pad64(c.q_rank), lm.pad64(c.rot_dim)
        self.rp = next((r for r in (64, 128, 256, 512) if c.kv_rank <= r), lm.pad64(c.kv_rank))
        fit = lm.latent_head_pad(self.np + pad8(c.rot_dim), c.vdim)
        self.dk, self.dv = fit or (lm.pad64(self.np + pad8(c.rot_dim)), lm.pad64(c.vdim))
        self.expands = fit is not None and dtype == torch.bfloat16
        H, W = c.heads, lm.pad64(width)
        self.down = _param(self.qp + self.rp + self.op, W, dtype=dtype)
        self.q_norm = _param(self.qp, dtype=torch.float32)
        self.kv_norm = _param(self.rp, dtype=torch.float32)
        self.uq = _param(H * self.dk, self.qp, dtype=dtype)
        self.uk = _param(H, self.rp, self.kn, dtype=dtype)       # queries into latent space
        self.ukv = _param(H, self.np + self.dv, self.rp, dtype=dtype)
        self.sink = _param(H, dtype=torch.float32)
        self.o = _param(W, H * self.dv, dtype=dtype)
        self.register_buffer("freq", lm.rope_freq(c.rot_base, c.rot_dim).to(self.o.device), persistent=False)

    def shapes(self) -> Dict[str, tuple]:
        c, D = self.c, self.width
        return {"dq": (c.q_rank, D), "dq.norm": (c.q_rank,), "uq": (c.heads * (c.dim + c.rot_dim), c.q_rank),
                "dkv": (c.kv_rank + c.rot_dim, D), "dkv.norm": (c.kv_rank,), "uk": (c.heads * c.dim, c.kv_rank),
                "uv": (c.heads * c.vdim, c.kv_rank), "sink": (c.heads,), "o": (D, c.heads * c.vdim)}

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        c, W, H = self.c, self.down.shape[1], self.c.heads
        dkv = get("dkv")
        q = get("uq").reshape(H, c.dim + c.rot_dim, c.q_rank)
        uk, uv = get("uk").reshape(H, c.dim, c.kv_rank), get("uv").reshape(H, c.vdim, c.kv_rank)
        o = get("o").reshape(self.width, H, c.vdim)
        return {"down": torch.cat([_padded(get("dq"), self.qp, W), _padded(dkv[:c.kv_rank], self.rp, W),
                                   _padded(dkv[c.kv_rank:], self.op, W)]),
                "q_norm": _padded(get("dq.norm"), self.qp), "kv_norm": _padded(get("dkv.norm"), self.rp),
                "uq": torch.cat([_padded(q[:, :c.dim], H, self.np, self.qp),
                                 _padded(q[:, c.dim:], H, self.dk - self.np, self.qp)], 1).reshape(H * self.dk, self.qp),
                "uk": _padded(uk.transpose(1, 2), H, self.rp, self.kn),
                "ukv": torch.cat([_padded(uk, H, self.np, self.rp), _padded(uv, H, self.dv, self.rp)], 1),
                "sink": get("sink"), "o": _padded(o, W, H, self.dv).reshape(W, H * self.dv)}

    def forward(self, h, batch, cache, step):
        """``step``: the step's shared work (:class:`StepShared`)."""
        c = self.c
        rope, plan = step.rope(self), step.plan(self.expands)
        down = lm.matmul_parts(h, self.down, torch.float32)
        cq = lm.latent_prep(down, self.q_norm, self.kv_norm, rope, batch, cache, self.eps, c.q_rank, c.kv_rank)
        q = lm.matmul(cq, self.uq, epi=lm.EPI_ROTARY, rope=rope, head=self.dk, rot0=self.np)
        return lm.matmul_parts(self.attend(q, batch, cache, plan), self.o)

    def attend(self, q, batch, cache, plan):
        """q [T, H dk], turned, over the cached latents (this step's included) -> [T, H dv]."""
        c, H = self.c, self.c.heads
        if not plan.groups:
            return self._in_latent_space(q, batch, cache, plan)
        o = torch.empty(q.shape[0], H * self.dv, dtype=q.dtype, device=q.device)
        for g in plan.groups:
            lat = lm.latent_gather(cache, batch.block_table, g)
            kv = lm.matmul(lat[:, :self.rp], self.ukv.view(-1, self.rp))
            lm.latent_prefill(q, kv, lat, o, g, self.sink, H, self.np, c.rot_dim, self.rp, c.scale)
        if plan.n:
            rows = plan.rows
            o.index_copy_(0, rows.long(), self._in_latent_space(q.index_select(0, rows), batch, cache, plan))
        return o

    def _in_latent_space(self, q, batch, cache, plan):
        c, n = self.c, q.shape[0]
        ql = lm.matmul_heads(q.view(n, c.heads, self.dk)[..., :self.kn], self.uk)
        ol = lm.latent_rows(ql, q, cache, batch.block_table, plan, self.sink, self.np, c.rot_dim, c.scale)
        return lm.matmul_heads(ol, self.ukv[:, self.np:]).view(n, c.heads * self.dv)

    def cache_shape(self, blocks: int, block: int):
        return blocks, block, self.rp + self.op

    @property
    def rope_key(self):
        return self.c.rot_base, self.c.rot_dim, None

    state_width = None

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


class StepShared:
    """What the layers of one step share: rotation angles per (base, dims) and the attention plan per kind."""

    def __init__(self, batch):
        self.batch, self._ropes, self._plans = batch, {}, {}

    def rope(self, mix):
        """Angles for a mixer with ``rope_key`` (what its frequencies follow from) and ``freq``."""
        key = mix.rope_key
        if key not in self._ropes:
            self._ropes[key] = lm.rope_rows(self.batch.positions, mix.freq)
        return self._ropes[key]

    def plan(self, expands: bool):
        if expands not in self._plans:
            self._plans[expands] = lm.latent_plan(self.batch, expands)
        return self._plans[expands]


class MinGRU(nn.Module):
    """Gated recurrence whose gates read the current token only; output gated by silu and projected.  One product gives
    the output gate (weights' dtype) and the recurrence's inputs (fp32)."""

    def __init__(self, width: int, size: int, dtype=torch.bfloat16):
        super().__init__()
        if size < 1:
            raise ValueError(f"bad recurrence width {size}")
        self.width, self.size = width, size
        self.sp = lm.pad64(size)
        self.gzx = _param(3 * self.sp, lm.pad64(width), dtype=dtype)
        self.bias = _param(2 * self.sp, dtype=torch.float32)
        self.o = _param(lm.pad64(width), self.sp, dtype=dtype)

    @property
    def state_width(self) -> int:
        return self.sp

    def shapes(self) -> Dict[str, tuple]:
        n, D = self.size, self.width
        return {"z": (n, D), "z.b": (n,), "x": (n, D), "x.b": (n,), "g": (n, D), "o": (D, n)}

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        W = self.gzx.shape[1]
        return {"gzx": torch.cat([_padded(get(n), self.sp, W) for n in ("g", "z", "x")]),
                "bias": torch.cat([_padded(get(n), self.sp) for n in ("z.b", "x.b")]),
                "o": _padded(get("o"), W, self.sp)}

    def forward(self, h, batch, state, step=None):
        g, zx = lm.matmul_with_side(h, self.gzx, 2 * self.sp)
        return lm.matmul_parts(lm.mingru_scan(zx, g, self.bias, state, batch), self.o)

    def cache_shape(self, blocks: int, block: int):
        return None

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


class XieluMLP(nn.Module):
    """Dense feed-forward with the xIELU activation; its two learned numbers enter as softplus(p), 1/2 + softplus(q)."""

    def __init__(self, width: int, ff: int, dtype=torch.bfloat16):
        super().__init__()
        self.width, self.ff = width, ff
        self.up = _param(lm.pad64(ff), lm.pad64(width), dtype=dtype)
        self.down = _param(lm.pad64(width), lm.pad64(ff), dtype=dtype)
        self.act = _param(2, dtype=torch.float32)

    def shapes(self) -> Dict[str, tuple]:
        return {"up": (self.ff, self.width), "down": (self.width, self.ff), "act": (2,)}

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        act = torch.nn.functional.softplus(get("act").double())
        return {"up": _padded(get("up"), *self.up.shape), "down": _padded(get("down"), *self.down.shape),
                "act": (act + torch.tensor([0.0, 0.5], dtype=act.dtype, device=act.device)).float()}

    def forward(self, h):
        return lm.matmul_parts(lm.matmul(h, self.up, epi=lm.EPI_XIELU, vec=self.act), self.down)

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


class AffineNorm(nn.Module):
    """Layer norm with gain and bias (applied by ``ops.lm.residual_norm``)."""

    def __init__(self, width: int):
        super().__init__()
        self.width = width
        self.weight = _param(lm.pad64(width), dtype=torch.float32)
        self.bias = _param(lm.pad64(width), dtype=torch.float32)

    @property
    def affine(self) -> lm.Affine:
        return lm.Affine(self.weight, self.bias)

    def shapes(self) -> Dict[str, tuple]:
        return {"": (self.width,), ".b": (self.width,)}

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        return {"weight": _padded(get(""), lm.pad64(self.width)), "bias": _padded(get(".b"), lm.pad64(self.width))}

    def init_random_(self, gen):
        self.weight[:self.width] = 1.0


class TokenShift(InputConv):
    """A mixer's input moved towards the previous token's, channel by channel: h + (h' - h) s, i.e. a convolution of two
    taps (s, -s) added to h."""

    def __init__(self, width: int):
        super().__init__(width, 2)

    def pack(self, t: torch.Tensor) -> torch.Tensor:
        return super().pack(torch.stack([t.float(), -t.float()], 1))

    def init_random_(self, gen):
        s = torch.rand(self.width, generator=gen, device=gen.device)
        self.weight[0, :self.width], self.weight[1, :self.width] = s, -s


@dataclass
class WindowAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int                                  # a position sees itself and the window - 1 before it
    rot_dims: int                                # rotated dimensions of a head
    rot_base: float = 10000.0
    rot_scaling: Optional[lm.RopeScaling] = None
    kv_from: Optional[int] = None                # layer whose keys and values are used

    def __post_init__(self):
        if (self.heads % self.kv_heads or self.window < 1 or self.rot_dims % 2 or not 0 < self.rot_dims <= self.dim
                or min(self.dim, self.vdim) < 1):
            raise ValueError(f"bad attention sizes: {self}")


class WindowAttention(nn.Module):
    """Sliding-window attention with rotated (half against half) and rms-normed queries and keys and a sigmoid gate per
    output element.  q, k, v and the gate logits come from one GEMM; with ``kv_from`` only q and the gate, and the keys and
    values are those in another layer's cache."""

    state_shape = None

    def __init__(self, width: int, c: WindowAttentionConfig, eps: float, dtype=torch.bfloat16):
        super().__init__()
        self.c, self.width, self.eps = c, width, eps
        self.dk, self.dv = lm.head_pad(c.dim, c.vdim)
        kv = c.kv_heads * (self.dk + self.dv) if c.kv_from is None else 0
        self.qkvg = _param(c.heads * (self.dk + self.dv) + kv, lm.pad64(width), dtype=dtype)
        self.o = _param(lm.pad64(width), c.heads * self.dv, dtype=dtype)
        self.register_buffer("freq", lm.rope_freq(c.rot_base, c.rot_dims, c.rot_scaling).to(self.o.device),
                             persistent=False)

    @property
    def rope_key(self):
        return self.c.rot_base, self.c.rot_dims, self.c.rot_scaling

    def shapes(self) -> Dict[str, tuple]:
        c, D = self.c, self.width
        s = {"q": (c.heads * c.dim, D), "g": (c.heads * c.vdim, D), "o": (D, c.heads * c.vdim)}
        if c.kv_from is None:
            s.update({"k": (c.kv_heads * c.dim, D), "v": (c.kv_heads * c.vdim, D)})
        return s

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        c, W = self.c, self.qkvg.shape[1]
        rows = [_head_rows(get("q"), c.heads, c.dim, self.dk, W)]
        if c.kv_from is None:
            rows += [_head_rows(get("k"), c.kv_heads, c.dim, self.dk, W),
                     _head_rows(get("v"), c.kv_heads, c.vdim, self.dv, W)]
        rows.append(_head_rows(get("g"), c.heads, c.vdim, self.dv, W))
        return {"qkvg": torch.cat(rows), "o": _head_columns(get("o"), c.heads, c.vdim, self.dv, W)}

    def forward(self, h, batch, cache, step):
        c = self.c
        o = lm.gated_attention(lm.matmul(h, self.qkvg), *cache, batch, c.heads, c.window, c.scale, window=True,
                               per_element=True, own_kv=c.kv_from is None,
                               turn=lm.HeadTurn(step.rope(self), c.dim, self.eps))
        return lm.matmul_parts(o, self.o)

    def cache_shapes(self, blocks: int, block: int):
        if self.c.kv_from is not None:
            return None
        g = self.c.kv_heads
        return (blocks, g, block, self.dk), (blocks, g, block, self.dv)

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


@dataclass
class Hgrn2Config:
    heads: int
    dim: int
    vdim: int

    def __post_init__(self):
        if min(self.heads, self.dim, self.vdim) < 1:
            raise ValueError(f"bad recurrence sizes: {self}")


class Hgrn2(nn.Module):
    """Linear attention with a matrix state per head whose forget gate (bounded below) also decides what is written; every
    head's output is rms-normed.  One product gives queries and values (weights' dtype) and forget logits (fp32)."""

    def __init__(self, width: int, c: Hgrn2Config, eps: float, dtype=torch.bfloat16):
        super().__init__()
        self.c, self.width, self.eps = c, width, eps
        self.dk, self.dv = lm.head_pad(c.dim, c.vdim)
        H, W = c.heads, lm.pad64(width)
        self.qvf = _param(H * (2 * self.dk + self.dv), W, dtype=dtype)
        self.bias = _param(H * self.dk, dtype=torch.float32)
        self.lower = _param(H * self.dk, dtype=torch.float32)
        self.gain = _param(self.dv, dtype=torch.float32)
        self.o = _param(W, H * self.dv, dtype=dtype)

    @property
    def state_shape(self) -> tuple:
        return self.c.heads, self.dk, self.dv

    def shapes(self) -> Dict[str, tuple]:
        c, D = self.c, self.width
        n, m = c.heads * c.dim, c.heads * c.vdim
        return {"q": (n, D), "f": (n, D), "f.b": (n,), "lower": (n,), "v": (m, D), "norm": (c.vdim,), "o": (D, m)}

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        c, H, W = self.c, self.c.heads, self.qvf.shape[1]
        rows = lambda name, dim, pad: _head_rows(get(name), H, dim, pad, W)
        lower = get("lower").reshape(H, c.dim)
        pads = torch.cat([lower, lower.new_ones(H, self.dk - c.dim)], 1)      # a pad channel keeps its (zero) state
        return {"qvf": torch.cat([rows("q", c.dim, self.dk), rows("v", c.vdim, self.dv), rows("f", c.dim, self.dk)]),
                "bias": _padded(get("f.b").reshape(H, c.dim), H, self.dk).reshape(-1), "lower": pads.reshape(-1),
                "gain": _padded(get("norm"), self.dv), "o": _head_columns(get("o"), H, c.vdim, self.dv, W)}

    def forward(self, h, batch, state, step=None):
        qv, z = lm.matmul_with_side(h, self.qvf, self.c.heads * self.dk)
        o = lm.hgrn2(qv, z, self.bias, self.lower, self.gain, state, batch, self.c.vdim, self.eps)
        return lm.matmul_parts(o, self.o)

    def cache_shapes(self, blocks: int, block: int):
        return None

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


class GeluGLU(nn.Module):
    """Dense feed-forward down (gelu_tanh(gate h) up h)."""

    def __init__(self, width: int, ff: int, dtype=torch.bfloat16):
        super().__init__()
        self.width, self.ff = width, ff
        self.gate_up = _param(2 * lm.pad64(ff), lm.pad64(width), dtype=dtype)
        self.down = _param(lm.pad64(width), lm.pad64(ff), dtype=dtype)

    def shapes(self) -> Dict[str, tuple]:
        return {"gate": (self.ff, self.width), "up": (self.ff, self.width), "down": (self.width, self.ff)}

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        W, F = self.down.shape
        return {"gate_up": _interleave(get("gate"), get("up"), F, W), "down": _padded(get("down"), W, F)}

    def forward(self, h):
        return lm.matmul_parts(lm.matmul(h, self.gate_up, epi=lm.EPI_GELU_GLU), self.down)

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


class TokenSide(nn.Module):
    """Per-layer token input: proj (gelu_tanh(gate x) * the token's row of a table), rms-normed by the residual add."""

    def __init__(self, width: int, dim: int, dtype=torch.bfloat16):
        super().__init__()
        self.width, self.dim = width, dim
        n, W = lm.pad64(dim), lm.pad64(width)
        self.gate = _param(n, W, dtype=dtype)
        self.proj = _param(W, n, dtype=dtype)
        self.norm = _param(W, dtype=torch.float32)

    def shapes(self) -> Dict[str, tuple]:
        return {"gate": (self.dim, self.width), "proj": (self.width, self.dim), "norm": (self.width,)}

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        return {"gate": _padded(get("gate"), *self.gate.shape), "proj": _padded(get("proj"), *self.proj.shape),
                "norm": _padded(get("norm"), *self.norm.shape)}

    def forward(self, h, ids, table):
        g = lm.matmul(h, self.gate, epi=lm.EPI_GELU_ROWS, ids=ids, table=table)
        return lm.matmul_parts(g, self.proj)

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


# ---------------------------------------------------------------------------------------------- joint layers
class JointLayer(nn.Module):
    """Sublayers that read one norm's output and whose sum is added to the residual: one or more mixers and an ungated
    squared-ReLU feed-forward (``ff`` 0: none).  One product gives every mixer's inputs and the activated feed-forward, one
    product over the mixers' outputs and the feed-forward sums them all in fp32.

    A mixer supplies the rows of its input projections (``in_rows``, with an fp32 part of ``side_rows``) and the columns of its
    output projection (``out_cols``), reads its inputs from the step's rows and writes its output beside the others'."""

    def __init__(self, width: int, mixers, ff: int, dtype=torch.bfloat16):
        super().__init__()
        self.width, self.ff, self.fp = width, ff, lm.pad64(ff)
        self.mixers = nn.ModuleDict(mixers)              # name in the checkpoint ("only": none) -> mixer
        self.out_cols = sum(m.out_cols for m in self.mixers.values())
        self.in_rows = sum(m.in_rows for m in self.mixers.values())
        self.side_rows = sum(m.side_rows for m in self.mixers.values())
        W = lm.pad64(width)
        self.w_in = _param(self.fp + self.in_rows + self.side_rows, W, dtype=dtype)
        self.w_out = _param(W, self.out_cols + self.fp, dtype=dtype)

    def shapes(self) -> Dict[str, tuple]:
        s = {f"mix.{self._dot(n)}{k}": v for n, m in self.mixers.items() for k, v in m.shapes().items()}
        if self.ff:
            s.update({"mlp.up": (self.ff, self.width), "mlp.down": (self.width, self.ff)})
        return s

    @staticmethod
    def _dot(name: str) -> str:
        return "" if name == "only" else name + "."

    def _gets(self, get):
        return [(m, lambda k, p=f"mix.{self._dot(n)}": get(p + k)) for n, m in self.mixers.items()]

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        """This layer's own parameters (a mixer packs the rest of its tensors)."""
        W, gets = self.w_in.shape[1], self._gets(get)
        rows = ([_padded(get("mlp.up"), self.fp, W)] if self.ff else []) + [m.pack_in(g) for m, g in gets]
        rows += [m.pack_side(g) for m, g in gets if m.side_rows]
        cols = [m.pack_out(g) for m, g in gets] + ([_padded(get("mlp.down"), W, self.fp)] if self.ff else [])
        return {"w_in": torch.cat(rows), "w_out": torch.cat(cols, 1)}

    def pack_all(self, get) -> Dict[str, torch.Tensor]:
        out = self.pack(get)
        for (n, m), (_, g) in zip(self.mixers.items(), self._gets(get)):
            out.update({f"mixers.{n}.{k}": v for k, v in m.pack(g).items()})
        return out

    def forward(self, h, batch, cache, state, step):
        """``cache`` / ``state``: what the mixers that have a key-value cache / a recurrent state keep of this layer run."""
        n = self.out_cols + self.fp
        rows = torch.empty(h.shape[0], n + self.in_rows, dtype=h.dtype, device=h.device)
        side = lm.matmul_joint(h, self.w_in, rows[:, self.out_cols:], self.fp, self.side_rows)
        i, s, o = n, 0, 0
        for m in self.mixers.values():
            m(rows[:, i:i + m.in_rows], side[:, s:s + m.side_rows] if m.side_rows else None, rows[:, o:o + m.out_cols], batch,
              cache if m.cached else state, step)
            i, s, o = i + m.in_rows, s + m.side_rows, o + m.out_cols
        return lm.matmul_parts(rows[:, :n], self.w_out)

    def cache_shapes(self, blocks: int, block: int):
        return next((m.cache_shapes(blocks, block) for m in self.mixers.values() if m.cached), None)

    def state_shapes(self):
        """[(shape per slot, whether it is fp32 in a bf16 model too)] of the recurrent mixer, or None."""
        return next((m.state_shapes() for m in self.mixers.values() if not m.cached), None)

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


@dataclass
class TiedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int                                     # of queries, keys and values
    scale: float
    rot_dims: int
    rot_base: float = 10000.0
    out_scale: float = 1.0                       # factor on the mixer's output

    def __post_init__(self):
        if (min(self.heads, self.kv_heads, self.dim) < 1 or self.heads % self.kv_heads or self.rot_dims % 2
                or not 0 < self.rot_dims <= self.dim):
            raise ValueError(f"bad attention sizes: {self}")


class TiedAttention(nn.Module):
    """Causal attention whose values are the projected keys: queries and keys rms-normed per head with a gain and then rotated
    (half against half), a factor per head on the scores, a learned sink per head in the denominator."""

    cached, side_rows = True, 0

    def __init__(self, width: int, c: TiedAttentionConfig, eps: float):
        super().__init__()
        self.c, self.width, self.eps = c, width, eps
        self.dk, _ = lm.head_pad(c.dim, c.dim)
        self.in_rows, self.out_cols = (c.heads + c.kv_heads) * self.dk, c.heads * self.dk
        f32 = lambda n: _param(n, dtype=torch.float32)
        self.q_gain, self.k_gain, self.temp, self.sink = f32(self.dk), f32(self.dk), f32(c.heads), f32(c.heads)
        self.register_buffer("freq", lm.rope_freq(c.rot_base, c.rot_dims).to(self.sink.device), persistent=False)

    @property
    def rope_key(self):
        return self.c.rot_base, self.c.rot_dims, None

    def shapes(self) -> Dict[str, tuple]:
        c, D = self.c, self.width
        return {"q": (c.heads * c.dim, D), "k": (c.kv_heads * c.dim, D), "q.norm": (c.dim,), "k.norm": (c.dim,),
                "temp": (c.heads,), "sink": (c.heads,), "o": (D, c.heads * c.dim)}

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        return {"q_gain": _padded(get("q.norm"), self.dk), "k_gain": _padded(get("k.norm"), self.dk), "temp": get("temp"),
                "sink": get("sink")}

    def pack_in(self, get):
        c, W = self.c, lm.pad64(self.width)
        return torch.cat([_head_rows(get("q"), c.heads, c.dim, self.dk, W), _head_rows(get("k"), c.kv_heads, c.dim, self.dk, W)])

    def pack_out(self, get):
        return _head_columns(get("o"), self.c.heads, self.c.dim, self.dk, lm.pad64(self.width))

    def forward(self, x, side, out, batch, cache, step):
        c = self.c
        lm.gated_attention(x, *cache, batch, c.heads, lm.WHOLE, c.scale, window=True,
                           turn=lm.HeadTurn(step.rope(self), c.dim, self.eps, self.q_gain, self.k_gain),
                           plain=lm.Ungated(self.temp, self.sink, out, c.out_scale))

    def cache_shapes(self, blocks: int, block: int):
        return ((blocks, self.c.kv_heads, block, self.dk),) * 2

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


@dataclass
class DeltaRuleConfig:
    heads: int
    kv_heads: int                                # heads of queries and keys
    dim: int
    vdim: int
    taps: int
    ranks: Optional[tuple] = None                # of the thin products for (decay, output gate); None: whole products,
                                                 # and one decay per head instead of one per key channel
    gate: int = lm.GATE_SILU
    out_scale: float = 1.0

    def __post_init__(self):
        if min(self.heads, self.kv_heads, self.dim, self.vdim, *(self.ranks or ())) < 1 or self.heads % self.kv_heads:
            raise ValueError(f"bad delta rule sizes: {self}")
        if not 1 <= self.taps <= lm.MAX_TAPS:
            raise ValueError(f"short convolutions of 1 to {lm.MAX_TAPS} taps are supported, got {self.taps}")


class DeltaRule(nn.Module):
    """Linear attention whose matrix state per head is decayed (per head, or per key channel) and written by the delta rule;
    queries, keys and values pass a short convolution and silu, queries and keys are unit vectors, every head's output is
    rms-normed and gated.  Decay and write strength logits leave their products in fp32."""

    cached = False

    def __init__(self, width: int, c: DeltaRuleConfig, eps: float, dtype=torch.bfloat16):
        super().__init__()
        self.c, self.width, self.eps, self.dtype = c, width, eps, dtype
        H, G = c.heads, c.kv_heads
        self.dk, self.dv = lm.head_pad(c.dim, c.vdim)
        self.channels = 2 * G * self.dk + H * self.dv
        self.low = [lm.pad64(r) for r in c.ranks] if c.ranks else None
        self.in_rows = self.channels + (sum(self.low) if self.low else H * self.dv)
        self.side_rows = H if self.low else 2 * H
        self.out_cols = H * self.dv
        f32 = lambda *n: _param(*n, dtype=torch.float32)
        self.conv = f32(c.taps, self.channels)
        self.rate, self.bias, self.gain = f32(H), f32(H * (self.dk if self.low else 1)), f32(self.dv)
        if self.low:   # both thin products' second halves as one: [gate | decay] from [decay part | gate part]
            self.up = _param(H * (self.dv + self.dk), sum(self.low), dtype=dtype)
        self.shape = lm.RuleShape(G, c.dim, c.vdim, c.gate)

    def shapes(self) -> Dict[str, tuple]:
        c, D, H = self.c, self.width, self.c.heads
        kv, n, m = c.kv_heads * c.dim, H * c.dim, H * c.vdim
        s = {"b": (H, D), "A_log": (H,), "norm": (c.vdim,), "o": (D, m), "dt_bias": (n if c.ranks else H,)}
        for name, rows in (("q", kv), ("k", kv), ("v", m)):
            s.update({name: (rows, D), name + ".conv": (rows, c.taps)})
        if c.ranks:
            a, g = c.ranks
            s.update({"a1": (a, D), "a2": (n, a), "g1": (g, D), "g2": (m, g)})
        else:
            s.update({"a": (H, D), "g": (m, D)})
        return s

    def _spread(self, get, suffix: str, width: int) -> torch.Tensor:
        """Rows of queries, keys and values, every head padded."""
        c = self.c
        return torch.cat([_head_rows(get(n + suffix), heads, d, pad, width)
                          for n, heads, d, pad in (("q", c.kv_heads, c.dim, self.dk), ("k", c.kv_heads, c.dim, self.dk),
                                                   ("v", c.heads, c.vdim, self.dv))])

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        c, H = self.c, self.c.heads
        out = {"conv": self._spread(get, ".conv", c.taps).T, "rate": get("A_log").double().exp().float(),
               "gain": _padded(get("norm").float() * c.out_scale, self.dv), "bias": get("dt_bias")}
        if self.low:
            a, g = self.low
            out["bias"] = _padded(get("dt_bias").reshape(H, c.dim), H, self.dk).reshape(-1)
            gate = _head_rows(get("g2"), H, c.vdim, self.dv, g)
            decay = _head_rows(get("a2"), H, c.dim, self.dk, a)
            out["up"] = torch.cat([torch.cat([gate.new_zeros(len(gate), a), gate], 1),
                                   torch.cat([decay, decay.new_zeros(len(decay), g)], 1)])
        return out

    def pack_in(self, get):
        W = lm.pad64(self.width)
        last = ([_padded(get(n), r, W) for n, r in zip(("a1", "g1"), self.low)] if self.low
                else [_head_rows(get("g"), self.c.heads, self.c.vdim, self.dv, W)])
        return torch.cat([self._spread(get, "", W)] + last)

    def pack_side(self, get):
        return _padded(torch.cat([get(n) for n in (("b",) if self.low else ("b", "a"))]), self.side_rows, lm.pad64(self.width))

    def pack_out(self, get):
        return _head_columns(get("o"), self.c.heads, self.c.vdim, self.dv, lm.pad64(self.width))

    def forward(self, x, side, out, batch, state, step):
        H, n = self.c.heads, self.channels
        gate, decay = x[:, n:], side[:, H:]
        if self.low:
            gate, decay = lm.matmul_with_side(gate, self.up, H * self.dk)
        lm.delta_rule(x[:, :n], gate, decay, side[:, :H], self.conv, self.rate, self.bias, self.gain, *state, batch, out,
                      self.shape, self.eps)

    def state_shapes(self):
        return [((self.c.heads, self.dk, self.dv), True), ((self.c.taps, self.channels), False)]

    def init_random_(self, gen):
        _init_packed(self, self.pack, self.shapes(), gen)


@dataclass
class RetentionConfig:
    decay: tuple                                 # of every head
    dim: int
    vdim: int
    rot_dims: int
    rot_base: float = 10000.0

    def __post_init__(self):
        if (not self.decay or min(self.dim, self.vdim) < 1 or self.rot_dims % 2 or not 0 < self.rot_dims <= self.dim
                or not all(0.0 <= d <= 1.0 for d in self.decay)):
            raise ValueError(f"bad retention sizes: {self}")


class Retention(nn.Module):
    """Linear attention with a matrix state and a fixed decay per head, rotated queries and keys, every head's output
    rms-normed and gated by silu."""

    cached, side_rows = False, 0

    def __init__(self, width: int, c: RetentionConfig, eps: float):
        super().__init__()
        self.c, self.width, self.eps = c, width, eps
        self.H = H = len(c.decay)
        self.dk, self.dv = lm.head_pad(c.dim, c.vdim)
        self.in_rows, self.out_cols = H * (2 * self.dk + 2 * self.dv), H * self.dv
        self.shape = lm.RuleShape(H, c.dim, c.vdim, lm.GATE_SILU)
        self.register_buffer("freq", lm.rope_freq(c.rot_base, c.rot_dims), persistent=False)
        self.register_buffer("decay", lm.decay_rates(c.decay), persistent=False)

    @property
    def rope_key(self):
        return self.c.rot_base, self.c.rot_dims, None

    def shapes(self) -> Dict[str, tuple]:
        c, D, n, m = self.c, self.width, self.H * self.c.dim, self.H * self.c.vdim
        return {"q": (n, D), "k": (n, D), "v": (m, D), "g": (m, D), "o": (D, m)}

    def pack(self, get) -> Dict[str, torch.Tensor]:
        return {}

    def pack_in(self, get):
        c, W = self.c, lm.pad64(self.width)
        return torch.cat([_head_rows(get(n), self.H, d, pad, W) for n, d, pad in (
            ("q", c.dim, self.dk), ("k", c.dim, self.dk), ("v", c.vdim, self.dv), ("g", c.vdim, self.dv))])

    def pack_out(self, get):
        return _head_columns(get("o"), self.H, self.c.vdim, self.dv, lm.pad64(self.width))

    def forward(self, x, side, out, batch, state, step):
        n = self.H * (2 * self.dk + self.dv)
        lm.retention(x[:, :n], x[:, n:], self.decay, step.rope(self), state[0], batch, out, self.shape, self.eps)

    def state_shapes(self):
        return [((self.H, self.dk, self.dv), True)]


def _init_packed(module: nn.Module, pack, shapes: Dict[str, tuple], gen) -> None:
    """Fill a block from random full-size tensors of its checkpoint shapes: matrices N(0, 1 / fan_in), gains 1, other
    vectors 0."""
    dev, dtype = gen.device, next(module.parameters()).dtype

    def draw(name):
        if len(shapes[name]) == 1:
            return torch.full(shapes[name], float(name.endswith(("norm", "temp"))), device=dev)
        return (torch.randn(shapes[name], generator=gen, device=dev) / math.sqrt(shapes[name][1])).to(dtype)
    for k, v in pack(draw).items():
        module.get_parameter(k).copy_(v)
