"""Building blocks of decoders that are described layer by layer in their config (fp32 residual stream).

Each block keeps its weights in the layout of :mod:`shai_amd.ops.lm` (width padded to 64, head sizes to 64 / 128 / 256,
gate / up rows interleaved, experts stacked) and packs them from checkpoint tensors in ``pack``: ``pack(get)`` maps the
block's own tensor names (``get("q")``) to its parameters, so a model only supplies the prefix.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Callable, Dict, Optional

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
class MoEConfig:
    experts: int
    top: int
    expert: ClampedGLUConfig
    groups: int = 1
    keep: int = 1
    shared: Optional[ClampedGLUConfig] = None

    def __post_init__(self):
        if (self.experts % self.groups or not 1 <= self.keep <= self.groups
                or not 1 <= self.top <= self.keep * (self.experts // self.groups)
                or self.experts > lm.MAX_EXPERTS or self.top > lm.MAX_TOP):
            raise ValueError(f"bad router sizes: {self}")


def _interleave(gate: torch.Tensor, up: torch.Tensor, ff: int, width: int) -> torch.Tensor:
    """(gate_i, up_i) row pairs, [2 ff, width]."""
    return torch.stack([_padded(gate, ff, width), _padded(up, ff, width)], 1).reshape(2 * ff, width)


class MoE(nn.Module):
    """Softmax-scored experts chosen inside the best expert groups (scores not renormalised), clamped-GLU experts, and
    an optional shared expert.  Returns :class:`ops.lm.Experts` for the next residual add to combine."""

    def __init__(self, width: int, c: MoEConfig, dtype=torch.bfloat16):
        super().__init__()
        self.c, self.width = c, width
        W, F = lm.pad64(width), lm.pad64(c.expert.ff)
        # the shared expert's gate / up rows and the router's rows: one product
        S = lm.pad64(c.shared.ff) if c.shared is not None else 0
        self.front = _param(2 * S + c.experts, W, dtype=dtype)
        self.gate_up = _param(c.experts, 2 * F, W, dtype=dtype)
        self.down = _param(c.experts, W, F, dtype=dtype)
        if c.shared is not None:
            self.shared_down = _param(W, S, dtype=dtype)

    def shapes(self) -> Dict[str, tuple]:
        c, D = self.c, self.width
        s = {"router": (c.experts, D)}
        named = [(f"e{i}", c.expert) for i in range(c.experts)] + ([("shared", c.shared)] if c.shared else [])
        for name, e in named:
            s.update({f"{name}.gate": (e.ff, D), f"{name}.up": (e.ff, D), f"{name}.down": (D, e.ff)})
        return s

    def pack(self, get: Callable[[str], torch.Tensor]) -> Dict[str, torch.Tensor]:
        c, W, F = self.c, self.front.shape[1], self.down.shape[2]
        out = {"front": _padded(get("router"), c.experts, W),
               "gate_up": torch.stack([_interleave(get(f"e{i}.gate"), get(f"e{i}.up"), F, W)
                                       for i in range(c.experts)]),
               "down": torch.stack([_padded(get(f"e{i}.down"), W, F) for i in range(c.experts)])}
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
        wts, plan = lm.route_experts(z, c.top, c.groups, c.keep)
        a = lm.matmul(h, self.gate_up, epi=lm.EPI_CLAMP_GLU, param=c.expert.limit, plan=plan, gather=True)
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


def _init_packed(module: nn.Module, pack, shapes: Dict[str, tuple], gen) -> None:
    """Fill a block from random full-size tensors of its checkpoint shapes (N(0, 1 / fan_in))."""
    dev, dtype = gen.device, next(module.parameters()).dtype
    draw = lambda name: (torch.randn(shapes[name], generator=gen, device=dev) / math.sqrt(shapes[name][1])).to(dtype)
    for k, v in pack(draw).items():
        getattr(module, k).copy_(v)
