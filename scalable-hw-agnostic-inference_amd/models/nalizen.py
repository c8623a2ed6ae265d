"""Nalizen: a decoder described layer by layer in config.json -- sliding-window attention with normed queries and keys (whose
keys and values a later layer may share) or HGRN2 linear attention as the mixer, a token shift on every mixer's input, layer
norms on the sublayers' outputs only, dense gated or mixture-of-experts feed-forward blocks, a token input of its own for
every layer, and an output projection tied to the embedding.

The model runs on the engine like the Llama family: :class:`shai_amd.engines.llm.LLMEngine` owns blocks, state slots,
scheduling and sampling.  An attention layer has its own K/V pools or reads those of the layer it shares with; an HGRN2 layer
has a matrix state per head and sequence slot; every layer keeps its last mixer input per slot (token shift).  The residual
stream is fp32; one launch adds a sublayer's normed output (and sums expert outputs or partial products) and hands the next
sublayer its input, shifted where a mixer comes next.  A layer of a decode step is 10 launches with a dense feed-forward and
12 with experts (one more with split attention; routing takes two above 16 rows).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Union

import torch
import torch.nn as nn

from .blocks import (AffineNorm, GeluGLU, Hgrn2, Hgrn2Config, MoE, MoEConfig, ReLU2Config, StepShared, TokenShift, TokenSide,
                     WindowAttention, WindowAttentionConfig, _padded, _param, check_checkpoint)
from .llama import KV_BLOCK, Batch
from ..ops import lm
from ..parallel.state import tp


@dataclass
class GeluGLUConfig:
    ff: int


@dataclass
class NalizenLayerConfig:
    mixer: Union[WindowAttentionConfig, Hgrn2Config]
    mlp: Union[GeluGLUConfig, MoEConfig, None] = None


@dataclass
class NalizenConfig:
    vocab_size: int
    width: int
    layers: List[NalizenLayerConfig]
    side_dim: int
    eps: float = 1e-6
    embed_scale: float = 1.0
    max_position_embeddings: int = 1 << 20               # angles are computed: bounded by the cache only
    bos_token_id: int = 0
    eos_token_id: Optional[int] = None

    def __post_init__(self):
        if not self.layers or self.side_dim < 1:
            raise ValueError("a Nalizen model needs at least one layer and a token input")
        for i, lc in enumerate(self.layers):
            c = lc.mixer
            j = getattr(c, "kv_from", None)
            if j is None:
                continue
            src = self.layers[j].mixer if 0 <= j < i else None
            if not isinstance(src, WindowAttentionConfig) or src.kv_from is not None:
                raise ValueError(f"layer {i}: keys and values come from an earlier attention layer with its own, not {j}")
            same = lambda m: (m.heads, m.kv_heads, m.dim, m.vdim, m.rot_base, m.rot_dims, m.rot_scaling)
            if same(src) != same(c):
                raise ValueError(f"layers {j} and {i} share keys: their heads and rotation must be equal")

    @staticmethod
    def from_json(d: dict) -> "NalizenConfig":
        def mixer(kind, m):
            if kind == "hgrn2":
                return Hgrn2Config(int(m["heads"]), int(m["dim"]), int(m["vdim"]))
            if kind != "attention":
                raise ValueError(f"unknown mixer type {kind!r}")
            rot, src = m["rot"], m.get("kv_from")
            sc = rot.get("scaling")
            return WindowAttentionConfig(
                int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), float(m["scale"]), int(m["mask"]["size"]),
                int(rot["dims"]), float(rot["base"]),
                lm.RopeScaling(*(float(sc[k]) for k in ("factor", "low", "high", "original"))) if sc else None,
                int(src) if src is not None else None)

        def mlp(m):
            if m is None:
                return None
            if m["kind"] == "dense":
                return GeluGLUConfig(int(m["ff"]))
            if m["kind"] != "moe":
                raise ValueError(f"unknown feed-forward kind {m['kind']!r}")
            return MoEConfig(int(m["router"]["experts"]), int(m["router"]["top"]), ReLU2Config(int(m["expert"]["ff"])),
                             bias=True, renorm=True)

        eos = d.get("eos_token_id")
        return NalizenConfig(
            vocab_size=int(d["vocab"]), width=int(d["width"]),
            layers=[NalizenLayerConfig(mixer(x["type"], x["mixer"]), mlp(x.get("mlp"))) for x in d["layers"]],
            side_dim=int(d["token_side"]["dim"]), eps=float(d["norm"]["eps"]), embed_scale=float(d["embedding"]["scale"]),
            bos_token_id=int(d.get("bos_token_id") or 0), eos_token_id=int(eos) if eos is not None else None)

    @staticmethod
    def uniform(layers: str, width: int, heads: int, kv_heads: int, dim: int, window: int, state_heads: int, state_dim: int,
                state_vdim: int, ff: int, experts: int, top: int, expert_ff: int, side_dim: int, vocab: int) -> "NalizenConfig":
        """Layers of equal sizes (benchmarks, tests).  ``layers``: a letter each, A attention, S attention that shares the
        keys and values of the A before it, R HGRN2; upper case with experts, lower case with a dense feed-forward."""
        out: List[NalizenLayerConfig] = []
        moe = MoEConfig(experts, top, ReLU2Config(expert_ff), bias=True, renorm=True)
        src = None
        for i, kind in enumerate(layers):
            if kind.upper() == "R":
                mix = Hgrn2Config(state_heads, state_dim, state_vdim)
            else:
                src = i if kind.upper() == "A" else src
                mix = WindowAttentionConfig(heads, kv_heads, dim, dim, dim ** -0.5, window, dim // 2, 10000.0,
                                            lm.RopeScaling(8.0, 1.0, 4.0, 8192.0), src if kind.upper() == "S" else None)
            out.append(NalizenLayerConfig(mix, moe if kind.isupper() else GeluGLUConfig(ff)))
        return NalizenConfig(vocab, width, out, side_dim)

    @staticmethod
    def tiny() -> "NalizenConfig":
        return NalizenConfig.uniform("aRSr", width=128, heads=4, kv_heads=2, dim=32, window=40, state_heads=2, state_dim=24,
                                     state_vdim=40, ff=192, experts=6, top=2, expert_ff=48, side_dim=24, vocab=512)


class NalizenLayer(nn.Module):
    def __init__(self, cfg: NalizenConfig, c: NalizenLayerConfig, dtype):
        super().__init__()
        D = cfg.width
        self.shift = TokenShift(D)
        self.mix = (Hgrn2 if isinstance(c.mixer, Hgrn2Config) else WindowAttention)(D, c.mixer, cfg.eps, dtype)
        self.norm1 = AffineNorm(D)
        self.mlp = self.norm2 = None
        if c.mlp is not None:
            self.mlp = GeluGLU(D, c.mlp.ff, dtype) if isinstance(c.mlp, GeluGLUConfig) else MoE(D, c.mlp, dtype)
            self.norm2 = AffineNorm(D)
        self.side = TokenSide(D, cfg.side_dim, dtype)

    def blocks(self):
        """(prefix of the checkpoint names, block) of everything with tensors but the shift."""
        return [(p, b) for p, b in (("norm1", self.norm1), ("norm2", self.norm2), ("mix.", self.mix), ("mlp.", self.mlp),
                                    ("side.", self.side)) if b is not None]


class NalizenForCausalLM(nn.Module):
    needs_prev_token = False
    has_state = True             # sequences hold a state slot (allocate_state); their prefixes cannot be shared by blocks
    dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, cfg: NalizenConfig, dtype=torch.bfloat16):
        super().__init__()
        if tp().size > 1:
            raise ValueError("Nalizen runs on one GPU per replica (tensor parallel size 1)")
        self.cfg, self.dtype = cfg, dtype
        self.embed = _param(cfg.vocab_size, lm.pad64(cfg.width), dtype=dtype)
        self.side_embed = _param(cfg.vocab_size, len(cfg.layers) * lm.pad64(cfg.side_dim), dtype=dtype)
        self.layers = nn.ModuleList([NalizenLayer(cfg, c, dtype) for c in cfg.layers])
        self.final_norm = AffineNorm(cfg.width)

    def init_random_(self, gen):
        self.embed[:, :self.cfg.width].normal_(0, self.cfg.width ** -0.5, generator=gen)
        self.side_embed.view(self.cfg.vocab_size, len(self.layers), -1)[..., :self.cfg.side_dim].normal_(0, 1.0, generator=gen)

    # ---- engine interface
    def fold_norms(self):
        """The norm gains stay apart: with an fp32 residual the norm is its own (fused) launch."""

    def _attention(self):
        return [layer.mix for layer in self.layers if isinstance(layer.mix, WindowAttention)]

    @property
    def kv_heads_local(self) -> int:
        return max((m.c.kv_heads for m in self._attention()), default=1)

    @property
    def attn_span(self) -> int:
        """The most keys a position of any layer sees."""
        return max((m.c.window for m in self._attention()), default=1)

    def cache_bytes_per_block(self) -> int:
        size = torch.finfo(self.dtype).bits // 8
        shapes = [layer.mix.cache_shapes(1, KV_BLOCK) for layer in self.layers]
        return max(1, sum(size * torch.Size(s).numel() for pair in shapes if pair is not None for s in pair))

    def allocate_cache(self, blocks: int, device):
        """(buffers to keep alive, [(k, v) of every layer, shared ones included, or None without attention])."""
        kv = []
        for layer in self.layers:
            shapes, src = layer.mix.cache_shapes(blocks, KV_BLOCK), getattr(layer.mix.c, "kv_from", None)
            kv.append(kv[src] if src is not None else shapes and tuple(torch.zeros(s, dtype=self.dtype, device=device)
                                                                       for s in shapes))
        return kv, kv

    def allocate_state(self, slots: int, device):
        """(last mixer inputs [layers, slots, 1, width], [recurrent state or None] of every layer), fp32.  A sequence's first
        token ignores what its slot holds, so slots need no clearing."""
        shapes = [layer.mix.state_shape for layer in self.layers]
        shift = torch.zeros(len(shapes), slots, 1, lm.pad64(self.cfg.width), device=device)
        return shift, [None if s is None else torch.zeros(slots, *s, device=device) for s in shapes]

    def forward(self, batch: Batch, kv_caches, trail: Optional[list] = None) -> torch.Tensor:
        """fp32 logits [rows, vocab]: every row of a decode step, the rows ``batch.last_index`` of a prefill step.
        ``trail`` (a list) receives the residual stream after every layer."""
        cfg, (shift_state, states) = self.cfg, batch.states
        norm = lambda source, delta, wb, w, **kw: lm.residual_norm(source, delta, wb, 1.0, None, w, cfg.eps, cfg.width,
                                                                   self.dtype, batch=batch, **kw)
        step, n = StepShared(batch), lm.pad64(cfg.side_dim)
        tail = None
        if batch.is_prefill:
            tail = torch.empty(len(self.layers), batch.B, 1, shift_state.shape[3], device=shift_state.device)
        x, delta, wb = lm.Embedding(batch.input_ids, self.embed, cfg.embed_scale), None, None
        for i, layer in enumerate(self.layers):
            conv = lm.Conv(layer.shift.weight, shift_state[i], tail[i] if tail is not None else None)
            x, h = norm(x, delta, wb, lm.PLAIN, conv=conv)
            y = layer.mix(h, batch, kv_caches[i] if kv_caches[i] is not None else states[i], step)
            x, h = norm(x, y, layer.norm1.affine, lm.PLAIN)
            if layer.mlp is not None:
                x, h = norm(x, layer.mlp(h), layer.norm2.affine, lm.PLAIN)
            delta, wb = layer.side(h, batch.input_ids, self.side_embed[:, i * n:(i + 1) * n]), layer.side.norm
            if trail is not None:
                trail.append(norm(x.clone(), delta, wb, None)[0][:, :cfg.width])
        if tail is not None:
            lm.conv_commit(shift_state, tail, batch)
        rows = batch.last_index.int() if batch.is_prefill else None
        h = norm(x, delta, wb, self.final_norm.affine, rows=rows, keep=False)[1]
        return lm.matmul(h, self.embed, torch.float32)

    # ---- checkpoint
    def checkpoint_shapes(self) -> Dict[str, tuple]:
        """Every tensor of a checkpoint and its shape."""
        c = self.cfg
        s = {"embed": (c.vocab_size, c.width), "side.embed": (c.vocab_size, len(c.layers) * c.side_dim)}
        s.update({"final.norm" + k: v for k, v in self.final_norm.shapes().items()})
        for i, layer in enumerate(self.layers):
            s[f"l{i}.shift"] = (c.width,)
            for prefix, block in layer.blocks():
                s.update({f"l{i}.{prefix}{k}": v for k, v in block.shapes().items()})
        return s

    def convert_hf_state_dict(self, sd: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
        """Checkpoint tensors -> packed parameters; a missing, unknown or misshapen tensor is an error."""
        check_checkpoint(sd, self.checkpoint_shapes())
        c, L = self.cfg, len(self.layers)
        side = _padded(sd["side.embed"].reshape(c.vocab_size, L, c.side_dim), c.vocab_size, L, lm.pad64(c.side_dim))
        out = {"embed": _padded(sd["embed"], *self.embed.shape), "side_embed": side.reshape(c.vocab_size, -1)}
        pack = lambda name, prefix, block: out.update(
            {f"{name}.{k}": v for k, v in block.pack(lambda key: sd[prefix + key]).items()})
        pack("final_norm", "final.norm", self.final_norm)
        for i, layer in enumerate(self.layers):
            out[f"layers.{i}.shift.weight"] = layer.shift.pack(sd[f"l{i}.shift"])
            for prefix, block in layer.blocks():
                pack(f"layers.{i}.{prefix.rstrip('.')}", f"l{i}.{prefix}", block)
        return out
