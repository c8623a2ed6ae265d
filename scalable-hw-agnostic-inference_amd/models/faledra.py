"""Faledra: a decoder described layer by layer in config.json -- latent attention with a sink per head or a minGRU as the
mixer, a short causal convolution on every mixer's input, norms before and after each sublayer, dense xIELU feed-forward
blocks, and a run of layers that is passed several times with the same weights.

The model runs on the engine like the Llama family: :class:`shai_amd.engines.llm.LLMEngine` owns blocks, state slots,
scheduling and sampling.  Every layer RUN (a looped layer counts once per pass) has its own cache or state: a paged pool
of latents (one row per token, all heads), or a recurrent state per sequence slot, and the convolution's last inputs per
slot.  The residual stream is fp32; one launch adds a sublayer's normed output, norms the sum and applies the next
convolution.  An attention layer of a decode step is 11 launches (12 with split attention), a minGRU layer 7.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple, Union

import torch
import torch.nn as nn

from .blocks import (GainNorm, InputConv, LatentAttention, LatentAttentionConfig, MinGRU, SoftcapHead, StepShared,
                     XieluMLP, _padded, _param, check_checkpoint)
from .llama import KV_BLOCK, Batch
from ..ops import lm
from ..parallel.state import tp


@dataclass
class MinGRUConfig:
    width: int


@dataclass
class FaledraLayerConfig:
    mixer: Union[LatentAttentionConfig, MinGRUConfig]
    ff: Optional[int] = None


@dataclass
class FaledraConfig:
    vocab_size: int
    width: int
    layers: List[FaledraLayerConfig]
    taps: int
    eps: float = 1e-5
    embed_scale: float = 1.0
    residual_mult: float = 1.0
    loop: Optional[Tuple[int, int, int]] = None          # (start, stop, times)
    max_position_embeddings: int = 1 << 20               # angles are computed: bounded by the cache only
    bos_token_id: int = 0
    eos_token_id: Optional[int] = None

    def __post_init__(self):
        n = len(self.layers)
        if n < 1:
            raise ValueError("a Faledra model needs at least one layer")
        if self.loop is not None:
            a, b, t = self.loop
            if not (0 <= a < b <= n and t >= 1):
                raise ValueError(f"bad loop {self.loop} for {n} layers")

    @property
    def order(self) -> List[Tuple[int, Optional[int]]]:
        """(layer index, pass that starts with it or None) of every layer run."""
        a, b, t = self.loop or (0, 0, 0)
        runs = [(i, None) for i in range(a)]
        for k in range(t):
            runs += [(i, k if i == a else None) for i in range(a, b)]
        return runs + [(i, None) for i in range(b, len(self.layers))]

    @staticmethod
    def from_json(d: dict) -> "FaledraConfig":
        def mixer(kind, m):
            if kind == "mingru":
                return MinGRUConfig(int(m["width"]))
            if kind != "latent_attention":
                raise ValueError(f"unknown mixer type {kind!r}")
            rot = m["rot"]
            if int(rot.get("dims", m["rot_dim"])) != int(m["rot_dim"]):
                raise ValueError("latent attention rotates the whole rotated part: rot.dims must be rot_dim")
            return LatentAttentionConfig(int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]),
                                         int(m["q_rank"]), int(m["kv_rank"]), float(m["scale"]), float(rot["base"]))

        def ff(m):
            if m is None:
                return None
            if m.get("kind", "dense") != "dense":
                raise ValueError(f"unknown feed-forward kind {m['kind']!r}")
            return int(m["ff"])

        lp, eos = d.get("loop"), d.get("eos_token_id")
        return FaledraConfig(
            vocab_size=int(d["vocab"]), width=int(d["width"]),
            layers=[FaledraLayerConfig(mixer(x["type"], x["mixer"]), ff(x.get("mlp"))) for x in d["layers"]],
            taps=int(d["canon"]["taps"]), eps=float(d["norm"]["eps"]), embed_scale=float(d["embedding"]["scale"]),
            residual_mult=float(d["residual_mult"]),
            loop=(int(lp["start"]), int(lp["stop"]), int(lp["times"])) if lp else None,
            bos_token_id=int(d.get("bos_token_id") or 0), eos_token_id=int(eos) if eos is not None else None)

    @staticmethod
    def uniform(attention: int, mingru: int, width: int, heads: int, dim: int, rot_dim: int, vdim: int, q_rank: int,
                kv_rank: int, gru_width: int, ff: int, vocab: int, taps: int = 4, loop=None) -> "FaledraConfig":
        """``attention`` equal attention layers, then ``mingru`` equal minGRU layers (benchmarks, tests)."""
        att = LatentAttentionConfig(heads, dim, rot_dim, vdim, q_rank, kv_rank, (dim + rot_dim) ** -0.5)
        layers = [FaledraLayerConfig(att, ff)] * attention + [FaledraLayerConfig(MinGRUConfig(gru_width), ff)] * mingru
        return FaledraConfig(vocab, width, layers, taps, embed_scale=width ** 0.5, residual_mult=0.5, loop=loop)

    @staticmethod
    def tiny() -> "FaledraConfig":
        return FaledraConfig.uniform(1, 1, width=128, heads=4, dim=24, rot_dim=8, vdim=40, q_rank=48, kv_rank=80,
                                     gru_width=160, ff=192, vocab=512, taps=3, loop=(0, 1, 2))


class FaledraLayer(nn.Module):
    def __init__(self, cfg: FaledraConfig, c: FaledraLayerConfig, dtype):
        super().__init__()
        D = cfg.width
        self.norm1, self.norm1b = GainNorm(D), GainNorm(D)
        self.conv = InputConv(D, cfg.taps)
        self.mix = (MinGRU(D, c.mixer.width, dtype) if isinstance(c.mixer, MinGRUConfig)
                    else LatentAttention(D, c.mixer, cfg.eps, dtype))
        self.norm2, self.norm2b, self.mlp = ((None, None, None) if c.ff is None
                                             else (GainNorm(D), GainNorm(D), XieluMLP(D, c.ff, dtype)))

    # checkpoint tensors of one gain, taps or row each: (checkpoint name, block)
    parts = (("norm1", "norm1"), ("norm1b", "norm1b"), ("canon1", "conv"), ("norm2", "norm2"), ("norm2b", "norm2b"))


class FaledraForCausalLM(nn.Module):
    needs_prev_token = False
    has_state = True             # sequences hold a state slot (allocate_state); their prefixes cannot be shared by blocks
    attn_span: Optional[int] = None
    dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, cfg: FaledraConfig, dtype=torch.bfloat16):
        super().__init__()
        if tp().size > 1:
            raise ValueError("Faledra runs on one GPU per replica (tensor parallel size 1)")
        self.cfg, self.dtype = cfg, dtype
        W = lm.pad64(cfg.width)
        self.embed = _param(cfg.vocab_size, W, dtype=dtype)
        self.step = _param(cfg.loop[2], W, dtype=torch.float32) if cfg.loop else None
        self.layers = nn.ModuleList([FaledraLayer(cfg, c, dtype) for c in cfg.layers])
        self.final_norm = GainNorm(cfg.width)
        self.head = SoftcapHead(cfg.vocab_size, cfg.width, None, dtype)
        self.order = cfg.order

    def init_random_(self, gen):
        self.embed[:, :self.cfg.width].normal_(0, self.cfg.width ** -0.5, generator=gen)
        if self.step is not None:
            self.step[:, :self.cfg.width].normal_(0, 0.1, generator=gen)

    # ---- engine interface
    def fold_norms(self):
        """The norm gains stay apart: with an fp32 residual the norm is its own (fused) launch."""

    @property
    def kv_heads_local(self) -> int:
        """Workgroups of a decode row per split of its context."""
        heads = max((layer.mix.c.heads for layer in self.layers if isinstance(layer.mix, LatentAttention)), default=1)
        return lm.latent_head_groups(heads)

    def cache_bytes_per_block(self) -> int:
        size = torch.finfo(self.dtype).bits // 8
        shapes = [self.layers[i].mix.cache_shape(1, KV_BLOCK) for i, _ in self.order]
        return max(1, sum(size * torch.Size(s).numel() for s in shapes if s is not None))

    def allocate_cache(self, blocks: int, device):
        """(buffers to keep alive, [latent pool, or None without attention] of every layer run)."""
        shapes = [self.layers[i].mix.cache_shape(blocks, KV_BLOCK) for i, _ in self.order]
        kv = [None if s is None else torch.zeros(s, dtype=self.dtype, device=device) for s in shapes]
        return kv, kv

    def allocate_state(self, slots: int, device):
        """(convolution inputs [runs, slots, taps - 1, width], [recurrent state or None] of every layer run), fp32.  A
        sequence's first token ignores what its slot holds, so slots need no clearing."""
        widths = [self.layers[i].mix.state_width for i, _ in self.order]
        conv = torch.zeros(len(widths), slots, self.cfg.taps - 1, lm.pad64(self.cfg.width), device=device)
        return conv, [None if n is None else torch.zeros(slots, n, device=device) for n in widths]

    def forward(self, batch: Batch, kv_caches, trail: Optional[list] = None) -> torch.Tensor:
        """fp32 logits [rows, vocab]: every row of a decode step, the rows ``batch.last_index`` of a prefill step.
        ``trail`` (a list) receives the residual stream after every layer run."""
        cfg, (conv_state, states) = self.cfg, batch.states
        norm = lambda source, delta, wb, step, w, **kw: lm.residual_norm(
            source, delta, wb, cfg.residual_mult, step, w, cfg.eps, cfg.width, self.dtype, batch=batch, **kw)
        shared = StepShared(batch)
        tail = None
        if batch.is_prefill:
            tail = torch.empty(len(self.order), batch.B, cfg.taps - 1, conv_state.shape[3], device=conv_state.device)
        x, delta, wb = lm.Embedding(batch.input_ids, self.embed, cfg.embed_scale), None, None
        for r, (i, turn) in enumerate(self.order):
            layer = self.layers[i]
            conv = lm.Conv(layer.conv.weight, conv_state[r], tail[r] if tail is not None else None)
            x, h = norm(x, delta, wb, self.step[turn] if turn is not None else None, layer.norm1.weight, conv=conv)
            mem = kv_caches[r] if kv_caches[r] is not None else states[r]
            delta, wb = layer.mix(h, batch, mem, shared), layer.norm1b.weight
            if layer.mlp is not None:
                x, h = norm(x, delta, wb, None, layer.norm2.weight)
                delta, wb = layer.mlp(h), layer.norm2b.weight
            if trail is not None:
                trail.append(norm(x.clone(), delta, wb, None, None)[0][:, :cfg.width])
        if tail is not None:
            lm.conv_commit(conv_state, tail, batch)
        rows = batch.last_index.int() if batch.is_prefill else None
        return self.head(norm(x, delta, wb, None, self.final_norm.weight, rows=rows, keep=False)[1])

    # ---- checkpoint
    def checkpoint_shapes(self) -> Dict[str, tuple]:
        """Every tensor of a checkpoint and its shape."""
        c = self.cfg
        s = {"embed": (c.vocab_size, c.width), "final.norm": (c.width,), "head": (c.vocab_size, c.width)}
        if c.loop is not None:
            s["loop.step"] = (c.loop[2], c.width)
        for i, layer in enumerate(self.layers):
            for name, block in layer.parts:
                if getattr(layer, block) is not None:
                    s[f"l{i}.{name}"] = (c.width, c.taps) if block == "conv" else (c.width,)
            for block in ("mix", "mlp"):
                m = getattr(layer, block)
                if m is not None:
                    s.update({f"l{i}.{block}.{k}": v for k, v in m.shapes().items()})
        return s

    def convert_hf_state_dict(self, sd: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
        """Checkpoint tensors -> packed parameters; a missing, unknown or misshapen tensor is an error."""
        check_checkpoint(sd, self.checkpoint_shapes())
        W = lm.pad64(self.cfg.width)
        wide = lambda t: _padded(t, t.shape[0], W)
        out = {"embed": wide(sd["embed"]), "head.weight": wide(sd["head"]),
               "final_norm.weight": self.final_norm.pack(sd["final.norm"])}
        if self.step is not None:
            out["step"] = wide(sd["loop.step"])
        for i, layer in enumerate(self.layers):
            for name, block in layer.parts:
                if getattr(layer, block) is not None:
                    out[f"layers.{i}.{block}.weight"] = getattr(layer, block).pack(sd[f"l{i}.{name}"])
            for block in ("mix", "mlp"):
                m = getattr(layer, block)
                if m is not None:
                    packed = m.pack(lambda name, p=f"l{i}.{block}.": sd[p + name])
                    out.update({f"layers.{i}.{block}.{k}": v for k, v in packed.items()})
        return out
