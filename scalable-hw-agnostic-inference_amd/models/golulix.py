"""Golulix: a decoder described layer by layer in config.json -- chunked attention without positions and a per-head
output gate, group-limited mixture of experts with a shared expert, a bigram embedding, a run of layers that is passed
several times with the same weights, and a logit softcap.

The model runs on the engine's paged KV cache like the Llama family: :class:`shai_amd.engines.llm.LLMEngine` owns
blocks, scheduling, prefix reuse and sampling.  Every layer RUN (a looped layer counts once per pass) has its own K/V
pools, indexed by the same block table.  The residual stream is fp32; every add is fused with the norm that follows it
(and, after an MoE layer, with the weighted sum of the expert outputs).  A layer of a decode step is 10 launches: norm,
q/k/v/gate GEMM, attention (cache write and gate inside; one more to fold its splits), output GEMM, norm, router + shared
gate/up GEMM, routing and sort (two above 16 rows), expert gate/up, expert down, shared down.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import torch
import torch.nn as nn

from .blocks import (BigramEmbedding, ChunkAttention, ChunkAttentionConfig, ClampedGLUConfig, MoE, MoEConfig,
                     OffsetNorm, SoftcapHead, check_checkpoint)
from .llama import KV_BLOCK, Batch
from ..ops import lm
from ..parallel.state import tp


@dataclass
class GolulixLayerConfig:
    mixer: ChunkAttentionConfig
    mlp: Optional[MoEConfig] = None


@dataclass
class GolulixConfig:
    vocab_size: int
    width: int
    layers: List[GolulixLayerConfig]
    eps: float = 1e-6
    loop: Optional[Tuple[int, int, int]] = None          # (start, stop, times)
    bigram: Optional[Tuple[int, int, int]] = None        # (buckets, mul_prev, mul_cur)
    logit_softcap: Optional[float] = None
    max_position_embeddings: int = 1 << 20               # no positional table: bounded by the cache only
    bos_token_id: int = 0
    eos_token_id: Optional[int] = None

    def __post_init__(self):
        n = len(self.layers)
        if n < 1:
            raise ValueError("a Golulix model needs at least one layer")
        if self.loop is not None:
            a, b, t = self.loop
            if not (0 <= a < b <= n and t >= 1):
                raise ValueError(f"bad loop {self.loop} for {n} layers")

    @property
    def order(self) -> List[Tuple[int, bool]]:
        """(layer index, embedding output added before it) of every layer run."""
        a, b, t = self.loop or (0, 0, 1)
        runs = [(i, False) for i in range(a)]
        for k in range(t):
            runs += [(i, k > 0 and i == a) for i in range(a, b)]
        return runs + [(i, False) for i in range(b, len(self.layers))]

    @staticmethod
    def from_json(d: dict) -> "GolulixConfig":
        def glu(e):
            return ClampedGLUConfig(int(e["ff"]), float(e["limit"]))

        def mlp(m):
            if m is None:
                return None
            if m.get("kind", "moe") != "moe":
                raise ValueError(f"unknown feed-forward kind {m['kind']!r}")
            r, g = m["router"], m["router"].get("groups") or {"count": 1, "keep": 1}
            return MoEConfig(int(r["experts"]), int(r["top"]), glu(m["expert"]), int(g["count"]), int(g["keep"]),
                             glu(m["shared"]) if m.get("shared") else None)

        def layer(x):
            if x["type"] != "attention":
                raise ValueError(f"unknown mixer type {x['type']!r}")
            m = x["mixer"]
            return GolulixLayerConfig(ChunkAttentionConfig(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]),
                                                           int(m["vdim"]), float(m["scale"]), int(m["mask"]["size"])),
                                      mlp(x.get("mlp")))

        lp, big = d.get("loop"), (d.get("embedding") or {}).get("bigram")
        eos = d.get("eos_token_id")
        return GolulixConfig(
            vocab_size=int(d["vocab"]), width=int(d["width"]), layers=[layer(x) for x in d["layers"]],
            eps=float(d["norm"]["eps"]), loop=(int(lp["start"]), int(lp["stop"]), int(lp["times"])) if lp else None,
            bigram=(int(big["buckets"]), int(big["mul_prev"]), int(big["mul_cur"])) if big else None,
            logit_softcap=float(d["logit_softcap"]) if d.get("logit_softcap") else None,
            bos_token_id=int(d.get("bos_token_id") or 0), eos_token_id=int(eos) if eos is not None else None)

    @staticmethod
    def uniform(layers: int, width: int, heads: int, kv_heads: int, dim: int, chunk: int, experts: int, top: int,
                ff: int, shared_ff: int, vocab: int, groups: int = 1, keep: int = 1, loop=None) -> "GolulixConfig":
        """A stack of equal layers (benchmarks, tests)."""
        lc = GolulixLayerConfig(ChunkAttentionConfig(heads, kv_heads, dim, dim, dim ** -0.5, chunk),
                                MoEConfig(experts, top, ClampedGLUConfig(ff, 7.0), groups, keep,
                                          ClampedGLUConfig(shared_ff, 7.0)))
        return GolulixConfig(vocab, width, [lc] * layers, loop=loop, bigram=(1 << 16 | 1, 8191, 131),
                             logit_softcap=30.0)

    @staticmethod
    def tiny() -> "GolulixConfig":
        return GolulixConfig.uniform(layers=2, width=128, heads=4, kv_heads=2, dim=32, chunk=48, experts=8, top=2,
                                     ff=96, shared_ff=64, vocab=512, groups=2, keep=1, loop=(0, 1, 2))


class GolulixLayer(nn.Module):
    def __init__(self, width: int, c: GolulixLayerConfig, eps: float, dtype):
        super().__init__()
        self.norm1 = OffsetNorm(width, eps)
        self.mix = ChunkAttention(width, c.mixer, dtype)
        self.norm2 = OffsetNorm(width, eps) if c.mlp is not None else None
        self.mlp = MoE(width, c.mlp, dtype) if c.mlp is not None else None


class GolulixForCausalLM(nn.Module):
    has_state = False
    needs_prev_token = True   # Batch.prev_ids: the bigram embedding reads every row's preceding token
    dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, cfg: GolulixConfig, dtype=torch.bfloat16):
        super().__init__()
        if tp().size > 1:
            raise ValueError("Golulix runs on one GPU per replica (tensor parallel size 1)")
        self.cfg, self.dtype = cfg, dtype
        buckets, mul_prev, mul_cur = cfg.bigram or (None, 0, 0)
        self.embed = BigramEmbedding(cfg.vocab_size, cfg.width, buckets, mul_prev, mul_cur, dtype)
        self.layers = nn.ModuleList([GolulixLayer(cfg.width, c, cfg.eps, dtype) for c in cfg.layers])
        self.final_norm = OffsetNorm(cfg.width, cfg.eps)
        self.head = SoftcapHead(cfg.vocab_size, cfg.width, cfg.logit_softcap, dtype)
        self.order = cfg.order

    # ---- engine interface
    def fold_norms(self):
        """The norm gains stay apart: with an fp32 residual the norm is its own (fused) launch."""

    @property
    def kv_heads_local(self) -> int:
        return max(layer.mix.c.kv_heads for layer in self.layers)

    @property
    def attn_span(self) -> int:
        """The most keys a position of any layer sees."""
        return max(layer.mix.c.chunk for layer in self.layers)

    def cache_bytes_per_block(self) -> int:
        size = torch.finfo(self.dtype).bits // 8
        return sum(size * torch.Size(s).numel() for i, _ in self.order
                   for s in self.layers[i].mix.cache_shapes(1, KV_BLOCK))

    def allocate_cache(self, blocks: int, device):
        """(buffers to keep alive, [(k, v)] of every layer run)."""
        kv = [tuple(torch.zeros(s, dtype=self.dtype, device=device)
                    for s in self.layers[i].mix.cache_shapes(blocks, KV_BLOCK)) for i, _ in self.order]
        return kv, kv

    def forward(self, batch: Batch, kv_caches, trail: Optional[list] = None) -> torch.Tensor:
        """fp32 logits [rows, vocab]: every row of a decode step, the rows ``batch.last_index`` of a prefill step.
        ``trail`` (a list) receives a copy of the residual stream after every layer run."""
        cfg = self.cfg
        x, h = self.embed(batch.input_ids, batch.prev_ids, self.layers[self.order[0][0]].norm1)
        x0 = x.clone() if any(inject for _, inject in self.order) else None
        delta = None
        for r, (i, inject) in enumerate(self.order):
            layer = self.layers[i]
            if r > 0:
                h = lm.add_norm(x, delta, x0 if inject else None, layer.norm1.weight, cfg.eps, cfg.width, self.dtype)
            delta = layer.mix(h, batch, *kv_caches[r])
            if layer.mlp is not None:
                h = lm.add_norm(x, delta, None, layer.norm2.weight, cfg.eps, cfg.width, self.dtype)
                delta = layer.mlp(h)
            if trail is not None:
                t = x.clone()
                lm.add_norm(t, delta, None, None, cfg.eps, cfg.width, self.dtype)
                trail.append(t[:, :cfg.width])
        rows = batch.last_index.int() if batch.is_prefill else None
        h = lm.add_norm(x, delta, None, self.final_norm.weight, cfg.eps, cfg.width, self.dtype, rows=rows)
        return self.head(h)

    # ---- checkpoint
    def checkpoint_shapes(self) -> Dict[str, tuple]:
        """Every tensor of a checkpoint and its shape."""
        c = self.cfg
        s = {"embed": (c.vocab_size, c.width), "final.norm": (c.width,), "head": (c.vocab_size, c.width)}
        if c.bigram is not None:
            s["bigram"] = (c.bigram[0] + 1, c.width)
        for i, layer in enumerate(self.layers):
            s[f"l{i}.norm1"] = (c.width,)
            s.update({f"l{i}.mix.{k}": v for k, v in layer.mix.shapes().items()})
            if layer.mlp is not None:
                s[f"l{i}.norm2"] = (c.width,)
                s.update({f"l{i}.mlp.{k}": v for k, v in layer.mlp.shapes().items()})
        return s

    def convert_hf_state_dict(self, sd: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
        """Checkpoint tensors -> packed parameters; a missing, unknown or misshapen tensor is an error."""
        check_checkpoint(sd, self.checkpoint_shapes())
        W = lm.pad64(self.cfg.width)
        wide = lambda t: torch.nn.functional.pad(t, (0, W - t.shape[1]))
        out = {"embed.weight": wide(sd["embed"]), "head.weight": wide(sd["head"]),
               "final_norm.weight": self.final_norm.pack(sd["final.norm"])}
        if self.cfg.bigram is not None:
            out["embed.bigram"] = wide(sd["bigram"])
        for i, layer in enumerate(self.layers):
            for block in ("norm1", "norm2"):
                if getattr(layer, block) is not None:
                    out[f"layers.{i}.{block}.weight"] = getattr(layer, block).pack(sd[f"l{i}.{block}"])
            for block in ("mix", "mlp"):
                m = getattr(layer, block)
                if m is not None:
                    packed = m.pack(lambda name, p=f"l{i}.{block}.": sd[p + name])
                    out.update({f"layers.{i}.{block}.{k}": v for k, v in packed.items()})
        return out
