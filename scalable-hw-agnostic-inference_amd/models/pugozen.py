"""Pugozen: a decoder described layer by layer in config.json -- every layer adds a mixer and a squared-ReLU feed-forward that
read the same norm.  A mixer is retention (linear attention with a fixed decay per head), the gated delta rule (one decay per
head), or tied causal attention beside a delta rule with a decay per key channel.  A layer may use the weights of another
one, with a cache and a state of its own.

The model runs on the engine like the Llama family: :class:`shai_amd.engines.llm.LLMEngine` owns blocks, state slots,
scheduling and sampling.  An attention has its K/V pools, a recurrence a matrix state per head and sequence slot (fp32) and the
last inputs of its short convolutions.  The residual stream is fp32.  A layer is one norm, one product for all inputs, the
mixer's kernel(s) and one product for all outputs: 4 launches of a decode step for retention and the delta rule, 6 (7 with
split attention) for attention beside a delta rule.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple, Union

import torch
import torch.nn as nn

from .blocks import (DeltaRule, DeltaRuleConfig, GainNorm, JointLayer, Retention, RetentionConfig, SoftcapHead, StepShared,
                     TiedAttention, TiedAttentionConfig, _padded, _param, check_checkpoint)
from .llama import KV_BLOCK, Batch
from ..ops import lm
from ..parallel.state import tp


@dataclass
class PugozenLayerConfig:
    mixer: Union[RetentionConfig, DeltaRuleConfig, Tuple[TiedAttentionConfig, DeltaRuleConfig]]
    ff: Optional[int] = None
    weights_of: Optional[int] = None


@dataclass
class PugozenConfig:
    vocab_size: int
    width: int
    layers: List[PugozenLayerConfig]
    eps: float = 1e-6
    embed_scale: float = 1.0
    max_position_embeddings: int = 1 << 20               # angles are computed: bounded by the cache only
    bos_token_id: int = 0
    eos_token_id: Optional[int] = None

    def __post_init__(self):
        if not self.layers:
            raise ValueError("a Pugozen model needs at least one layer")
        for i, lc in enumerate(self.layers):
            j = lc.weights_of
            if j is None:
                continue
            if not 0 <= j < len(self.layers) or self.layers[j].weights_of is not None:
                raise ValueError(f"layer {i}: weights come from a layer with its own, not {j}")
            if (self.layers[j].mixer, self.layers[j].ff) != (lc.mixer, lc.ff):
                raise ValueError(f"layers {j} and {i} share weights: their sizes must be equal")

    @property
    def order(self) -> List[int]:
        """The layer whose weights every layer uses."""
        return [i if lc.weights_of is None else lc.weights_of for i, lc in enumerate(self.layers)]

    @staticmethod
    def from_json(d: dict, shapes: Optional[Dict[str, tuple]] = None) -> "PugozenConfig":
        """``shapes``: the checkpoint's tensors, whose shapes alone tell the ranks of thin products (without them: the head
        size)."""
        entries = d["layers"]

        def own(i, x):
            """The layer whose tensors layer i uses, if not its own."""
            j = x.get("weights_of")
            for _ in entries:
                if j is None or not 0 <= int(j) < len(entries) or entries[int(j)].get("weights_of") is None:
                    return None if j is None else int(j)
                j = entries[int(j)]["weights_of"]
            raise ValueError(f"layer {i}: no layer has its weights")

        def rule(m, **kw):
            return DeltaRuleConfig(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), int(m["conv"]), **kw)

        def mixer(i, x):
            m, kind = x["mixer"], x["type"]
            if kind == "retention":
                if len(m["decay"]) != int(m["heads"]):
                    raise ValueError(f"layer {i}: one decay per head")
                return RetentionConfig(tuple(float(v) for v in m["decay"]), int(m["dim"]), int(m["vdim"]),
                                       int(m["rot"]["dims"]), float(m["rot"]["base"]))
            if kind == "delta":
                return rule(m)
            if kind != "parallel":
                raise ValueError(f"unknown mixer type {kind!r}")
            a, r, j = m["left"], m["right"], own(i, x)
            if int(a["vdim"]) != int(a["dim"]):
                raise ValueError(f"layer {i}: values are the projected keys, so vdim must be dim")
            at = f"l{i if j is None else j}.mix.right."
            ranks = tuple(int(shapes[at + n][0]) if shapes and at + n in shapes else int(r["dim"]) for n in ("a1", "g1"))
            return (TiedAttentionConfig(int(a["heads"]), int(a["kv_heads"]), int(a["dim"]), float(a["scale"]),
                                        int(a["rot"]["dims"]), float(a["rot"]["base"]), float(m["left_scale"])),
                    rule(r, ranks=ranks, gate=lm.GATE_SIGMOID, out_scale=float(m["right_scale"])))

        def ff(m):
            if m is None:
                return None
            if m["kind"] != "dense":
                raise ValueError(f"unknown feed-forward kind {m['kind']!r}")
            return int(m["ff"])

        eos = d.get("eos_token_id")
        return PugozenConfig(
            vocab_size=int(d["vocab"]), width=int(d["width"]),
            layers=[PugozenLayerConfig(mixer(i, x), ff(x.get("mlp")), own(i, x)) for i, x in enumerate(entries)],
            eps=float(d["norm"]["eps"]), embed_scale=float(d["embedding"]["scale"]),
            bos_token_id=int(d.get("bos_token_id") or 0), eos_token_id=int(eos) if eos is not None else None)

    @staticmethod
    def uniform(layers: str, width: int, heads: int, kv_heads: int, dim: int, state_heads: int, state_kv_heads: int,
                state_dim: int, state_vdim: int, rank: int, ff: int, vocab: int, taps: int = 4) -> "PugozenConfig":
        """Layers of equal sizes (benchmarks, tests).  ``layers``: a letter each, D delta rule, P attention beside a delta
        rule, R retention; lower case: the weights of the last layer of that kind with its own."""
        rule = lambda kv, **kw: DeltaRuleConfig(state_heads, kv, state_dim, state_vdim, taps, **kw)
        decay = tuple(1.0 - 2.0 ** -(5.0 + 5.0 * h / state_heads) for h in range(state_heads))
        kinds = {"D": rule(state_kv_heads), "R": RetentionConfig(decay, state_dim, state_vdim, state_dim),
                 "P": (TiedAttentionConfig(heads, kv_heads, dim, dim ** -0.5, dim // 2, out_scale=0.7),
                       rule(state_heads, ranks=(rank, rank), gate=lm.GATE_SIGMOID, out_scale=0.7))}
        out, last = [], {}
        for i, kind in enumerate(layers):
            if kind.isupper():
                last[kind] = i
            out.append(PugozenLayerConfig(kinds[kind.upper()], ff, None if kind.isupper() else last[kind.upper()]))
        return PugozenConfig(vocab, width, out)

    @staticmethod
    def tiny() -> "PugozenConfig":
        return PugozenConfig.uniform("PDRp", width=128, heads=4, kv_heads=2, dim=32, state_heads=4, state_kv_heads=2,
                                     state_dim=24, state_vdim=40, rank=16, ff=192, vocab=512)


class PugozenLayer(nn.Module):
    def __init__(self, cfg: PugozenConfig, c: PugozenLayerConfig, dtype):
        super().__init__()
        D = cfg.width
        if isinstance(c.mixer, tuple):
            mixers = {"left": TiedAttention(D, c.mixer[0], cfg.eps), "right": DeltaRule(D, c.mixer[1], cfg.eps, dtype)}
        elif isinstance(c.mixer, RetentionConfig):
            mixers = {"only": Retention(D, c.mixer, cfg.eps)}
        else:
            mixers = {"only": DeltaRule(D, c.mixer, cfg.eps, dtype)}
        self.norm1 = GainNorm(D)
        self.joint = JointLayer(D, mixers, c.ff or 0, dtype)


class PugozenForCausalLM(nn.Module):
    needs_prev_token = False
    has_state = True             # sequences hold a state slot (allocate_state); their prefixes cannot be shared by blocks
    attn_span: Optional[int] = None
    dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, cfg: PugozenConfig, dtype=torch.bfloat16):
        super().__init__()
        if tp().size > 1:
            raise ValueError("Pugozen runs on one GPU per replica (tensor parallel size 1)")
        self.cfg, self.dtype, self.order = cfg, dtype, cfg.order
        self.embed = _param(cfg.vocab_size, lm.pad64(cfg.width), dtype=dtype)
        self.layers = nn.ModuleDict({str(i): PugozenLayer(cfg, cfg.layers[i], dtype) for i in sorted(set(self.order))})
        self.final_norm = GainNorm(cfg.width)
        self.head = SoftcapHead(cfg.vocab_size, cfg.width, None, dtype)

    def runs(self) -> List[PugozenLayer]:
        """The weights of every layer run."""
        return [self.layers[str(i)] for i in self.order]

    def init_random_(self, gen):
        self.embed[:, :self.cfg.width].normal_(0, self.cfg.width ** -0.5, generator=gen)

    # ---- engine interface
    def fold_norms(self):
        """The norm gains stay apart: with an fp32 residual the norm is its own (fused) launch."""

    @property
    def kv_heads_local(self) -> int:
        return max((lc.mixer[0].kv_heads for lc in self.cfg.layers if isinstance(lc.mixer, tuple)), default=1)

    def cache_bytes_per_block(self) -> int:
        size = torch.finfo(self.dtype).bits // 8
        shapes = [layer.joint.cache_shapes(1, KV_BLOCK) for layer in self.runs()]
        return max(1, sum(size * torch.Size(s).numel() for pair in shapes if pair is not None for s in pair))

    def allocate_cache(self, blocks: int, device):
        """(buffers to keep alive, [(k, v) or None without attention] of every layer run)."""
        shapes = [layer.joint.cache_shapes(blocks, KV_BLOCK) for layer in self.runs()]
        kv = [s and tuple(torch.zeros(x, dtype=self.dtype, device=device) for x in s) for s in shapes]
        return kv, kv

    def allocate_state(self, slots: int, device):
        """[recurrent state (fp32) and, with short convolutions, their last inputs] of every layer run.  A sequence's first
        token ignores what its slot holds, so slots need no clearing."""
        make = lambda shape, f32: torch.zeros(slots, *shape, dtype=torch.float32 if f32 else self.dtype, device=device)
        return [[make(*s) for s in layer.joint.state_shapes()] for layer in self.runs()]

    def forward(self, batch: Batch, kv_caches, trail: Optional[list] = None) -> torch.Tensor:
        """fp32 logits [rows, vocab]: every row of a decode step, the rows ``batch.last_index`` of a prefill step.
        ``trail`` (a list) receives the residual stream after every layer."""
        cfg, step = self.cfg, StepShared(batch)
        norm = lambda source, delta, w, **kw: lm.residual_norm(source, delta, lm.PLAIN, 1.0, None, w, cfg.eps, cfg.width,
                                                               self.dtype, batch=batch, **kw)
        x, delta = lm.Embedding(batch.input_ids, self.embed, cfg.embed_scale), None
        for r, layer in enumerate(self.runs()):
            x, h = norm(x, delta, layer.norm1.weight)
            delta = layer.joint(h, batch, kv_caches[r], batch.states[r], step)
            if trail is not None:
                trail.append(norm(x.clone(), delta, None)[0][:, :cfg.width])
        rows = batch.last_index.int() if batch.is_prefill else None
        return self.head(norm(x, delta, self.final_norm.weight, rows=rows, keep=False)[1])

    # ---- checkpoint
    def checkpoint_shapes(self) -> Dict[str, tuple]:
        """Every tensor of a checkpoint and its shape."""
        c = self.cfg
        s = {"embed": (c.vocab_size, c.width), "final.norm": (c.width,), "head": (c.vocab_size, c.width)}
        for i, layer in self.layers.items():
            s[f"l{i}.norm1"] = (c.width,)
            s.update({f"l{i}.{k}": v for k, v in layer.joint.shapes().items()})
        return s

    def convert_hf_state_dict(self, sd: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
        """Checkpoint tensors -> packed parameters; a missing, unknown or misshapen tensor is an error."""
        check_checkpoint(sd, self.checkpoint_shapes())
        wide = lambda t: _padded(t, t.shape[0], lm.pad64(self.cfg.width))
        out = {"embed": wide(sd["embed"]), "head.weight": wide(sd["head"]),
               "final_norm.weight": self.final_norm.pack(sd["final.norm"])}
        for i, layer in self.layers.items():
            out[f"layers.{i}.norm1.weight"] = layer.norm1.pack(sd[f"l{i}.norm1"])
            out.update({f"layers.{i}.joint.{k}": v
                        for k, v in layer.joint.pack_all(lambda name, p=f"l{i}.": sd[p + name]).items()})
        return out
