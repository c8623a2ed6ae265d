"""Causal language models the LLM engine serves: config.json -> config object -> model class.

A model class offers the engine: ``forward(batch, kv_caches)`` -> logits, ``kv_heads_local``, ``fold_norms()``,
``allocate_cache(blocks, device)``, ``cache_bytes_per_block()``, and the attributes ``dtypes`` (weight formats it runs
in), ``needs_prev_token`` (rows carry their preceding token), ``attn_span`` (most keys a position sees, or None) and
``has_state`` (sequences hold a slot of the state that ``allocate_state(slots, device)`` makes; ``Batch.states``).
"""
from __future__ import annotations

import json
import os
from typing import Callable, Dict, Optional

from .faledra import FaledraConfig, FaledraForCausalLM
from .golulix import GolulixConfig, GolulixForCausalLM
from .llama import LlamaConfig, LlamaForCausalLM
from .mllama import MllamaConfig, MllamaForConditionalGeneration
from .nalizen import NalizenConfig, NalizenForCausalLM
from .pugozen import PugozenConfig, PugozenForCausalLM

MODELS = {LlamaConfig: LlamaForCausalLM, MllamaConfig: MllamaForConditionalGeneration,
          GolulixConfig: GolulixForCausalLM, FaledraConfig: FaledraForCausalLM,
          NalizenConfig: NalizenForCausalLM, PugozenConfig: PugozenForCausalLM}

# config.json "architecture" -> config reader, for designs that name themselves that way
ARCHITECTURES: Dict[str, Callable[[dict], object]] = {"Golulix": GolulixConfig.from_json,
                                                       "Faledra": FaledraConfig.from_json,
                                                       "Nalizen": NalizenConfig.from_json,
                                                       "Pugozen": PugozenConfig.from_json}
# those with sizes that only the shapes of the checkpoint's tensors tell
SIZED_BY_TENSORS = ("Pugozen",)


def config_from_json(d: dict, shapes: Optional[Dict[str, tuple]] = None):
    """The config object of a parsed config.json (HF-style files: Llama family, or mllama with a vision tower).  ``shapes``:
    those of the checkpoint's tensors, for the designs that need them."""
    name = d.get("architecture")
    if name is not None:
        if name not in ARCHITECTURES:
            raise ValueError(f"unknown architecture {name!r}: known are {sorted(ARCHITECTURES)}")
        return ARCHITECTURES[name](d, shapes) if name in SIZED_BY_TENSORS else ARCHITECTURES[name](d)
    if "vision_config" in d and "text_config" in d:
        return MllamaConfig.from_hf(d)
    return LlamaConfig.from_hf(d.get("text_config", d))


def config_from_path(path: Optional[str]):
    """Config of a checkpoint folder, or None without a config.json."""
    f = os.path.join(path, "config.json") if path else None
    if not f or not os.path.exists(f):
        return None
    with open(f) as h:
        d = json.load(h)
    if d.get("architecture") not in SIZED_BY_TENSORS:
        return config_from_json(d)
    from ..weights import find_safetensors, safetensors_shapes
    return config_from_json(d, safetensors_shapes(find_safetensors(path)))


def model_class(cfg):
    return MODELS[type(cfg)]
