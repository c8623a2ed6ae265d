"""Trace replay: feed given token ids through a model step by step and write the logits it computes.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N   < steps.jsonl

Every input line is one step, ``{"step": n, "entries": [{"id", "tokens", "want"}], "end": [id, ...]}``: its entries run
as one batch through :meth:`LLMEngine.extend` (the engine's packed prefill step, or its decode program when every entry
is a single token), then the requests in ``end`` give their cache back.  The logits of the wanted places go to
``<out>/<step>.f32`` (little-endian fp32, [wanted, vocab]); after every step ``done <step>`` is printed.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import torch

MAX_LIVE = 4   # sequence slots
DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


def build_engine(model_dir: str, dtype: str, max_tokens: int, device="cuda"):
    """An engine whose KV pool holds ``max_tokens`` tokens (whole 64-token blocks), with weights from ``model_dir``."""
    from ..models.llama import KV_BLOCK
    from ..models.registry import config_from_path
    from ..weights import find_safetensors
    from .llm import LLMEngine
    cfg = config_from_path(model_dir)
    if cfg is None or not find_safetensors(model_dir):
        raise FileNotFoundError(f"{model_dir}: config.json and *.safetensors expected")
    blocks = max(1, -(-max_tokens // KV_BLOCK))
    return LLMEngine(cfg, device=device, model_path=model_dir, max_num_seqs=MAX_LIVE, max_model_len=blocks * KV_BLOCK,
                     num_kv_blocks=blocks, enable_prefix_caching=False, dtype=DTYPES[dtype])


def replay(engine, lines, out_dir: str, log=print) -> None:
    live = {}
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = []
        for e in step["entries"]:
            if e["id"] not in live:
                live[e["id"]] = engine.open_request()
            entries.append((live[e["id"]], e["tokens"], e.get("want", [])))
        logits = engine.extend(entries) if entries else None
        if logits is not None:
            path = os.path.join(out_dir, f"{step['step']}.f32")
            logits.float().cpu().contiguous().numpy().astype("<f4").tofile(path)
        for rid in step.get("end", []):
            if rid in live:
                engine.close_request(live.pop(rid))
        log(f"done {step['step']}")


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a token trace and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=sorted(DTYPES), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens live requests hold at any time")
    a = ap.parse_args(argv)
    os.makedirs(a.out, exist_ok=True)
    engine = build_engine(a.model, a.dtype, a.max_tokens)
    replay(engine, sys.stdin, a.out, lambda s: print(s, flush=True))
    return 0


if __name__ == "__main__":
    sys.exit(main())
