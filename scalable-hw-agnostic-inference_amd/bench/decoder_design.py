"""Prefill and decode throughput of a layer-list design (Golulix, Faledra, Nalizen, Pugozen) beside models of equal size.

Both run through :class:`LLMEngine` (scheduler, paged cache, HIP-graph decode) with random weights.  A pair has the same
width, layers, heads and vocabulary.  The Llama MLP is as wide as the feed-forward work one Golulix token does (top x
expert + shared expert), or has as many weights as the Faledra feed-forward (3 D I = 2 D ff), so the two do the same
matrix work per token there.  Nalizen runs beside Golulix too (both are mixtures of experts): equal routing, gated experts
of the same number of weights as its ungated ones, and a chunk that holds the whole sequence.  Pugozen runs beside a Nalizen
model with dense feed-forwards of as many weights: window attention (a window that holds the sequence) where Pugozen has
attention beside a delta rule, HGRN2 of equal heads where it has a recurrence alone.

    python bench.py --workload golulix|faledra|nalizen|pugozen [--design-size small|large|both]
    python -m shai_amd.bench.decoder_design --design faledra --model faledra --size small --batch 64      # profiling
"""
from __future__ import annotations

import argparse
import time

# width, layers, heads, kv heads, head size, chunk, experts, top, expert ff, shared ff, vocab, expert groups, kept
SIZES = {"small": (2048, 8, 16, 4, 128, 2048, 64, 6, 1408, 2816, 32768, 8, 4),
         "large": (4096, 6, 32, 8, 128, 8192, 64, 4, 2048, 4096, 65536, 4, 2)}
# width, attention layers, minGRU layers, heads, unrotated / rotated / value head size, query latent, key-value latent,
# minGRU width, ff, vocab, kv heads of the Llama model (head size: the unrotated one)
FALEDRA_SIZES = {"small": (2048, 6, 2, 16, 128, 64, 128, 768, 512, 2048, 8448, 32768, 4),
                 "large": (4096, 4, 2, 32, 128, 64, 128, 1536, 512, 4096, 16896, 65536, 8)}


# layers (NalizenConfig.uniform), width, heads, kv heads, head size, window, recurrence heads, their key and value size, dense
# ff, experts, top, expert ff, token input size, vocab
NALIZEN_SIZES = {"small": ("aRRSARRS", 2048, 16, 4, 128, 1024, 16, 128, 128, 8448, 64, 6, 2112, 256, 32768),
                 "large": ("aRSARS", 4096, 32, 8, 128, 4096, 32, 128, 128, 8192, 64, 4, 3072, 256, 65536)}

# layers (PugozenConfig.uniform), width, heads, kv heads, head size, recurrence heads, query / key heads of the delta rule, key and
# value size, rank of thin products, ff, vocab
PUGOZEN_SIZES = {"small": ("DPRPDPRP", 2048, 16, 4, 128, 16, 8, 128, 128, 128, 8448, 32768),
                 "large": ("DPRDPR", 4096, 32, 8, 128, 32, 16, 128, 128, 128, 12288, 65536)}


def configs(size: str, design: str = "golulix"):
    from ..models.llama import LlamaConfig
    out = {}
    if design == "faledra":
        from ..models.faledra import FaledraConfig
        D, A, R, H, d, rot, dv, q, kv, gru, ff, V, G = FALEDRA_SIZES[size]
        cfg, L, inner = FaledraConfig.uniform(A, R, D, H, d, rot, dv, q, kv, gru, ff, V), A + R, 2 * ff // 3
    elif design == "pugozen":
        from ..models.nalizen import NalizenConfig
        from ..models.pugozen import PugozenConfig
        kinds, D, H, G, d, sh, _, sd, sv, _, ff, V = PUGOZEN_SIZES[size]
        cfg, L, inner = PugozenConfig.uniform(*PUGOZEN_SIZES[size]), len(kinds), 2 * ff // 3
        out["nalizen"] = NalizenConfig.uniform("".join("a" if k.upper() == "P" else "r" for k in kinds), D, H, G, d, 1 << 20, sh,
                                               sd, sv, inner, 1, 1, 64, 64, V)
    elif design == "nalizen":
        from ..models.golulix import GolulixConfig
        from ..models.nalizen import NalizenConfig
        kinds, D, H, G, d, window, _, _, _, ff, E, top, eff, _, V = NALIZEN_SIZES[size]
        cfg, L, inner = NalizenConfig.uniform(*NALIZEN_SIZES[size]), len(kinds), 2 * top * eff // 3
        out["golulix"] = GolulixConfig.uniform(layers=L, width=D, heads=H, kv_heads=G, dim=d, chunk=2 * window, experts=E,
                                               top=top, ff=2 * eff // 3, shared_ff=64, vocab=V)
    else:
        from ..models.golulix import GolulixConfig
        D, L, H, G, d, chunk, E, top, ff, sff, V, groups, keep = SIZES[size]
        cfg = GolulixConfig.uniform(layers=L, width=D, heads=H, kv_heads=G, dim=d, chunk=chunk, experts=E, top=top, ff=ff,
                                    shared_ff=sff, vocab=V, groups=groups, keep=keep)
        inner = top * ff + sff
    ll = LlamaConfig(vocab_size=V, hidden_size=D, intermediate_size=inner, num_hidden_layers=L, num_attention_heads=H,
                     num_key_value_heads=G, head_dim=d, max_position_embeddings=32768)
    return {design: cfg, **out, "llama": ll}


def measure(cfg, batch: int, prompt: int, gen: int, repeats: int = 3, device: str = "cuda:0") -> dict:
    """Median prefill and decode tokens/s of ``batch`` prompts of ``prompt`` tokens, ``gen`` sampled tokens each."""
    import numpy as np
    import torch
    from ..engines.llm import LLMEngine, SamplingParams
    eng = LLMEngine(cfg, device=device, max_num_seqs=batch, max_model_len=prompt + gen + 64, enable_prefix_caching=False,
                    prefill_token_budget=batch * prompt)
    rng = np.random.default_rng(0)
    params = SamplingParams(temperature=0.7, top_k=50, top_p=0.9, max_tokens=gen, ignore_eos=True)
    sync = torch.cuda.synchronize if eng.device.type == "cuda" else (lambda: None)
    pre, dec = [], []
    with torch.inference_mode():
        for r in range(repeats + 1):            # the first pass captures graphs and tunes GEMMs: not counted
            seqs = [eng.add_request(rng.integers(0, cfg.vocab_size, prompt).tolist(), params) for _ in range(batch)]
            sync()
            t0 = time.perf_counter()
            while any(not s.output for s in seqs):
                eng.step()
            sync()
            t1 = time.perf_counter()
            while eng.has_work():
                eng.step()
            sync()
            t2 = time.perf_counter()
            if r:
                pre.append(batch * prompt / (t1 - t0))
                dec.append(batch * (gen - 1) / (t2 - t1) if gen > 1 else 0.0)
    del eng
    if device != "cpu":
        torch.cuda.empty_cache()
    return {"prefill_tok_s": round(sorted(pre)[len(pre) // 2], 1), "decode_tok_s": round(sorted(dec)[len(dec) // 2], 1)}


def bench(args, rank: int, world: int) -> dict:
    """The bench.py line: every (size, batch) pair of both models; ``value`` is the design's decode at the largest batch."""
    import torch
    design = args.workload
    if world != 1:
        raise SystemExit(f"--workload {design} runs on one GPU")
    sizes = list(SIZES) if args.design_size == "both" else [args.design_size]
    rows, P, G, t0 = [], 1024, 64, time.perf_counter()
    steps = max(1, args.steps)
    for size in sizes:
        cfgs = configs(size, design)
        for batch in (1, 8, args.batch):
            row = {"size": size, "batch": batch, "prompt_len": P, "gen_len": G}
            for name, cfg in cfgs.items():
                row[name] = measure(cfg, batch, P, G, steps, f"cuda:{torch.cuda.current_device()}")
            rows.append(row)
    last = rows[-1]
    model = {"golulix": lambda n: f"Golulix {n}: (width, layers, heads, kv heads, head size, chunk, experts, top, expert "
                                  f"ff, shared ff, vocab, groups, kept) = {SIZES[n]}",
             "faledra": lambda n: f"Faledra {n}: (width, attention layers, minGRU layers, heads, unrotated / rotated / value "
                                  f"head size, query latent, key-value latent, minGRU width, ff, vocab) = "
                                  f"{FALEDRA_SIZES[n][:-1]}",
             "nalizen": lambda n: f"Nalizen {n}: (layers, width, heads, kv heads, head size, window, recurrence heads, key and "
                                  f"value size, dense ff, experts, top, expert ff, token input, vocab) = "
                                  f"{NALIZEN_SIZES[n]}",
             "pugozen": lambda n: f"Pugozen {n}: (layers, width, heads, kv heads, head size, recurrence heads, query / key heads "
                                  f"of the delta rule, key and value size, rank, ff, vocab) = {PUGOZEN_SIZES[n]}"}[design](last["size"])
    return {"metric": f"{design.capitalize()} decode tokens/s (random weights, beside a Llama model of equal size)",
            "value": last[design]["decode_tok_s"], "unit": "tokens/s", "n_gpus": 1, "steps": steps, "warmup": 1,
            "ms_per_step": round(1000 * (time.perf_counter() - t0) / (sum(len(configs(r['size'], design)) for r in rows) * (steps + 1)), 2),
            "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16",
            "data": "synthetic prompts, random-init weights",
            "config": {"model": model, "global_batch": last["batch"], "seq_len": P + G, "parallelism": "dp1"},
            "pairs": rows}


def main(argv=None):
    ap = argparse.ArgumentParser()
    ap.add_argument("--design", choices=["golulix", "faledra", "nalizen", "pugozen"], default="golulix")
    ap.add_argument("--model", choices=["design", "golulix", "faledra", "nalizen", "pugozen", "llama"], default="design")
    ap.add_argument("--size", choices=sorted(SIZES), default="small")
    ap.add_argument("--batch", type=int, default=64)
    ap.add_argument("--prompt", type=int, default=1024)
    ap.add_argument("--gen", type=int, default=64)
    ap.add_argument("--repeats", type=int, default=2)
    a = ap.parse_args(argv)
    cfgs = configs(a.size, a.design)
    name = a.design if a.model == "design" else a.model
    if name not in cfgs:
        ap.error(f"--model {a.model} is not part of --design {a.design}")
    print(measure(cfgs[name], a.batch, a.prompt, a.gen, a.repeats), flush=True)


if __name__ == "__main__":
    main()
