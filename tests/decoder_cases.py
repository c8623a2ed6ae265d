"""What the tests of the layer-list decoders (Golulix, Faledra) share: cases on the framework's engine, driven by portions,
batches, generation and trace replay, and their comparison with a design's oracle."""
import json

import numpy as np
import torch

from shai_amd.engines import trace

# error of a position: rms over the vocabulary of the logit difference (mean taken off), in units of the logits' rms
F32_TOL, BF16_TOL = 1e-4, 0.06


def position_errors(got, want):
    d = got.double().cpu() - want.double()
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.double().pow(2).mean().sqrt()


def assert_logits(got, want, dtype, what=""):
    e = position_errors(got, want)
    if dtype == torch.float32:
        assert e.max() < F32_TOL, f"{what}: {e.max():.2e} at {int(e.argmax())}"
    else:   # a near tie in a router may flip an expert in bf16: nearly all positions, not all
        assert e.quantile(0.9) < BF16_TOL and e.median() < BF16_TOL / 2, f"{what}: {e.quantile(0.9):.3f}"


def name(dtype):
    return {torch.float32: "float32", torch.bfloat16: "bfloat16"}[dtype]


def tensors(x):
    """The tensors of nested lists and tuples."""
    if isinstance(x, torch.Tensor):
        yield x
    elif x is not None:
        for y in x:
            yield from tensors(y)


class Case:
    """A random model: config, oracle weights, checkpoint folder, and engines on it."""

    ref = None   # the design's oracle module

    def __init__(self, tmp, device, dtype, seed=0, **sizes):
        R = self.ref
        self.cfg = R.random_config(**sizes)
        self.w = R.random_weights(self.cfg, seed)
        self.path = R.save_checkpoint(tmp / f"m{seed}", self.cfg, self.w)
        self.device, self.dtype = device, dtype
        self.rng = np.random.default_rng(seed + 100)

    def tokens(self, n):
        return self.rng.integers(0, self.cfg["vocab"], n).tolist()

    def oracle(self, tokens):
        return self.ref.forward(tokens, self.cfg, self.w)[0]

    def engine(self, max_tokens=512, dirty=True):
        eng = trace.build_engine(self.path, name(self.dtype), max_tokens, self.device)
        if dirty:   # whatever an unwritten cache row or state slot holds must not matter
            for t in tensors((eng.kv, eng.states)):
                t.fill_(37.0)
        return eng


def run(eng, s, tokens, cuts):
    """Logits of every token of ``tokens``, fed to request ``s`` in portions of the sizes ``cuts`` (cycled)."""
    out, at, i = [], 0, 0
    while at < len(tokens):
        n = min(cuts[i % len(cuts)], len(tokens) - at)
        out.append(eng.extend([(s, tokens[at:at + n], list(range(n)))]).double().cpu())
        at, i = at + n, i + 1
    return torch.cat(out)


def run_batches(c, eng, reqs, check=assert_logits):
    """``reqs`` (name -> tokens) with up to four live at a time, portions beside single tokens, some pausing; pages and
    slots are reused, and every request gets the logits it gets alone."""
    want = {k: c.oracle(t) for k, t in reqs.items()}
    todo, live, got = list(reqs), {}, {k: [] for k in reqs}
    while todo or live:
        while todo and len(live) < 4 and sum(-(-len(reqs[k]) // 64) for k in (*live, todo[0])) <= 8:
            k = todo.pop(0)
            live[k] = [eng.open_request(), 0]
        entries, steps = [], []
        for k, (s, at) in live.items():
            if len(live) > 1 and c.rng.random() < 0.2:
                continue                            # left out of this step
            n = min(int(c.rng.choice([1, 1, 1, 2, 3, 17, 64])), len(reqs[k]) - at)
            entries.append((s, reqs[k][at:at + n], list(range(n))))
            steps.append((k, n))
        if not entries:
            continue
        out, at = eng.extend(entries).double().cpu(), 0
        for k, n in steps:
            got[k].append(out[at:at + n])
            at += n
            live[k][1] += n
            if live[k][1] == len(reqs[k]):
                eng.close_request(live.pop(k)[0])
    assert eng.bm.num_free == eng.num_kv_blocks
    for k in reqs:
        check(torch.cat(got[k]), want[k], c.dtype, k)


def greedy_oracle(c, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(c.oracle(toks)[-1].argmax()))
    return toks[len(prompt):]


def replay_lines(c, toks):
    yield json.dumps({"step": 0, "entries": [{"id": "a", "tokens": toks[:30], "want": [0, 29]}], "end": []})
    yield json.dumps({"step": 1, "entries": [{"id": "a", "tokens": toks[30:31], "want": []}], "end": []})
    yield json.dumps({"step": 7, "entries": [{"id": "b", "tokens": toks[:2], "want": [1]},
                                             {"id": "a", "tokens": toks[31:32], "want": [0]}], "end": ["a", "b"]})
    yield json.dumps({"step": 8, "entries": [{"id": "a", "tokens": toks[:1], "want": [0]}], "end": ["a"]})


def check_replay_files(c, toks, out, said, dtype):
    want = c.oracle(toks)
    assert said == ["done 0", "done 1", "done 7", "done 8"]
    read = lambda n: torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, c.cfg["vocab"]))
    assert_logits(read(0), want[[0, 29]], dtype)
    assert_logits(read(7), want[[1, 31]], dtype)
    assert_logits(read(8), want[[0]], dtype)
    assert not (out / "1.f32").exists()
