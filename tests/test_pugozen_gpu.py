"""Pugozen through the gfx950 kernels, bf16 and fp32, against the plain oracle."""
import os
import subprocess
import sys

import pugozen_cases as C
import pytest
import torch

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.mark.parametrize("dtype", DTYPES, ids=C.name)
@pytest.mark.parametrize("check", C.MECHANISMS, ids=lambda f: f.__name__)
def test_mechanism(cuda, check, dtype):
    check(cuda, dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=C.name)
@pytest.mark.parametrize("key", sorted(C.SHAPES))
def test_shapes(cuda, tmp_path, key, dtype):
    C.check_shape(tmp_path, cuda, dtype, key)


@pytest.mark.parametrize("dtype", DTYPES, ids=C.name)
@pytest.mark.parametrize("check", C.MODELS, ids=lambda f: f.__name__)
def test_model(cuda, tmp_path, check, dtype):
    check(tmp_path, cuda, dtype)


@pytest.mark.parametrize("kw", [{}, {"use_graphs": False}, {"num_kv_blocks": 7}], ids=["graphs", "eager", "preempt"])
def test_greedy_generation(cuda, tmp_path, kw):
    C.check_greedy(tmp_path, cuda, torch.float32, **kw)


def test_greedy_generation_bf16(cuda, tmp_path):
    C.check_greedy(tmp_path, cuda, torch.bfloat16)


def test_captured_decode_replays_equal_eager(cuda, tmp_path):
    """Decode-program replays, with eager steps and synchronisations between them, against the same steps run eagerly."""
    from shai_amd.engines.llm import LLMEngine
    from shai_amd.models.registry import config_from_path
    c = C.Case(tmp_path, cuda, torch.bfloat16, seed=21)
    mk = lambda g: LLMEngine(config_from_path(c.path), device=cuda, model_path=c.path, max_num_seqs=4, max_model_len=192,
                             use_graphs=g)
    a, b = mk(True), mk(False)
    sa, sb = [[e.open_request() for _ in range(3)] for e in (a, b)]
    toks = [c.tokens(120) for _ in range(3)]
    at = 0
    for i, n in enumerate((9, 1, 1, 2, 1, 1, 1, 30, 1, 1, 1, 1)):
        out = [e.extend([(s, t[at:at + n], [n - 1]) for s, t in zip(ss, toks)]) for e, ss in ((a, sa), (b, sb))]
        at += n
        assert torch.equal(out[0], out[1]), i
        torch.cuda.synchronize()


def test_trace_run_program(cuda, tmp_path):
    c = C.Case(tmp_path, cuda, torch.float32, seed=22)
    toks = c.tokens(32)
    for dtype in DTYPES:
        out = tmp_path / C.name(dtype)
        r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", c.path, "--dtype",
                            C.name(dtype), "--out", str(out), "--max-tokens", "128"],
                           input="\n".join(C.replay_lines(c, toks)) + "\n", capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr[-2000:]
        said = [ln for ln in r.stdout.splitlines() if ln.startswith("done")]
        C.check_replay_files(c, toks, out, said, dtype)


def test_prompts_in_rounds(cuda, monkeypatch):
    """Heads whose prepared chunks do not fit the workspace together run in several rounds."""
    monkeypatch.setattr(C.lm, "RULE_WORKSPACE", 1)
    C.check_mixers(cuda, torch.bfloat16)
    monkeypatch.setattr(C.lm, "RULE_WORKSPACE", 1 << 20)
    C.check_delta(cuda, torch.bfloat16)
    C.check_retention(cuda, torch.bfloat16)


@pytest.mark.parametrize("rows", [32, 96])
def test_prompts_in_segments(cuda, monkeypatch, rows):
    """Prompts cut into segments that are scanned side by side: at every head size, in batches of unequal lengths."""
    monkeypatch.setattr(C.lm, "rule_segment", lambda *_: rows)
    for check in (C.check_delta, C.check_delta_memory, C.check_retention, C.check_mixers):
        check(cuda, torch.bfloat16)
