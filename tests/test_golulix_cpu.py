"""Golulix on the CPU references: the engine integration (registry, loader, cache, scheduler, sampling, trace replay)
against the plain oracle, and that the comparison notices a planted mistake."""
import golulix_cases as C
import golulix_reference as R
import pytest
import torch

CPU, F32, BF16 = "cpu", torch.float32, torch.bfloat16


@pytest.mark.parametrize("check", C.MECHANISMS, ids=lambda f: f.__name__)
def test_mechanism(check):
    check(CPU, F32)


def test_mechanism_bf16():
    C.check_moe(CPU, BF16)
    C.check_attention(CPU, BF16)


@pytest.mark.parametrize("key", sorted(C.SHAPES))
def test_shapes(tmp_path, key):
    C.check_shape(tmp_path, CPU, F32, key)


@pytest.mark.parametrize("check", C.MODELS, ids=lambda f: f.__name__)
def test_model(tmp_path, check):
    check(tmp_path, CPU, F32)


def test_model_bf16(tmp_path):
    C.check_batches(tmp_path, CPU, BF16)


@pytest.mark.parametrize("kw", [{}, {"async_decode": False, "enable_prefix_caching": False}, {"mixed_steps": False},
                                {"num_kv_blocks": 7, "enable_prefix_caching": False}],
                         ids=["default", "sync", "unmixed", "preempt"])
def test_greedy_generation(tmp_path, kw):
    C.check_greedy(tmp_path, CPU, F32, **kw)


def test_planted_mistakes_show(tmp_path):
    c = C.Case(tmp_path, CPU, F32, seed=11)
    toks = c.tokens(64)
    eng = c.engine()
    s = eng.open_request()
    got = C.run(eng, s, toks, (40, 1, 2))
    assert C.position_errors(got, c.oracle(toks)).max() < C.F32_TOL
    for what, cfg, w in C.planted(c.cfg, c.w):
        e = C.position_errors(got, R.forward(toks, cfg, w)[0])
        assert e.max() > 50 * C.F32_TOL, what


def test_checkpoint_must_fit(tmp_path):
    from shai_amd.engines import trace
    c = C.Case(tmp_path, CPU, F32, seed=12)
    for change in (lambda w: w.pop("l1.mix.g"), lambda w: w.update({"l0.mix.sink": torch.zeros(4)}),
                   lambda w: w.update({"bigram": w["bigram"][:-1]})):
        w = dict(c.w)
        change(w)
        path = R.save_checkpoint(tmp_path / "bad", c.cfg, w)
        with pytest.raises(ValueError, match="does not fit"):
            trace.build_engine(path, "float32", 128, CPU)


def test_registry_and_config(tmp_path):
    from shai_amd.engines.llm import LLMEngine, llama_config_for
    from shai_amd.models.golulix import GolulixConfig, GolulixForCausalLM
    from shai_amd.models.llama import LlamaConfig, LlamaForCausalLM
    from shai_amd.models.registry import config_from_json, model_class
    c = C.Case(tmp_path, CPU, F32, seed=13)
    cfg = llama_config_for("anything", c.path)
    assert isinstance(cfg, GolulixConfig) and model_class(cfg) is GolulixForCausalLM
    assert cfg.order == [(0, False), (1, False), (1, True), (1, True), (2, False)] == R.layer_order(c.cfg)
    assert model_class(LlamaConfig.tiny()) is LlamaForCausalLM
    assert isinstance(llama_config_for("golulix", None, "tiny"), GolulixConfig)
    for bad in (dict(c.cfg, architecture="Other"), dict(c.cfg, loop={"start": 2, "stop": 9, "times": 1}),
                dict(c.cfg, layers=[dict(c.cfg["layers"][0], type="recurrent")])):
        with pytest.raises(ValueError):
            config_from_json(bad)
    with pytest.raises(ValueError):
        LLMEngine(LlamaConfig.tiny(), device=CPU, dtype=torch.float32)
    with pytest.raises(ValueError):
        LLMEngine(GolulixConfig.tiny(), device=CPU, quantization="fp8")


def test_random_init_generates():
    """No checkpoint: deterministic random weights, zero padding, tokens through the scheduler and the sampler."""
    from shai_amd.engines.llm import LLMEngine, SamplingParams
    from shai_amd.models.golulix import GolulixConfig
    mk = lambda: LLMEngine(GolulixConfig.tiny(), device=CPU, max_num_seqs=2, max_model_len=128)
    a, b = mk(), mk()
    assert all(torch.equal(x, y) for x, y in zip(a.model.parameters(), b.model.parameters()))
    p = SamplingParams(max_tokens=6, seed=1)
    out = [s.output for s in a.generate([[1, 2, 3], [7] * 70], p)]
    assert out == [s.output for s in b.generate([[1, 2, 3], [7] * 70], p)] and all(len(o) == 6 for o in out)


def test_trace_replay(tmp_path):
    from shai_amd.engines import trace
    c = C.Case(tmp_path, CPU, F32, seed=14)
    toks, said = c.tokens(32), []
    out = tmp_path / "out"
    out.mkdir()
    eng = trace.build_engine(c.path, "float32", 128, CPU)
    assert eng.num_kv_blocks == 2 and eng.max_num_seqs == 4
    trace.replay(eng, C.replay_lines(c, toks), str(out), said.append)
    C.check_replay_files(c, toks, out, said, F32)


def test_llama_requests_can_be_driven_too():
    """open_request / extend are the engine's, not one model's: Llama logits by portions equal the whole prompt's."""
    from shai_amd.engines.llm import LLMEngine
    from shai_amd.models.llama import LlamaConfig
    eng = LLMEngine(LlamaConfig.tiny(), device=CPU, max_num_seqs=2, max_model_len=192, enable_prefix_caching=False)
    toks = list(range(5, 105))
    a, b = eng.open_request(), eng.open_request()
    whole = eng.extend([(a, toks, list(range(100)))]).float()
    cut = C.run(eng, b, toks, (37, 1, 2, 1))
    assert (whole - cut).abs().max() < 0.05 * whole.abs().max()


def test_serving_api_with_golulix():
    from fastapi.testclient import TestClient
    from shai_amd.serving.common import ServerEnv
    from shai_amd.serving.llm_api import create_app
    env = ServerEnv(app="llm", model_id="golulix", device="cpu", config="tiny", pod_name="p")
    with TestClient(create_app(env=env)) as client:
        r = client.post("/generate", json={"prompt": "hello there", "max_new_tokens": 4})
        assert r.status_code == 200 and r.json()["text"]


def test_bench_option_measures_both_models(monkeypatch):
    from shai_amd.bench import decoder_design as dd
    monkeypatch.setitem(dd.SIZES, "small", (64, 1, 2, 1, 32, 32, 4, 2, 32, 32, 128, 2, 1))
    for cfg in dd.configs("small").values():
        r = dd.measure(cfg, 2, 40, 3, repeats=1, device="cpu")
        assert r["prefill_tok_s"] > 0 and r["decode_tok_s"] > 0
