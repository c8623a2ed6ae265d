"""Faledra on the CPU references: the engine integration (registry, loader, cache, state slots, scheduler, sampling, trace
replay) against the plain oracle, and that the comparison notices a planted mistake."""
import faledra_cases as C
import faledra_reference as R
import pytest
import torch

CPU, F32, BF16 = "cpu", torch.float32, torch.bfloat16


@pytest.mark.parametrize("check", C.MECHANISMS, ids=lambda f: f.__name__)
def test_mechanism(check):
    check(CPU, F32)


@pytest.mark.parametrize("check", [C.check_latent_attention, C.check_needle, C.check_blocks], ids=lambda f: f.__name__)
def test_mechanism_bf16(check):
    """Long portions expand their keys and values in a bf16 model only."""
    check(CPU, BF16)


@pytest.mark.parametrize("key", sorted(C.SHAPES))
def test_shapes(tmp_path, key):
    C.check_shape(tmp_path, CPU, F32, key)


@pytest.mark.parametrize("check", C.MODELS, ids=lambda f: f.__name__)
def test_model(tmp_path, check):
    check(tmp_path, CPU, F32)


def test_model_bf16(tmp_path):
    C.check_batches(tmp_path, CPU, BF16)


@pytest.mark.parametrize("kw", [{}, {"async_decode": False}, {"mixed_steps": False}, {"num_kv_blocks": 7}],
                         ids=["default", "sync", "unmixed", "preempt"])
def test_greedy_generation(tmp_path, kw):
    C.check_greedy(tmp_path, CPU, F32, **kw)


def test_planted_mistakes_show(tmp_path):
    c = C.Case(tmp_path, CPU, F32, seed=11)
    toks = c.tokens(64)
    eng = c.engine()
    got = C.run(eng, eng.open_request(), toks, (40, 1, 2))
    assert C.position_errors(got, c.oracle(toks)).max() < C.F32_TOL
    for what, cfg, w in C.planted(c.cfg, c.w):
        e = C.position_errors(got, R.forward(toks, cfg, w)[0])
        assert e.max() > 50 * C.F32_TOL, what


def test_long_portions_in_groups(monkeypatch):
    """Contexts that are too long to be expanded at once run in several groups."""
    monkeypatch.setattr(C.lm, "LATENT_GROUP_ROWS", 100)
    C.check_latent_attention(CPU, BF16)
    batch, _ = C.Stepper((90, 80, 5, 20), CPU).step((90, 80, 5, 20))
    plan = C.lm.latent_plan(batch, True)
    assert [g.seqs.tolist() for g in plan.groups] == [[0], [1, 3]] and plan.n == 5 and plan.seqs.tolist() == [2] * 5
    assert plan.groups[1].q_start.tolist() == [90, 175] and plan.groups[1].kv_start.tolist() == [0, 80]


def test_checkpoint_must_fit(tmp_path):
    from shai_amd.engines import trace
    c = C.Case(tmp_path, CPU, F32, seed=12)
    for change in (lambda w: w.pop("l1.mix.sink"), lambda w: w.update({"l0.mix.sink": torch.zeros(4)}),
                   lambda w: w.update({"loop.step": w["loop.step"][:-1]})):
        w = dict(c.w)
        change(w)
        path = R.save_checkpoint(tmp_path / "bad", c.cfg, w)
        with pytest.raises(ValueError, match="does not fit"):
            trace.build_engine(path, "float32", 128, CPU)


def test_registry_and_config(tmp_path):
    from shai_amd.engines.llm import LLMEngine, llama_config_for
    from shai_amd.models.faledra import FaledraConfig, FaledraForCausalLM
    from shai_amd.models.registry import config_from_json, model_class
    c = C.Case(tmp_path, CPU, F32, seed=13)
    cfg = llama_config_for("anything", c.path)
    assert isinstance(cfg, FaledraConfig) and model_class(cfg) is FaledraForCausalLM
    assert cfg.order == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)] == R.layer_order(c.cfg)
    assert isinstance(llama_config_for("faledra", None, "tiny"), FaledraConfig)
    att = c.cfg["layers"][1]
    for bad in (dict(c.cfg, loop={"start": 2, "stop": 9, "times": 1}), dict(c.cfg, canon={"taps": 99}),
                dict(c.cfg, layers=[dict(att, type="recurrent")]),
                dict(c.cfg, layers=[dict(att, mixer=dict(att["mixer"], rot_dim=7))]),
                dict(c.cfg, layers=[dict(att, mlp={"kind": "moe"})])):
        with pytest.raises(ValueError):
            cfg = config_from_json(dict(bad, loop=bad["loop"] if bad is not None and len(bad["layers"]) > 1 else None))
            model_class(cfg)(cfg, F32)
    with pytest.raises(ValueError):
        LLMEngine(FaledraConfig.tiny(), device=CPU, quantization="fp8")


def test_random_init_generates():
    """No checkpoint: deterministic random weights, zero padding, tokens through the scheduler and the sampler."""
    from shai_amd.engines.llm import LLMEngine, SamplingParams
    from shai_amd.models.faledra import FaledraConfig
    mk = lambda: LLMEngine(FaledraConfig.tiny(), device=CPU, max_num_seqs=2, max_model_len=128)
    a, b = mk(), mk()
    assert all(torch.equal(x, y) for x, y in zip(a.model.parameters(), b.model.parameters()))
    p = SamplingParams(max_tokens=6, seed=1)
    out = [s.output for s in a.generate([[1, 2, 3], [7] * 70], p)]
    assert out == [s.output for s in b.generate([[1, 2, 3], [7] * 70], p)] and all(len(o) == 6 for o in out)


def test_aborted_requests_give_slots_back():
    from shai_amd.engines.llm import LLMEngine
    from shai_amd.models.faledra import FaledraConfig
    eng = LLMEngine(FaledraConfig.tiny(), device=CPU, max_num_seqs=2, max_model_len=128)
    for _ in range(3):
        eng.add_request([1, 2, 3])
    eng.step()
    assert eng.state_slots.num_free == 0
    eng.abort_all()
    assert eng.state_slots.num_free == 2 and eng.bm.num_free == eng.num_kv_blocks


def test_trace_replay(tmp_path):
    from shai_amd.engines import trace
    c = C.Case(tmp_path, CPU, F32, seed=14)
    toks, said = c.tokens(32), []
    out = tmp_path / "out"
    out.mkdir()
    eng = trace.build_engine(c.path, "float32", 128, CPU)
    assert eng.num_kv_blocks == 2 and eng.max_num_seqs == 4 and eng.state_slots.num_free == 4
    trace.replay(eng, C.replay_lines(c, toks), str(out), said.append)
    C.check_replay_files(c, toks, out, said, F32)


def test_serving_api_with_faledra():
    from fastapi.testclient import TestClient
    from shai_amd.serving.common import ServerEnv
    from shai_amd.serving.llm_api import create_app
    env = ServerEnv(app="llm", model_id="faledra", device="cpu", config="tiny", pod_name="p")
    with TestClient(create_app(env=env)) as client:
        r = client.post("/generate", json={"prompt": "hello there", "max_new_tokens": 4})
        assert r.status_code == 200 and r.json()["text"]


def test_bench_option_measures_both_models(monkeypatch):
    from shai_amd.bench import decoder_design as dd
    monkeypatch.setitem(dd.FALEDRA_SIZES, "small", (64, 1, 1, 2, 32, 16, 32, 48, 64, 64, 96, 128, 1))
    for cfg in dd.configs("small", "faledra").values():
        r = dd.measure(cfg, 2, 40, 3, repeats=1, device="cpu")
        assert r["prefill_tok_s"] > 0 and r["decode_tok_s"] > 0
