"""Pugozen on the CPU references: the engine integration (registry, loader, cache, state slots, scheduler, sampling, trace
replay) against the plain oracle, and that the comparison notices a planted mistake."""
import copy

import pugozen_cases as C
import pugozen_reference as R
import pytest
import torch

CPU, F32, BF16 = "cpu", torch.float32, torch.bfloat16


@pytest.mark.parametrize("check", C.MECHANISMS, ids=lambda f: f.__name__)
def test_mechanism(check):
    check(CPU, F32)


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


def test_checkpoint_must_fit(tmp_path):
    from shai_amd.engines import trace
    c = C.Case(tmp_path, CPU, F32, seed=12)
    for change in (lambda w: w.pop("l0.mix.left.sink"), lambda w: w.update({"l3.norm1": w["l0.norm1"]}),
                   lambda w: w.update({"l1.mix.q.conv": w["l1.mix.q.conv"][:, 1:]}), lambda w: w.pop("l0.mix.right.a1"),
                   lambda w: w.update({"l0.mix.right.a1": w["l0.mix.right.a1"][1:]})):
        w = dict(c.w)
        change(w)
        path = R.save_checkpoint(tmp_path / "bad", c.cfg, w)
        with pytest.raises(ValueError, match="does not fit"):
            trace.build_engine(path, "float32", 128, CPU)


def test_registry_and_config(tmp_path):
    from shai_amd.engines.llm import LLMEngine, llama_config_for
    from shai_amd.models.pugozen import PugozenConfig, PugozenForCausalLM
    from shai_amd.models.registry import config_from_json, model_class
    c = C.Case(tmp_path, CPU, F32, seed=13)
    cfg = llama_config_for("anything", c.path)
    assert isinstance(cfg, PugozenConfig) and model_class(cfg) is PugozenForCausalLM
    assert cfg.order == [0, 1, 2, 0, 1] and cfg.layers[0].mixer[1].ranks == (10, 14)
    assert isinstance(llama_config_for("pugozen", None, "tiny"), PugozenConfig)
    chain = copy.deepcopy(c.cfg)
    chain["layers"].append(dict(chain["layers"][0], weights_of=3))
    assert config_from_json(chain).order[-1] == 0

    def changed(i, fn):
        layers = copy.deepcopy(c.cfg["layers"])
        fn(layers[i])
        return dict(c.cfg, layers=layers)
    for bad in (changed(3, lambda x: x.update(weights_of=1)), changed(3, lambda x: x.update(weights_of=3)),
                changed(3, lambda x: x.update(weights_of=9)), changed(3, lambda x: x["mixer"].update(left_scale=9.0)),
                changed(0, lambda x: x["mixer"]["left"].update(kv_heads=4)), changed(0, lambda x: x["mixer"]["left"].update(vdim=5)),
                changed(0, lambda x: x["mixer"]["left"]["rot"].update(dims=7)), changed(1, lambda x: x["mixer"].update(kv_heads=4)),
                changed(1, lambda x: x["mixer"].update(conv=17)), changed(2, lambda x: x["mixer"].update(heads=4)),
                changed(2, lambda x: x["mixer"].update(decay=[0.5, 0.5, 1.5])), changed(2, lambda x: x["mixer"]["rot"].update(dims=40)),
                changed(2, lambda x: x.update(type="recurrent")), changed(1, lambda x: x["mlp"].update(kind="moe")),
                changed(1, lambda x: x["mixer"].update(dim=300)), dict(c.cfg, layers=[])):
        with pytest.raises(ValueError):
            cfg = config_from_json(bad)
            model_class(cfg)(cfg, F32)
    with pytest.raises(ValueError):
        LLMEngine(PugozenConfig.tiny(), device=CPU, quantization="fp8")


def test_shared_weights_keep_their_own_memory():
    """A layer with another one's weights has no parameters, but a cache and a state of its own."""
    from shai_amd.models.pugozen import PugozenConfig, PugozenForCausalLM
    sizes = (64, 4, 2, 32, 2, 1, 24, 40, 8, 64, 50)
    one, two = (PugozenForCausalLM(PugozenConfig.uniform(k, *sizes)) for k in ("PD", "PDpd"))
    count = lambda m: sum(p.numel() for p in m.parameters())
    assert count(one) == count(two) and 2 * one.cache_bytes_per_block() == two.cache_bytes_per_block() > 0
    kv, _ = two.allocate_cache(3, CPU)
    assert kv[0][0] is not kv[2][0] and kv[1] is None
    states = two.allocate_state(2, CPU)
    assert len({t.data_ptr() for s in states for t in s}) == 8


def test_random_init_generates():
    """No checkpoint: deterministic random weights, zero padding, tokens through the scheduler and the sampler."""
    from shai_amd.engines.llm import LLMEngine, SamplingParams
    from shai_amd.models.pugozen import PugozenConfig
    mk = lambda: LLMEngine(PugozenConfig.tiny(), device=CPU, max_num_seqs=2, max_model_len=128)
    a, b = mk(), mk()
    assert all(torch.equal(x, y) for x, y in zip(a.model.parameters(), b.model.parameters()))
    p = SamplingParams(max_tokens=6, seed=1)
    out = [s.output for s in a.generate([[1, 2, 3], [7] * 70], p)]
    assert out == [s.output for s in b.generate([[1, 2, 3], [7] * 70], p)] and all(len(o) == 6 for o in out)


def test_aborted_requests_give_slots_back():
    from shai_amd.engines.llm import LLMEngine
    from shai_amd.models.pugozen import PugozenConfig
    eng = LLMEngine(PugozenConfig.tiny(), device=CPU, max_num_seqs=2, max_model_len=128)
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


def test_serving_api_with_pugozen():
    from fastapi.testclient import TestClient
    from shai_amd.serving.common import ServerEnv
    from shai_amd.serving.llm_api import create_app
    env = ServerEnv(app="llm", model_id="pugozen", device="cpu", config="tiny", pod_name="p")
    with TestClient(create_app(env=env)) as client:
        r = client.post("/generate", json={"prompt": "hello there", "max_new_tokens": 4})
        assert r.status_code == 200 and r.json()["text"]


def test_bench_option_measures_every_model(monkeypatch):
    from shai_amd.bench import decoder_design as dd
    monkeypatch.setitem(dd.PUGOZEN_SIZES, "small", ("PDRp", 64, 2, 1, 32, 2, 1, 32, 32, 16, 96, 128))
    cfgs = dd.configs("small", "pugozen")
    assert list(cfgs) == ["pugozen", "nalizen", "llama"]
    for cfg in cfgs.values():
        r = dd.measure(cfg, 2, 40, 3, repeats=1, device="cpu")
        assert r["prefill_tok_s"] > 0 and r["decode_tok_s"] > 0


def test_segments_of_prompts():
    """Whole chunks, at least four to a segment; both scans of a cut prompt are shorter than one over all of it, and the first
    one's workgroups run at once."""
    for retention in (False, True):
        for scans in (1, 3, 16, 32, 64, 100, 256, 5000):
            for rows in (1, 31, 384, 385, 1000, 1024, 8192, 100000):
                seg = C.lm.rule_segment(rows, scans, retention)
                if not seg:
                    continue
                cuts = -(-rows // seg)
                assert seg % C.lm.RULE_CHUNK == 0 and seg >= 4 * C.lm.RULE_CHUNK and cuts >= 3 and 2 * seg < rows
                assert scans * ((cuts - 1) if retention else 2 * cuts - 3) <= 256
    assert C.lm.rule_segment(8192, 16, False) == 928 and C.lm.rule_segment(8192, 16, True) == 512
    assert not C.lm.rule_segment(1024, 128, False) and not C.lm.rule_segment(100, 1, True)
