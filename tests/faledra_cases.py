"""What the CPU and GPU tests of the Faledra decoder share: each case runs the framework's ops, blocks or engine on a device
and compares with ``faledra_reference`` (the oracle recomputes every sequence from its first token)."""
import copy

import decoder_cases
import faledra_reference as R
import torch
from decoder_cases import (F32_TOL, JUNK, Stepper, check_replay_files, close, drive, greedy_oracle, name,  # noqa: F401
                           pad, position_errors, replay_lines, run, run_batches, whole)

from shai_amd.engines.llm import LLMEngine, SamplingParams
from shai_amd.models.blocks import LatentAttention, LatentAttentionConfig, MinGRU, StepShared, XieluMLP
from shai_amd.models.registry import config_from_json
from shai_amd.ops import lm


def assert_logits(got, want, dtype, what=""):
    """Every position (nothing in this design turns a rounding error into a jump)."""
    e = position_errors(got, want)
    assert e.max() < (F32_TOL if dtype == torch.float32 else 0.03), f"{what}: {e.max():.2e} at {int(e.argmax())}"


class Case(decoder_cases.Case):
    ref = R


# ---------------------------------------------------------------------------------------------- mechanisms alone
def check_matmul(device, dtype):
    """The epilogues and forms that the layers use: xIELU, rotation of a part of every head, a plain fp32 product beside
    a main one, products per head over strided rows."""
    g = torch.Generator().manual_seed(1)
    tol = 3e-4 if dtype == torch.float32 else 0.04
    for m, n, k in ((1, 64, 64), (17, 640, 128), (40, 3200, 64), (130, 192, 64), (700, 512, 192)):
        a = torch.randn(m, k, generator=g).to(dtype)
        w = (torch.randn(n, k, generator=g) / k ** 0.5).to(dtype)
        ref = a.double() @ w.double().T
        ad, wd = a.to(device), w.to(device)
        p, q = 0.7, -1.3
        vec = torch.nn.functional.softplus(torch.tensor([p, q])) + torch.tensor([0.0, 0.5])
        y = lm.matmul(ad, wd, torch.float32, lm.EPI_XIELU, vec=vec.to(device))
        close(y, R.xielu(ref, torch.tensor(p).double(), torch.tensor(q).double()), 1e-3, "xielu")
        pos = torch.randint(0, 5000, (m,), generator=g).int()
        for dims, rot0, head in ((2, 0, 64), (6, 24, 64), (64, 0, 64), (20, 40, 64)):
            rope = lm.rope_rows(pos.to(device), lm.rope_freq(900.0, dims).to(device))
            y = lm.matmul(ad, wd, epi=lm.EPI_ROTARY, rope=rope, head=head, rot0=rot0)
            want = ref.view(m, -1, head).clone()
            for t in range(m):
                want[t, :, rot0:rot0 + dims] = R.rotate(want[t:t + 1, :, rot0:rot0 + dims], 900.0, int(pos[t]))[0]
            close(y, want.view(m, n), tol, f"rotary {dims} {rot0}")
        for rows, main in ((n, n // 2 + 4), (n - 3, n // 2 - 4)):
            y, side = lm.matmul_with_side(ad, wd[:rows].contiguous(), rows - main)
            close(y, ref[:, :main], tol, "main")
            close(side, ref[:, main:rows], 3e-4, "side")
    for m, n, k in ((1, 64, 512), (16, 70, 576), (30, 640, 1024), (64, 3000, 640), (50, 130, 832), (65, 200, 1024),
                    (300, 520, 1088), (1000, 128, 2112)):
        a = torch.randn(m, k, generator=g).to(dtype)
        w = (torch.randn(n, k, generator=g) / k ** 0.5).to(dtype)
        y = lm.matmul_parts(a.to(device), w.to(device))
        assert y.dim() == (3 if device != "cpu" and dtype == torch.bfloat16 else 2)
        close(whole(y), a.double() @ w.double().T, 3e-4, "parts")
    for T, H, K, N, head in ((1, 3, 64, 64, 128), (19, 8, 128, 192, 192), (70, 20, 64, 512, 64)):
        a = torch.randn(T, H * head, generator=g).to(dtype)
        w = (torch.randn(H, N + 8, K, generator=g) / K ** 0.5).to(dtype)
        y = lm.matmul_heads(a.to(device).view(T, H, head)[..., :K], w.to(device)[:, 8:])
        want = torch.einsum("thk,hnk->thn", a.double().view(T, H, head)[..., :K], w[:, 8:].double())
        close(y, want, tol, "heads")


def check_rope_rows(device, dtype):
    """Angles of far positions keep their accuracy."""
    pos = torch.tensor([0, 1, 63, 64, 1000, 65535, 131071, 1000003], dtype=torch.int32)
    for base, dims in ((50.0, 2), (10000.0, 12), (1e6, 64)):
        got = lm.rope_rows(pos.to(device), lm.rope_freq(base, dims).to(device)).cpu().double()
        for i, p in enumerate(pos.tolist()):
            pair = torch.zeros(1, dims, dtype=torch.float64)
            pair[:, 0::2] = 1.0                              # (1, 0) turned is (cos, sin)
            close(got[i], R.rotate(pair, base, p)[0], 5e-7, f"{base} {p}")


def check_residual_norm(device, dtype):
    g = torch.Generator().manual_seed(2)
    tol = 2e-5 if dtype == torch.float32 else 0.05
    for T, width in ((1, 50), (9, 700), (5, 2049), (3, 5000)):
        r = lambda *s: torch.randn(*s, generator=g)
        up = lambda t: pad(t).to(device)
        x, d = r(T, width), r(T, width).to(dtype)
        wb, w, step = 1 + 0.3 * r(width), 1 + 0.3 * r(width), r(width)
        table, ids = r(11, width).to(dtype), torch.randint(0, 11, (T,), generator=g).int()
        for source, base in ((up(x), x.double()), (lm.Embedding(ids.to(device), up(table), 3.5), table.double()[ids.long()] * 3.5)):
            for delta, st in ((None, None), (d, None), (d, step), (None, step)):
                want = base.clone()
                if delta is not None:
                    want = want + 0.4 * R.rms_norm(d.double(), wb.double(), 1e-3)
                if st is not None:
                    want = want + step.double()
                src = source.clone() if isinstance(source, torch.Tensor) else source
                args = (None if delta is None else up(d), None if delta is None else up(wb), 0.4, None if st is None else up(step))
                xs, h = lm.residual_norm(src, *args, up(w), 1e-3, width, dtype)
                close(xs[:, :width], want, 2e-5, "x")
                assert not xs[:, width:].any() and not h[:, width:].any()
                close(h[:, :width], R.rms_norm(want, w.double(), 1e-3), tol, "h")
                if delta is not None and device != "cpu":   # the same output as partial sums
                    parts = torch.stack([up(d).float() * 0.5, up(d).float() * 0.25, up(d).float() * 0.25])
                    src = source.clone() if isinstance(source, torch.Tensor) else source
                    xp, hp = lm.residual_norm(src, parts, *args[1:], up(w), 1e-3, width, dtype)
                    close(xp[:, :width], want, 2e-5, "x of parts")
                    close(hp, h.double().cpu(), tol, "h of parts")
                src = source.clone() if isinstance(source, torch.Tensor) else source
                rows = torch.tensor([T - 1, 0, T - 1], dtype=torch.int32, device=device)
                none, h = lm.residual_norm(src, *args, up(w), 1e-3, width, torch.float32 if delta is None and src is not source
                                           else dtype, rows=rows, keep=False)
                assert none is None
                close(h[:, :width], R.rms_norm(want, w.double(), 1e-3)[[T - 1, 0, T - 1]], tol, "rows")
                src = source.clone() if isinstance(source, torch.Tensor) else source
                xs, h = lm.residual_norm(src, *args, None, 1e-3, width, dtype)
                assert h is None
                close(xs[:, :width], want, 2e-5, "no norm")


def check_conv(device, dtype):
    """The input convolution over portions of every size, in batches, with reused state slots: the inputs before a portion
    come from the state, the ones before a sequence's start are zero whatever the slot holds."""
    tol = 3e-5 if dtype == torch.float32 else 0.06
    for width, taps, lengths in ((50, 4, (70, 3, 21, 1)), (130, 1, (9, 4)), (64, 2, (40, 12)), (70, 9, (45, 17, 5)),
                                 (2050, 3, (11, 6)), (48, 16, (40, 30)), (5000, 4, (7, 2)),
                                 (9000, 2, (5, 3))):
        g = torch.Generator().manual_seed(width)
        r = lambda *s: torch.randn(*s, generator=g)
        xs, ds = [r(n, width) for n in lengths], [r(n, width).to(dtype) for n in lengths]
        wb, w, cw = 1 + 0.2 * r(width), 1 + 0.2 * r(width), 0.6 * r(width, taps)
        up = lambda t: pad(t).to(device).contiguous()
        for cuts in ((200,), (1,), (2,), (5, 1, 3, 0), (16, 2)):
            state = torch.full((2, len(lengths) + 2, taps - 1, lm.pad64(width)), JUNK, device=device)

            def fn(batch, rows):
                x, d = (up(torch.stack([t[b][p] for b, p in rows])) for t in (xs, ds))
                tail = (torch.full((2, batch.B, taps - 1, lm.pad64(width)), JUNK, device=device) if batch.is_prefill else None)
                conv = lm.Conv(up(cw.T), state[1], tail[1] if tail is not None else None)
                x, h = lm.residual_norm(x, d, up(wb), 0.7, None, up(w), 1e-4, width, dtype, conv=conv, batch=batch)
                if tail is not None:
                    tail[0] = 5.0
                    lm.conv_commit(state, tail, batch)
                return torch.cat([x, h.float()], 1)

            for turn in range(2):                       # the second turn finds the first one's inputs in the slots
                got = drive(lengths, cuts, device, fn)
                for x, d, y in zip(xs, ds, got):
                    want = x.double() + 0.7 * R.rms_norm(d.double(), wb.double(), 1e-4)
                    close(y[:, :width], want, 3e-5, "x")
                    h = R.rms_norm(want, w.double(), 1e-4)
                    close(y[:, lm.pad64(width):][:, :width], h + R.causal_conv(h, cw.double()), tol, f"{width} {taps} {cuts}")


def latent_block(width, device, dtype, seed=0, eps=1e-4, **sizes):
    cfg = R.random_config([R.attention_layer(**sizes)], width=width, loop=None, eps=eps)
    mc = cfg["layers"][0]["mixer"]
    w = {k[len("l0.mix."):]: v for k, v in R.random_weights(cfg, seed).items() if k.startswith("l0.mix.")}
    c = LatentAttentionConfig(mc["heads"], mc["dim"], mc["rot_dim"], mc["vdim"], mc["q_rank"], mc["kv_rank"], mc["scale"],
                              mc["rot"]["base"])
    m = LatentAttention(width, c, eps, dtype)
    for k, v in m.pack(lambda n: w[n]).items():
        getattr(m, k).copy_(v)
    return mc, w, m.to(device)


def check_latent_attention(device, dtype):
    """The whole mixer, sequences of unequal length in one batch, by portions: latent space and expanded keys agree."""
    for i, sizes in enumerate((dict(), dict(heads=1, dim=64, rot_dim=64, vdim=64, q_rank=64, kv_rank=64),
                               dict(heads=17, dim=24, rot_dim=2, vdim=100, q_rank=20, kv_rank=130, scale=-0.15),
                               dict(heads=2, dim=128, rot_dim=64, vdim=128, q_rank=100, kv_rank=512, scale=0.07),
                               dict(heads=40, dim=16, rot_dim=10, vdim=16, q_rank=70, kv_rank=40),
                               dict(heads=2, dim=130, rot_dim=40, vdim=200, q_rank=70, kv_rank=300, scale=0.06),
                               dict(heads=2, dim=300, rot_dim=12, vdim=30, q_rank=30, kv_rank=600, scale=0.05),
                               dict(heads=3, dim=10, rot_dim=80, vdim=40, q_rank=30, kv_rank=60, scale=0.1))):
        mc, w, m = latent_block(72, device, dtype, i, **sizes)
        lengths = (150, 1, 40, 65)
        g = torch.Generator().manual_seed(i)
        hs = [torch.randn(n, 72, generator=g).bfloat16().float() for n in lengths]
        want = [R.latent_attention(h.double(), mc, 1e-4, lambda n: w[n].double()) for h in hs]
        for cuts, splits in (((200,), 1), ((1,), 3), ((70, 1, 16, 17, 2), 1), ((64, 1, 1, 0), 2)):
            if cuts == (1,) and i > 3:
                continue
            cache = torch.full(m.cache_shape(Stepper(lengths, "cpu").blocks, 64), JUNK, dtype=dtype, device=device)

            def fn(batch, rows):
                h = pad(torch.stack([hs[b][p] for b, p in rows])).to(device, dtype)
                return whole(m(h, batch, cache, StepShared(batch)))[:, :72]

            got = drive(lengths, cuts, device, fn, splits)
            for a, b in zip(got, want):
                close(a / b.std(), b / b.std(), 5e-5 if dtype == torch.float32 else 0.12, f"{sizes} {cuts}")


def attend_step(m, q, c, turn, cuts, device, dtype, splits=1):
    """One sequence's turned queries q [n, H, dim + rot] over its latents c [n, R] and turned key parts [n, rot]."""
    n, H = q.shape[:2]
    cc = m.c
    rows = torch.cat([pad(q[..., :cc.dim], m.np), pad(q[..., cc.dim:], m.dk - m.np)], -1).reshape(n, -1).to(device, dtype)
    line = torch.cat([pad(c, m.rp), pad(turn, m.op)], -1).to(device, dtype)
    blocks = Stepper((n,), "cpu").blocks
    cache = torch.full(m.cache_shape(blocks, 64), JUNK, dtype=dtype, device=device)

    def fn(batch, at):
        t = torch.tensor([p for _, p in at], device=device)
        cache.view(-1, m.rp + m.op)[batch.slots.long()] = line[t]
        return m.attend(rows[t].contiguous(), batch, cache, lm.latent_plan(batch, m.expands))
    return drive((n,), cuts, device, fn, splits)[0].view(n, H, m.dv)[..., :cc.vdim].reshape(n, -1)


def attend_oracle(mc, w, q, c, turn):
    n, H = q.shape[:2]
    k = torch.cat([(c @ w["uk"].double().T).view(n, H, mc["dim"]), turn[:, None].expand(n, H, mc["rot_dim"])], -1)
    v = (c @ w["uv"].double().T).view(n, H, mc["vdim"])
    return R.attend(q, k, v, w["sink"].double(), mc["scale"])


def check_needle(device, dtype):
    """One key whose score stands out, at page borders, at the sequence's ends and far away: every later query copies its
    value, no earlier one sees it; with and without a sink that outweighs it."""
    sizes = dict(heads=2, dim=24, rot_dim=8, vdim=16, kv_rank=32, scale=1.0)
    mc, w, m = latent_block(64, device, dtype, 3, **sizes)
    n = 330
    tol = 1e-4 if dtype == torch.float32 else 0.08
    for at in (0, 1, 2, 62, 63, 64, 65, 127, 128, 255, 256, 313, 328, 329):
        for sink in (0.0, 60.0):
            g = torch.Generator().manual_seed(at)
            r = lambda *s: (torch.randn(*s, generator=g) * 0.3).bfloat16().float()
            q, c, turn = r(n, 2, 32), r(n, 32), r(n, 8)
            w["sink"] = torch.tensor([sink, -3.0])
            m.sink.copy_(w["sink"])
            q[:, :, 24] = 4.0
            turn[:, 0] = 0.0
            turn[at, 0] = 8.0                           # score 32 above the others
            c[at] = 1.0
            want = attend_oracle(mc, w, q.double(), c.double(), turn.double())
            if sink == 0.0:
                v = w["uv"].double().sum(1)
                assert (want[at:] - v).abs().max() < 1e-6
            else:                                       # the first head's sink swallows the needle, the second's does not
                assert want[:, :16].abs().max() < 1e-9 and (want[at:, 16:] - w["uv"].double().sum(1)[16:]).abs().max() < 1e-6
            for cuts, splits in (((n,), 1), ((64, 1, 5), 3)) if at % 2 else (((17, 16, 1, 1, 90), 1), ((300, 1), 5)):
                close(attend_step(m, q, c, turn, cuts, device, dtype, splits), want, tol, f"{at} {sink} {cuts}")


def check_low_scores(device, dtype):
    """Scores far below zero and sinks far below or above them, in one to many splits of a decode step, some empty."""
    mc, w, m = latent_block(64, device, dtype, 4, heads=3, dim=16, rot_dim=8, vdim=16, kv_rank=40, scale=1.0)
    n = 450
    g = torch.Generator().manual_seed(17)
    r = lambda *s: torch.randn(*s, generator=g).bfloat16().float()
    q, c, turn = r(n, 3, 24), r(n, 40), r(n, 8)
    q[..., 16], turn[:, 0] = 8.0, -8.0
    turn[:, 1] -= torch.arange(n) * 0.02                # the splits' maxima differ
    turn = turn.bfloat16().float()
    w["sink"] = torch.tensor([-300.0, -60.0, -64.0])
    m.sink.copy_(w["sink"])
    want = attend_oracle(mc, w, q.double(), c.double(), turn.double())
    for splits in (1, 2, 3, 5, 7, 16):
        got = attend_step(m, q, c, turn, (430, 1, 3, 1), device, dtype, splits)
        # the first token's heads have their only key beside the sink
        close(got, want, 2e-4 if dtype == torch.float32 else 0.12, str(splits))


def check_scan(device, dtype):
    """The recurrence over portions and chunks of them, in batches, with reused slots; slow gates carry the first token's
    contribution to the end."""
    tol = 2e-5 if dtype == torch.float32 else 0.02
    for W, lengths in ((64, (200, 1, 65, 129)), (128, (70, 64, 3))) + (((192, (4500, 260)),) if device != "cpu" else ()):
        g = torch.Generator().manual_seed(W)
        r = lambda *s: torch.randn(*s, generator=g)
        bias = torch.cat([r(W) - 3.0, r(W)])
        bias[0], bias[1], bias[2] = -12.0, 12.0, 0.0    # a channel that keeps, one that forgets
        zx, gs = [r(n, 2 * W) * 2 for n in lengths], [r(n, W).to(dtype) for n in lengths]
        for t in zx:
            t[0, 0], t[0, W] = 30.0, 4.0                # the keeping channel takes the first token in
        want = []
        for a, b in zip(zx, gs):
            z, u = (a + bias).double().chunk(2, 1)
            S = R.mingru_states(z, u)
            assert S[min(199, len(S) - 1), 0] > 2.0
            want.append(S * b.double() * torch.sigmoid(b.double()))
        for cuts in ((5000,), (1,), (2, 3), (64, 1, 65, 0), (130, 7)):
            if max(lengths) > 1000 and cuts[0] < 64:
                continue
            state = torch.full((len(lengths) + 2, W), JUNK, device=device)

            def fn(batch, rows):
                pick = lambda ts: torch.stack([ts[b][p] for b, p in rows]).to(device)
                return lm.mingru_scan(pick(zx), pick(gs), bias.to(device), state, batch)
            for turn in range(2):
                for a, b in zip(drive(lengths, cuts, device, fn), want):
                    close(a, b, tol * max(1.0, float(b.abs().max())), f"{W} {cuts}")


def check_blocks(device, dtype):
    """minGRU and feed-forward as blocks, at sizes that need padding."""
    for width, size, ff, n in ((50, 30, 70, 90), (128, 200, 64, 33)):
        cfg = R.random_config([R.mingru_layer(size, ff)], width=width, loop=None)
        w = R.random_weights(cfg, n)
        g = torch.Generator().manual_seed(n)
        h = torch.randn(n, width, generator=g).bfloat16().float()
        tol = 1e-4 if dtype == torch.float32 else 0.1
        m = MinGRU(width, size, dtype)
        for k, v in m.pack(lambda name: w["l0.mix." + name]).items():
            getattr(m, k).copy_(v)
        m.to(device)
        state = torch.full((3, m.sp), JUNK, device=device)
        fn = lambda batch, rows: whole(m(pad(h[[p for _, p in rows]]).to(device, dtype), batch, state))[:, :width]
        want = R.mingru(h.double(), lambda name: w["l0.mix." + name].double())
        for cuts in ((n,), (13, 1, 1)):
            close(drive((n,), cuts, device, fn)[0] / want.std(), want / want.std(), tol, "mingru")
        f = XieluMLP(width, ff, dtype)
        for k, v in f.pack(lambda name: w["l0.mlp." + name]).items():
            getattr(f, k).copy_(v)
        want = R.feed_forward(h.double(), lambda name: w["l0.mlp." + name].double())
        close(whole(f.to(device)(pad(h).to(device, dtype)))[:, :width] / want.std(), want / want.std(), tol, "xielu")


MECHANISMS = [check_matmul, check_rope_rows, check_residual_norm, check_conv, check_latent_attention, check_needle,
              check_low_scores, check_scan, check_blocks]

# ---------------------------------------------------------------------------------------------- whole models
A, G = R.attention_layer, R.mingru_layer
SHAPES = {
    "base": {},
    "attention_only": dict(layers=[A(), A(heads=5, dim=64, vdim=64, kv_rank=64, rot_dim=64)], loop=(0, 2, 3), taps=2),
    "mingru_only": dict(layers=[G(), G(64), G(20)], loop=(2, 3, 2), taps=5, width=64),
    "one_layer_one_tap": dict(layers=[A(heads=1)], loop=None, taps=1),
    "no_mlp": dict(layers=[A(ff=0), G(ff=0), A()], loop=(0, 1, 2), width=100, vocab=33),
    "no_mlp_last": dict(layers=[G(), A(ff=0)], loop=(1, 2, 2)),
    "whole_loop_once": dict(layers=[G(70, 90), A()], loop=(0, 2, 1), mult=1.0, embed_scale=1.0),
    "big_heads": dict(layers=[A(heads=2, dim=136, vdim=200, rot_dim=24, kv_rank=260)], loop=(0, 1, 2), width=72),
    "many_heads": dict(layers=[A(heads=36, dim=8, vdim=8, rot_dim=4), G()], loop=None, taps=9),
    "any_size": dict(layers=[A(heads=2, dim=270, vdim=20, rot_dim=70, kv_rank=520, scale=0.04)], loop=None),
    "negative_scale": dict(layers=[A(scale=-0.3), A(base=1e6)], loop=None, mult=0.2),
}


def check_shape(tmp, device, dtype, key):
    c = Case(tmp, device, dtype, seed=len(key), **SHAPES[key])
    eng = c.engine(256)
    toks = c.tokens(140)
    want = c.oracle(toks)
    for cuts in ((140,), (61, 1, 1, 2, 1)):
        s = eng.open_request()
        assert_logits(run(eng, s, toks, cuts), want, dtype, f"{key} {cuts}")
        eng.close_request(s)


def check_layers(tmp, device, dtype):
    """The residual stream after every layer run."""
    c = Case(tmp, device, dtype, seed=3)
    eng = c.engine()
    toks = c.tokens(50)
    s = eng.open_request()
    eng._ensure_blocks(s, len(toks))
    s.prompt = toks
    trail = []
    with torch.inference_mode():
        eng.model(eng._packed_batch([s], [len(toks)]), eng.kv, trail)
    want = R.forward(toks, c.cfg, c.w)[1]
    assert len(trail) == len(want) == 6
    for a, b in zip(trail, want):
        close(a / b.abs().max(), b / b.abs().max(), 1e-5 if dtype == torch.float32 else 0.03)


def check_portions(tmp, device, dtype):
    c = Case(tmp, device, dtype, seed=4)
    eng = c.engine()
    toks = c.tokens(150)
    want = c.oracle(toks)
    for cuts in ((150,), (2,), (3,), (64,), (1,), (63, 2, 1, 65), (16, 17, 1, 1, 44), (149, 1)):
        s = eng.open_request()
        assert_logits(run(eng, s, toks, cuts), want, dtype, str(cuts))
        eng.close_request(s)


def check_long_decode(tmp, device, dtype):
    """Decoding over many pages, token by token."""
    c = Case(tmp, device, dtype, seed=5, layers=[A(), G()], loop=(0, 1, 2))
    eng = c.engine(640)
    toks = c.tokens(420)
    s = eng.open_request()
    assert_logits(run(eng, s, toks, (5,) + (1,) * 500), c.oracle(toks), dtype)


def check_batches(tmp, device, dtype):
    c = Case(tmp, device, dtype, seed=6)
    eng = c.engine(512)
    run_batches(c, eng, {f"q{i}": c.tokens(n) for i, n in enumerate((130, 1, 75, 64, 2, 190, 33, 128))}, assert_logits)
    assert eng.state_slots.num_free == eng.max_num_seqs


def check_slots(tmp, device, dtype):
    """A state slot that is used again, and a request that pauses while others run: neither leaks into the other."""
    c = Case(tmp, device, dtype, seed=7, layers=[G(), A()], loop=(0, 1, 2), taps=4)
    eng = c.engine(256)
    a, b = c.tokens(90), c.tokens(60)
    wa, wb = c.oracle(a), c.oracle(b)
    sa = eng.open_request()
    assert_logits(run(eng, sa, a[:50], (50,)), wa[:50], dtype)
    for first in (1, 2, 3, 60):
        sb = eng.open_request()
        assert_logits(run(eng, sb, b, (first, 1, 9)), wb, dtype, str(first))
        slot = sb.state_slot
        eng.close_request(sb)
        again = eng.open_request()
        assert again.state_slot == slot                # the junk of the request before is in it
        eng.close_request(again)
    assert_logits(run(eng, sa, a[50:], (1, 2, 1)), wa[50:], dtype)
    eng.close_request(sa)
    assert len([eng.open_request() for _ in range(4)]) == 4
    try:
        eng.open_request()
        raise AssertionError("accepted")
    except MemoryError:
        pass


def check_greedy(tmp, device, dtype, **kw):
    """Greedy generation through the engine's scheduler: chunked prefill, mixed steps, look-ahead decode, and (small pool)
    preemption."""
    c = Case(tmp, device, dtype, seed=8, layers=[A(), G()], loop=(0, 1, 2))
    shared = c.tokens(64)
    prompts = [shared + c.tokens(30), c.tokens(3), shared + c.tokens(5), c.tokens(100), c.tokens(1)]
    eng = LLMEngine(config_from_json(c.cfg), device=device, model_path=c.path, max_num_seqs=4, max_model_len=192,
                    dtype=dtype, prefill_chunk=64, **kw)
    params = SamplingParams(temperature=0.0, max_tokens=20)
    for turn in range(2):                               # a common prefix is not shared: its state would be missing
        outs = eng.generate(prompts, params)
        for p, s in zip(prompts, outs):
            toks = (s.prompt + s.output)[len(p):]
            assert len(toks) == 20
            if dtype == torch.float32:
                assert toks == greedy_oracle(c, p, 20)
            else:                                       # every choice is at (or within rounding of) the maximum
                lg = c.oracle(p + toks)[len(p) - 1:-1]
                gap = lg.max(-1).values - lg.gather(1, torch.tensor(toks)[:, None])[:, 0]
                assert (gap / lg.std() < 0.1).all()
    assert eng.stats["prefix_hit_tokens"] == 0
    assert eng.bm.num_free == eng.num_kv_blocks and eng.state_slots.num_free == 4


def check_sampling(tmp, device, dtype):
    """A seeded request draws the same tokens alone and in a batch."""
    c = Case(tmp, device, dtype, seed=9, layers=[G(), A()], loop=None)
    cfg = config_from_json(c.cfg)
    p = SamplingParams(temperature=0.8, top_k=12, top_p=0.95, max_tokens=12, seed=5)
    mk = lambda: LLMEngine(cfg, device=device, model_path=c.path, max_num_seqs=4, max_model_len=128, dtype=dtype)
    prompts = [c.tokens(n) for n in (9, 40, 2)]
    alone = mk().generate([prompts[0]], p)[0].output
    assert mk().generate(prompts, p)[0].output == alone and len(set(alone)) > 1


def check_far_token(tmp, device, dtype):
    """The first token reaches the last position: through attention over several pages, through the recurrence, and both
    by portions; a model that drops it would be noticed."""
    for layers in ([A(heads=2, scale=0.3)], [G(64)]):
        c = Case(tmp, device, dtype, seed=10 + len(layers[0]["mixer"]), layers=layers, loop=None, vocab=40, taps=2)
        for k in c.w:
            if k.endswith("mix.z.b"):
                c.w[k] = c.w[k] * 0 - 5.0               # gates that hardly open
            if k.endswith("mix.z"):
                c.w[k] = (c.w[k] * 0.5).bfloat16().float()
        c.w["embed"][7] *= 8.0
        if layers[0]["type"] == "latent_attention":
            c.w["l0.mix.sink"] = (c.w["l0.mix.sink"] - 4.0).bfloat16().float()
        c.path = R.save_checkpoint(tmp / "far", c.cfg, c.w)
        toks = [7] + [t if t != 7 else 8 for t in c.tokens(199)]
        want = c.oracle(toks)
        eng = c.engine(256)
        for cuts in ((200,), (100, 1), (1, 63, 1, 1)):
            s = eng.open_request()
            assert_logits(run(eng, s, toks, cuts), want, dtype, str(cuts))
            eng.close_request(s)
        other = c.oracle([8] + toks[1:])
        assert position_errors(other[-1:], want[-1:]).max() > 10 * F32_TOL


MODELS = [check_layers, check_portions, check_long_decode, check_batches, check_slots, check_sampling, check_far_token]


def planted(cfg, w):
    """(what, config, weights) with one mistake each, for the oracle: the comparison must notice every one."""
    def changed(f):
        c, v = copy.deepcopy(cfg), dict(w)
        f(c, v)
        return c, v

    def weights(end, fn):
        return lambda c, v: v.update({k: fn(t) for k, t in v.items() if k.endswith(end)})

    def mixers(kind, fn):
        return lambda c, v: [fn(lc["mixer"]) for lc in c["layers"] if lc["type"] == kind]
    att = "latent_attention"
    yield ("embedding scale",) + changed(lambda c, v: c["embedding"].update(scale=1.0))
    yield ("residual multiplier",) + changed(lambda c, v: c.update(residual_mult=1.0))
    yield ("eps",) + changed(lambda c, v: c["norm"].update(eps=0.02))
    yield ("no loop",) + changed(lambda c, v: c.update(loop=None))
    yield ("one pass too many",) + changed(lambda c, v: (c["loop"].update(times=3), v.update(
        {"loop.step": torch.cat([v["loop.step"], v["loop.step"][:1]])})))
    yield ("step vectors swapped",) + changed(weights("loop.step", lambda t: t.flip(0)))
    yield ("step only between passes",) + changed(weights("loop.step", lambda t: torch.cat([t[:1] * 0, t[1:]])))
    yield ("no convolution",) + changed(weights("canon1", lambda t: t * 0))
    yield ("convolution reversed",) + changed(weights("canon1", lambda t: t.flip(1)))
    yield ("convolution one tap short",) + changed(weights("canon1", lambda t: torch.cat([t[:, :1] * 0, t[:, 1:]], 1)))
    yield ("no post norm gain",) + changed(weights("norm1b", lambda t: t * 0 + 1))
    yield ("no second post norm gain",) + changed(weights("norm2b", lambda t: t * 0 + 1))
    yield ("sink left out",) + changed(weights("sink", lambda t: t * 0 - 1e4))
    yield ("sink of zero",) + changed(weights("sink", lambda t: t * 0))
    yield ("scale",) + changed(mixers(att, lambda m: m.update(scale=m["scale"] * 1.1)))
    yield ("rotation base",) + changed(mixers(att, lambda m: m["rot"].update(base=1e4)))
    yield ("no query latent gain",) + changed(weights("dq.norm", lambda t: t * 0 + 1))
    yield ("no latent gain",) + changed(weights("dkv.norm", lambda t: t * 0 + 1))
    yield ("activation numbers swapped",) + changed(weights("mlp.act", lambda t: t.flip(0)))
    yield ("gate bias left out",) + changed(weights("mix.z.b", lambda t: t * 0))
    yield ("candidate bias left out",) + changed(weights("mix.x.b", lambda t: t * 0))
