"""What the CPU and GPU tests of the Pugozen decoder share: each case runs the framework's ops, blocks or engine on a device
and compares with ``pugozen_reference`` (the oracle recomputes every sequence from its first token)."""
import copy

import decoder_cases
import pugozen_reference as R
import torch
from decoder_cases import (F32_TOL, JUNK, Stepper, assert_logits, check_replay_files, close, drive,  # noqa: F401
                           greedy_oracle, name, pad, position_errors, replay_lines, run, run_batches, whole)

from shai_amd.engines.llm import LLMEngine, SamplingParams
from shai_amd.models.blocks import (DeltaRule, DeltaRuleConfig, JointLayer, Retention, RetentionConfig, StepShared, TiedAttention,
                                    TiedAttentionConfig)
from shai_amd.models.registry import config_from_path
from shai_amd.ops import lm

D, T, P = R.delta_layer, R.retention_layer, R.parallel_layer


class Case(decoder_cases.Case):
    ref = R


def joint(layers, i, width, eps, w, dtype, device):
    """Layer i of a random config as a framework block with its weights."""
    lc = layers[i]
    m = lc["mixer"]
    ranks = tuple(w[f"l{i}.mix.right.{n}"].shape[0] for n in ("a1", "g1")) if lc["type"] == "parallel" else None
    rule = lambda m, **kw: DeltaRule(width, DeltaRuleConfig(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], **kw),
                                     eps, dtype)
    if lc["type"] == "delta":
        mixers = {"only": rule(m)}
    elif lc["type"] == "retention":
        mixers = {"only": Retention(width, RetentionConfig(tuple(m["decay"]), m["dim"], m["vdim"], m["rot"]["dims"],
                                                           m["rot"]["base"]), eps)}
    else:
        a = m["left"]
        mixers = {"left": TiedAttention(width, TiedAttentionConfig(a["heads"], a["kv_heads"], a["dim"], a["scale"], a["rot"]["dims"],
                                                                   a["rot"]["base"], m["left_scale"]), eps),
                  "right": rule(m["right"], ranks=ranks, gate=lm.GATE_SIGMOID, out_scale=m["right_scale"])}
    block = JointLayer(width, mixers, lc["mlp"]["ff"] if lc.get("mlp") else 0, dtype)
    for k, v in block.pack_all(lambda n: w[f"l{i}.{n}"]).items():
        block.get_parameter(k).copy_(v)
    return block.to(device)


def memory(block, blocks, slots, dtype, device):
    """(cache, state) of a block, full of junk."""
    junk = lambda shape, dt: torch.full(shape, JUNK, dtype=dt, device=device)
    cache = block.cache_shapes(blocks, 64)
    state = block.state_shapes()
    return (cache and tuple(junk(s, dtype) for s in cache),
            state and [junk((slots, *s), torch.float32 if f32 else dtype) for s, f32 in state])


# ---------------------------------------------------------------------------------------------- mechanisms alone
def check_matmul(device, dtype):
    """One product with a squared-ReLU part, a plain part and an fp32 part, into rows of a wider buffer, and products over
    such rows, whole and as partial sums."""
    g = torch.Generator().manual_seed(1)
    tol = 3e-4 if dtype == torch.float32 else 0.04
    for m, act, plain, side, k in ((1, 64, 64, 4, 64), (3, 0, 128, 5, 128), (17, 192, 640, 0, 128), (40, 64, 320, 3, 64), (64, 4032, 128, 12, 256),
                                   (130, 128, 64, 7, 192), (700, 192, 448, 33, 128), (66, 64, 64, 2, 1024)):
        a = torch.randn(m, k, generator=g).to(dtype)
        w = (torch.randn(act + plain + side, k, generator=g) * 1.5 / k ** 0.5).to(dtype)
        ref, n = a.double() @ w.double().T, act + plain
        rows = torch.full((m, 64 + n + 64), JUNK, dtype=dtype, device=device)
        s = lm.matmul_joint(a.to(device), w.to(device), rows[:, 64:64 + n], act, side)
        close(rows[:, 64:64 + act], torch.relu(ref[:, :act]) ** 2, 5 * tol, "relu2") if act else None
        close(rows[:, 64 + act:64 + n], ref[:, act:n], 3 * tol, "plain")
        assert (s is None) == (side == 0)
        if side:
            close(s, ref[:, n:], 3e-4 if dtype == torch.float32 else 3e-3, "fp32 part")
        assert (rows[:, :64] == JUNK).all() and (rows[:, 64 + n:] == JUNK).all()
        v = (torch.randn(96, n, generator=g) / n ** 0.5).to(dtype)
        back = rows[:, 64:64 + n]
        close(whole(lm.matmul_parts(back, v.to(device))) / 2, back.double().cpu() @ v.double().T / 2, tol, "strided")


def check_norm(device, dtype):
    """A sublayer's output added without a norm: whole, as partial sums, absent; single rows."""
    g = torch.Generator().manual_seed(2)
    for n, width in ((1, 50), (9, 700), (5, 2049)):
        r = lambda *s: torch.randn(*s, generator=g)
        up = lambda t: pad(t).to(device).contiguous()
        x, d, w = r(n, width) * 2, (r(n, width) + 3.0).to(dtype), 1 + 0.3 * r(width)
        table, ids = r(11, width).to(dtype), torch.randint(0, 11, (n,), generator=g).int()
        deltas = [(None, 0.0), (up(d), d.double())]
        if device != "cpu":
            deltas.append((torch.stack([up(d).float() * f for f in (0.5, 0.25, 0.125, 0.125)]), d.double()))
        for delta, dv in deltas:
            for source, base in ((up(x), x.double()), (lm.Embedding(ids.to(device), up(table), 0.5), table.double()[ids.long()] * 0.5)):
                want = base + dv
                src = source.clone() if isinstance(source, torch.Tensor) else source
                y, h = lm.residual_norm(src, delta, lm.PLAIN, 1.0, None, up(w), 1e-3, width, dtype)
                close(y[:, :width], want, 3e-5, "x")
                hw = R.rms(want, 1e-3) * w.double()
                close(h[:, :width], hw, 2e-5 if dtype == torch.float32 else 0.06, "h")
                assert not h[:, width:].any() and not y[:, width:].any()
                src = source.clone() if isinstance(source, torch.Tensor) else source
                rows = torch.tensor([n - 1, 0], dtype=torch.int32, device=device)
                _, h = lm.residual_norm(src, delta, lm.PLAIN, 1.0, None, up(w), 1e-3, width, dtype, rows=rows, keep=False)
                close(h[:, :width], hw[[n - 1, 0]], 2e-5 if dtype == torch.float32 else 0.06, "rows")


def attend(q, k, scale, temp, sink, cuts, device, dtype, splits=1, turn=None, out_scale=1.0):
    """One sequence's rows through the cache: q [n, H, d], k [n, G, d] -> [n, H, d]; ``turn``: (rot, q gain, k gain)."""
    n, H, d = q.shape
    dk, _ = lm.head_pad(d, d)
    rows = torch.cat([pad(t, dk).reshape(n, -1) for t in (q, k)], 1).to(device, dtype)
    blocks = Stepper((n,), "cpu").blocks
    kc, vc = (torch.full((blocks, k.shape[1], 64, dk), JUNK, dtype=dtype, device=device) for _ in range(2))
    temp, sink = temp.to(device), sink.to(device)
    rot, qg, kg = turn or ({"base": 1.0, "dims": 2}, torch.ones(d), torch.ones(d))
    freq = lm.rope_freq(rot["base"], rot["dims"])
    if turn is None:
        freq = freq * 0

    def fn(batch, at):
        t = torch.tensor([p for _, p in at], device=device)
        wide = torch.full((len(at), rows.shape[1] + 128), JUNK, dtype=dtype, device=device)   # rows lie inside wider ones
        wide[:, 64:-64] = rows[t]
        out = torch.full((len(at), H * dk + 64), JUNK, dtype=dtype, device=device)
        gains = (pad(qg, dk).to(device), pad(kg, dk).to(device)) if turn is not None else (None, None)
        turned = lm.HeadTurn(lm.rope_rows(batch.positions, freq.to(device)), d, 1e-6, *gains) if turn is not None else None
        lm.gated_attention(wide[:, 64:-64], kc, vc, batch, H, lm.WHOLE, scale, window=True, turn=turned,
                           plain=lm.Ungated(temp, sink, out[:, :H * dk], out_scale))
        assert (out[:, H * dk:] == JUNK).all() and (wide[:, :64] == JUNK).all() and (wide[:, -64:] == JUNK).all()
        return out[:, :H * dk]
    return drive((n,), cuts, device, fn, splits)[0].view(n, H, dk)[..., :d].double()


def check_needle(device, dtype):
    """One key whose score stands out, at page borders, the sequence's ends and far away: every later query copies its value,
    none before it does; with a sink that takes half of it and a head whose factor turns the score around."""
    n = 330
    tol = 1e-4 if dtype == torch.float32 else 0.05
    temp, sink = torch.tensor([1.0, 1.0, -1.0, 0.5]), torch.tensor([-50.0, 36.0, 0.0, 17.0])
    for at in (0, 1, 63, 64, 65, 127, 128, 200, 328, 329):
        g = torch.Generator().manual_seed(at)
        r = lambda *s: (torch.randn(*s, generator=g) * 0.3).bfloat16().float()
        q, k = r(n, 4, 24), r(n, 2, 24)
        q[..., 20], k[..., 20], k[at, :, 20] = 6.0, 0.0, 6.0                     # score 36 above the others
        want = R.sink_attend(q.double(), k.double(), k.double(), temp.double(), sink.double())
        sees = (want[:, 0, 20] - 6.0).abs() < 0.1
        assert sees.nonzero()[:, 0].tolist() == list(range(at, n)) and (want[at:, 1, 20] - 3.0).abs().max() < 2.9
        runs = (((n,), 1), ((64, 1, 5), 3)) if at % 2 else (((17, 16, 1, 1, 90), 1), ((300, 1), 5))
        for cuts, splits in runs:
            close(attend(q, k, 1.0, temp, sink, cuts, device, dtype, splits), want, tol, f"{at} {cuts}")


def check_sink(device, dtype):
    """Sinks far above and far below the scores, scores far below zero whose level differs between the splits of a decode step,
    and a factor on the output."""
    n = 450
    g = torch.Generator().manual_seed(17)
    r = lambda *s: torch.randn(*s, generator=g).bfloat16().float()
    q, k = r(n, 4, 24), r(n, 1, 24)
    q[..., 16], k[..., 16] = 8.0, (-30.0 - 0.02 * torch.arange(n))[:, None].bfloat16().float()
    temp, sink = torch.tensor([1.0, 0.25, 1.0, 0.25]), torch.tensor([-240.0, -60.0, -400.0, 40.0])
    want = 0.7 * R.sink_attend(q.double(), k.double(), k.double(), temp.double(), sink.double())
    assert want[:, 3].abs().max() < 1e-12 and want[:, 2].abs().min(0).values.max() > 10
    for splits in (1, 2, 3, 7):
        got = attend(q, k, 1.0, temp, sink, (430, 1, 3, 1), device, dtype, splits, out_scale=0.7)
        scale = want.abs().max()
        close(got / scale, want / scale, 5e-4 if dtype == torch.float32 else 0.03, str(splits))


def check_turn(device, dtype):
    """Norm with a gain, then rotation against the distance: heads of very different lengths weigh the same, the values are
    the keys as they were, and a key scaled a thousand times changes only its value."""
    n, rot = 150, {"base": 30.0, "dims": 20}
    g = torch.Generator().manual_seed(6)
    r = lambda *s: torch.randn(*s, generator=g).bfloat16().float()
    q, k = r(n, 4, 24), r(n, 2, 24)
    q = q * torch.tensor([0.25, 1.0, 16.0, 256.0])[:, None]
    k[77] *= 64.0
    qg, kg = 1 + 0.5 * r(24), 1 + 0.5 * r(24)
    temp, sink = 1 + 0.3 * r(4), r(4)
    turned = lambda x, w: R.rotate_half(R.rms(x.double(), 1e-6) * w.double(), rot)
    want = R.sink_attend(turned(q, qg), turned(k, kg), k.double(), 0.4 * temp.double(), sink.double())
    for cuts, splits in (((n,), 1), ((1,), 2), ((40, 1, 1, 30), 1)):
        got, size = attend(q, k, 0.4, temp, sink, cuts, device, dtype, splits, (rot, qg, kg)), 1 + want.abs().amax((1, 2), True)
        close(got / size, want / size, 1e-4 if dtype == torch.float32 else 0.06, str(cuts))


def check_mixers(device, dtype):
    """Whole layers (mixers and feed-forward on one norm's output) at sizes that need padding and stored head sizes of every
    kind, sequences of unequal length in one batch, by portions, with a decode step's blocks split."""
    layers = [P(), D(), T(), P(heads=1, kv_heads=1, dim=64, dims=64, right_heads=2, right_kv=1, right_dim=64, right_vdim=64, conv=1, mlp=None),
              P(heads=17, kv_heads=1, dim=24, dims=2, scale=-0.2, right_heads=1, right_kv=1, right_dim=100, right_vdim=30, conv=16, left_scale=-1.0),
              P(heads=2, kv_heads=2, dim=130, dims=40, scale=0.1, right_heads=2, right_kv=2, right_dim=128, right_vdim=128, conv=2),
              D(heads=2, kv_heads=1, dim=128, vdim=128, conv=4, mlp=None), D(heads=3, kv_heads=3, dim=70, vdim=60, conv=6),
              D(heads=1, kv_heads=1, dim=130, vdim=200, conv=4), D(heads=5, kv_heads=1, dim=1, vdim=1, conv=1),
              T(decay=(0.75,), dim=128, vdim=128, dims=128), T(decay=(1.0, 0.0), dim=64, vdim=100, dims=64),
              T(decay=(0.99, 0.9), dim=140, vdim=12, dims=2, mlp=None)]
    width, eps = 72, 1e-4
    w = R.random_weights(R.random_config(layers, width=width, eps=eps), 5)
    for i, lc in enumerate(layers):
        block = joint(layers, i, width, eps, w, dtype, device)
        lengths = (150, 1, 40, 65)
        g = torch.Generator().manual_seed(i)
        hs = [torch.randn(n, width, generator=g).bfloat16().float() for n in lengths]
        want = []
        for h in hs:
            get = lambda k: w[f"l{i}.{k}"].double()
            y = R.MIXERS[lc["type"]](h.double(), lc["mixer"], eps, lambda k: get("mix." + k))
            want.append(y + R.feed_forward(h.double(), lambda k: get("mlp." + k)) if lc["mlp"] else y)
        for cuts, splits in (((200,), 1), ((1,), 3), ((70, 1, 16, 17, 2), 1), ((64, 1, 1, 0), 2)):
            if cuts == (1,) and i > 5:
                continue
            cache, state = memory(block, Stepper(lengths, "cpu").blocks, len(lengths) + 2, dtype, device)

            def fn(batch, rows):
                h = pad(torch.stack([hs[b][p] for b, p in rows])).to(device, dtype)
                return whole(block(h, batch, cache, state, StepShared(batch)))[:, :width].float()

            for turn in range(2):                       # the second turn finds the first one's state in the slots
                for a, b in zip(drive(lengths, cuts, device, fn, splits), want):
                    e = (a.double() - b).abs().amax(-1) / b.std()
                    assert e.quantile(0.95) < (1e-3 if dtype == torch.float32 else 0.15), f"{i} {cuts} {e.max():.2e}"


def rule_case(device, dtype, H, G, d, vd, taps, lengths, channels, seed, fill):
    """Random inputs of the delta rule, changed by ``fill``, and what they give: (tensors, outputs of every sequence)."""
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g)
    n = [G * d, G * d, H * vd]
    x = [r(m, sum(n)).to(dtype) for m in lengths]
    z, beta = [r(m, H * d if channels else H) * 2 for m in lengths], [r(m, H) for m in lengths]
    gate = [r(m, H * vd).to(dtype) for m in lengths]
    t = dict(conv=r(taps, sum(n)) * 0.6, rate=torch.exp(r(H)), bias=r(H * d if channels else H) - 4.0, gain=1 + 0.3 * r(vd))
    fill(x, z, beta, t)
    want = []
    for xs, zs, bs, gs in zip(x, z, beta, gate):
        m = len(xs)
        y = R.short_conv(xs.double(), t["conv"].double().T)
        q, k, v = y.split(n, 1)
        spread = lambda a: a.view(m, G, d).repeat_interleave(H // G, 1)
        decay = R.softplus(zs.double() + t["bias"].double()).view(m, H, -1) * t["rate"].double()[:, None]
        o = R.delta_rows(R.unit(spread(q)) * d ** -0.5, R.unit(spread(k)), v.view(m, H, vd),
                         torch.exp(-decay).expand(m, H, d), torch.sigmoid(bs.double()))
        act = torch.sigmoid(gs.double()) if channels else R.silu(gs.double())
        want.append((R.rms(o, 1e-5) * t["gain"].double()).reshape(m, -1) * act)
    return (x, z, beta, gate, t), want


def run_rule(case, device, dtype, H, G, d, vd, taps, lengths, channels, cuts, turns=2):
    (x, z, beta, gate, t), _ = case
    dk, dv = lm.head_pad(d, vd)
    up = lambda a: a.to(device).contiguous()
    spread = lambda a, heads, m, p: pad(a.reshape(len(a), heads, m), p).reshape(len(a), -1)
    rows = lambda a: torch.cat([spread(b, heads, m, p) for b, heads, m, p in
                                zip(a.split([G * d, G * d, H * vd], 1), (G, G, H), (d, d, vd), (dk, dk, dv))], 1)
    xs, gs = [up(rows(a)) for a in x], [up(spread(a, H, vd, dv)) for a in gate]
    zs, bs = [up(spread(a, H, d, dk) if channels else a) for a in z], [up(a) for a in beta]
    conv, rate, gain = up(rows(t["conv"])), up(t["rate"]), up(pad(t["gain"], dv))
    bias = up(pad(t["bias"].view(H, d), dk).reshape(-1) if channels else t["bias"])
    state = torch.full((len(lengths) + 2, H, dk, dv), JUNK, device=device)
    ring = torch.full((len(lengths) + 2, taps, conv.shape[1]), JUNK, dtype=dtype, device=device)
    shape = lm.RuleShape(G, d, vd, lm.GATE_SIGMOID if channels else lm.GATE_SILU)

    def fn(batch, at):
        pick = lambda ts: torch.stack([ts[b][p] for b, p in at])
        out = torch.full((len(at), H * dv), JUNK, dtype=dtype, device=device)
        lm.delta_rule(pick(xs), pick(gs), pick(zs), pick(bs), conv, rate, bias, gain, state, ring, batch, out, shape, 1e-5)
        return out
    return [[y.view(len(y), H, dv) for y in drive(lengths, cuts, device, fn)] for _ in range(turns)]


def check_delta(device, dtype):
    """The delta rule over portions and chunks of them, in batches, with reused slots, at every stored head size: heads and
    channels that keep, forget at once and change their mind, strengths at both ends, the first token's write read at the end,
    a key that is written again."""
    def fill(x, z, beta, t):
        for xs, zs, bs in zip(x, z, beta):
            zs[:, 0] = torch.where(torch.arange(len(zs)) % 40 < 20, 25.0, -25.0)     # forgets at once, keeps all
            zs[:, -1] = -30.0                                                         # hardly forgets
            bs[:, -1] = 0.0
            bs[0] = 30.0
            bs[:, 0] = torch.where(torch.arange(len(bs)) % 7 < 2, 30.0, -30.0)
            for at in range(11, len(xs), 11):
                xs[at] = xs[at - 9]
    sizes = [(2, 1, 24, 40, 4, (200, 1, 65, 129)), (1, 1, 64, 64, 1, (70, 64, 3)), (3, 3, 50, 128, 7, (90, 33)),
             (4, 2, 100, 64, 2, (90, 31)), (2, 2, 128, 100, 3, (66, 97)), (1, 1, 130, 200, 16, (80, 17))]
    if device != "cpu":
        sizes += [(2, 1, 128, 128, 4, (2100, 300)), (1, 1, 64, 64, 4, (3000, 129))]
    tol = 1e-3 if dtype == torch.float32 else 0.06
    for i, (H, G, d, vd, taps, lengths) in enumerate(sizes):
        for channels in (False, True):
            case = rule_case(device, dtype, H, G, d, vd, taps, lengths, channels, i, fill)
            for cuts in ((5000,), (1,), (2, 3), (64, 1, 65, 0), (130, 7), (31, 33, 500)):
                if (sum(lengths) > 500 and cuts[0] < 31) or (device == "cpu" and cuts in ((2, 3), (130, 7)) and i > 1):
                    continue
                for got in run_rule(case, device, dtype, H, G, d, vd, taps, lengths, channels, cuts):
                    for a, b in zip(got, case[1]):
                        assert not a[..., vd:].any()
                        e = (a[..., :vd].double() - b.view(len(b), H, vd)).abs().amax((1, 2))
                        assert e.max() < 6 * tol and e.quantile(0.98) < tol, (d, vd, taps, channels, cuts, e.max(), e.argmax())


def check_delta_memory(device, dtype):
    """A value written once under a key of its own comes back whole after a long time, is replaced by the next write under
    that key, and is gone after one token that forgets; the convolution's first inputs count as zeros and its window ends
    after the given number of taps."""
    d, vd, n = 24, 40, 150
    for channels in (False, True):
        for taps in (1, 4):
            def fill(x, z, beta, t):
                z[0][:] = -60.0                                    # keeps everything
                beta[0][:] = -60.0                                 # writes nothing
                t["rate"][:], t["bias"][:], t["gain"][:] = 1.0, 0.0, 1.0
                t["conv"][:] = 0.0
                t["conv"][-1] = 1.0
                if taps > 1:
                    t["conv"][0, 2 * d:] = 1.0                     # values: also the one of taps - 1 tokens ago
                x[0][:, :2 * d] = -8.0                             # silu takes it to zero
                x[0][:, 0], x[0][:, d] = 8.0, 8.0                  # queries and keys all the same
                for at in (0, 100):
                    beta[0][at] = 60.0
                z[0][130] = 60.0
            sizes = (1, 1, d, vd, taps, (n,), channels)
            case = rule_case(device, dtype, 1, 1, d, vd, taps, (n,), channels, 3, fill)
            xs = case[0][0][0].double()[:, 2 * d:]
            value = lambda t: R.silu(xs[t] + (xs[t - taps + 1] if taps > 1 and t >= taps - 1 else 0.0))
            gate = case[0][3][0].double()
            act = torch.sigmoid(gate) if channels else R.silu(gate)
            for t in range(130):
                v = value(0 if t < 100 else 100)
                close(case[1][0][t], R.rms(v, 1e-5 * d) * act[t], 0.03, f"oracle {t}")
            for cuts in ((n,), (1,), (99, 2, 1, 1), (32, 31)):
                for got in run_rule(case, device, dtype, *sizes, cuts):
                    close(got[0][:130, 0, :vd], case[1][0][:130], 1e-3 if dtype == torch.float32 else 0.05, f"{channels} {taps} {cuts}")
                    assert got[0][131:].abs().max() < 1e-3


def check_retention(device, dtype):
    """Retention over portions and chunks of them, in batches, with reused slots: heads that keep everything, forget at once
    and anything between; the first token's contribution carried to the end; rotation against the distance."""
    sizes = [((1.0, 0.0, 0.5), 24, 40, 6, (200, 1, 65, 129)), ((0.999,), 64, 64, 64, (70, 64, 3)), ((0.9, 0.99), 50, 128, 50, (90, 33)),
             ((0.9921875,), 128, 100, 2, (66, 97)), ((0.25, 0.998046875), 130, 200, 60, (80, 17))]
    if device != "cpu":
        sizes += [((0.9990234375, 0.96875), 128, 128, 128, (2100, 300))]
    for i, (decay, d, vd, rot, lengths) in enumerate(sizes):
        H, (dk, dv) = len(decay), lm.head_pad(d, vd)
        g = torch.Generator().manual_seed(i)
        r = lambda *s: torch.randn(*s, generator=g).to(dtype)
        qs, ks, vs, gs = ([r(n, H, m) for n in lengths] for m in (d, d, vd, vd))
        for v in vs:
            v[0] *= 100.0
        rt = {"base": 500.0, "dims": rot}
        want = []
        for q, k, v, z in zip(qs, ks, vs, gs):
            o = R.retention_rows(R.rotate_half(q.double(), rt), R.rotate_half(k.double(), rt) * d ** -0.5, v.double(),
                                 torch.tensor(decay, dtype=torch.float64))
            want.append(R.rms(o, 1e-5) * R.silu(z.double()))
        row = lambda t, m: pad(t, m).reshape(len(t), -1)
        xs = [torch.cat([row(q, dk), row(k, dk), row(v, dv)], 1).to(device) for q, k, v in zip(qs, ks, vs)]
        zs, freq, rates = [row(z, dv).to(device) for z in gs], lm.rope_freq(500.0, rot).to(device), lm.decay_rates(decay).to(device)
        for cuts in ((5000,), (1,), (2, 3), (64, 1, 65, 0), (31, 33, 500)):
            if sum(lengths) > 500 and cuts[0] < 31:
                continue
            state = torch.full((len(lengths) + 2, H, dk, dv), JUNK, device=device)

            def fn(batch, at):
                pick = lambda ts: torch.stack([ts[b][p] for b, p in at])
                out = torch.full((len(at), H * dv), JUNK, dtype=dtype, device=device)
                lm.retention(pick(xs), pick(zs), rates, lm.rope_rows(batch.positions, freq), state, batch, out,
                             lm.RuleShape(H, d, vd), 1e-5)
                return out
            for turn in range(2):
                for a, b in zip(drive(lengths, cuts, device, fn), want):
                    a = a.view(len(b), H, dv)
                    assert not a[..., vd:].any()
                    e = (a[..., :vd].double() - b).abs().amax((1, 2))
                    assert e.max() < (3e-3 if dtype == torch.float32 else 0.1), (decay, d, vd, cuts, e.max(), e.argmax())


MECHANISMS = [check_matmul, check_norm, check_needle, check_sink, check_turn, check_mixers, check_delta, check_delta_memory,
              check_retention]

# ---------------------------------------------------------------------------------------------- whole models
L3 = [P(), D(), T()]
SHAPES = {
    "base": {},
    "parallel_only": dict(layers=[P(heads=1, kv_heads=1, dim=64, dims=64, right_heads=1, right_kv=1), P(heads=5, kv_heads=1, mlp=None)]),
    "delta_only": dict(layers=[D(), D(1, 1, 64, 64, 4, R.dense(64)), D(4, 1, 9, 100, 1)], width=64),
    "retention_only": dict(layers=[T(), T((0.9,), 64, 64, 1e6, 64)], vocab=33),
    "one_layer": dict(layers=[T((0.875,) * 5, 1 + 1, 1, 10.0, 2, R.dense(1))], width=1),
    "no_mlp": dict(layers=[D(mlp=None), P(mlp=None), T(mlp=None)], width=100),
    "used_thrice": dict(layers=[T(), P(conv=2), R.again(P(conv=2), 1), D(), R.again(P(conv=2), 1), R.again(T(), 0)]),
    "big_heads": dict(layers=[P(heads=2, kv_heads=1, dim=136, dims=136, scale=0.1, right_heads=1, right_kv=1, right_dim=150, right_vdim=256),
                              D(2, 1, 129, 40), T((0.5, 0.99), 200, 130)], width=72),
    "many_heads": dict(layers=[P(heads=36, kv_heads=2, dim=8, dims=2, right_heads=20, right_kv=4), D(40, 20, 4, 8), T((0.9,) * 33, 8, 4, 9.0, 8)],
                       embed_scale=1.0),
    "signs": dict(layers=[P(scale=-0.3, left_scale=-0.5, right_scale=2.0), P(left_scale=1.0, right_scale=0.0)], eps=1e-2),
    "wide": dict(layers=L3, width=330, vocab=515),
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
    """The residual stream after every layer."""
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
    assert len(trail) == len(want) == 5
    for a, b in zip(trail, want):
        err = (a.double().cpu() - b).abs().amax(-1) / b.abs().max()
        assert err.quantile(0.9) < (2e-5 if dtype == torch.float32 else 0.03)


def check_portions(tmp, device, dtype):
    c = Case(tmp, device, dtype, seed=4)
    eng = c.engine()
    toks = c.tokens(150)
    want = c.oracle(toks)
    for cuts in ((150,), (2,), (3,), (64,), (1,), (63, 2, 1, 65), (16, 17, 1, 1, 44), (149, 1), (32, 33, 31)):
        s = eng.open_request()
        assert_logits(run(eng, s, toks, cuts), want, dtype, str(cuts))
        eng.close_request(s)


def check_long_decode(tmp, device, dtype):
    """Decoding over many pages and chunks, token by token."""
    c = Case(tmp, device, dtype, seed=5, layers=[P(), D(), T(), R.again(P(), 0)])
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
    c = Case(tmp, device, dtype, seed=7, layers=[D(), P(), T()])
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
    c = Case(tmp, device, dtype, seed=8, layers=[P(), D(), T(mlp=None), R.again(P(), 0)])
    shared = c.tokens(64)
    prompts = [shared + c.tokens(30), c.tokens(3), shared + c.tokens(5), c.tokens(100), c.tokens(1)]
    eng = LLMEngine(config_from_path(c.path), device=device, model_path=c.path, max_num_seqs=4, max_model_len=192,
                    dtype=dtype, prefill_chunk=64, **kw)
    params = SamplingParams(temperature=0.0, max_tokens=20)
    for turn in range(2):                               # a common prefix is not shared: its state would be missing
        outs = eng.generate(prompts, params)
        gaps = []
        for p, s in zip(prompts, outs):
            toks = (s.prompt + s.output)[len(p):]
            assert len(toks) == 20
            lg = c.oracle(p + toks)[len(p) - 1:-1]      # choices are at (or within rounding of) the maximum
            gaps.append((lg.max(-1).values - lg.gather(1, torch.tensor(toks)[:, None])[:, 0]) / lg.std())
        gaps = torch.cat(gaps)
        assert gaps.max() < 1e-4 if dtype == torch.float32 else gaps.quantile(0.95) < 0.1
    assert eng.stats["prefix_hit_tokens"] == 0
    assert eng.bm.num_free == eng.num_kv_blocks and eng.state_slots.num_free == 4


def check_sampling(tmp, device, dtype):
    """A seeded request draws the same tokens alone and in a batch."""
    c = Case(tmp, device, dtype, seed=9, layers=[D(), P()])
    cfg = config_from_path(c.path)
    p = SamplingParams(temperature=4.0, top_k=12, top_p=0.95, max_tokens=12, seed=5)
    mk = lambda: LLMEngine(cfg, device=device, model_path=c.path, max_num_seqs=4, max_model_len=128, dtype=dtype)
    prompts = [c.tokens(n) for n in (9, 40, 2)]
    alone = mk().generate([prompts[0]], p)[0].output
    assert mk().generate(prompts, p)[0].output == alone and len(set(alone)) > 1


def check_far_token(tmp, device, dtype):
    """The first token reaches the last position through each kind of mixer, by portions and by decoded tokens."""
    for layers in ([P(heads=2, scale=0.3, mlp=None, right_scale=0.0)], [P(left_scale=0.0, mlp=None)], [D(mlp=None)],
                   [T(decay=(0.998046875, 0.9990234375), mlp=None)]):
        kind = layers[0]["type"]
        c = Case(tmp, device, dtype, seed=20, layers=layers, vocab=40)
        for k in c.w:
            if k.endswith("dt_bias"):
                c.w[k] = c.w[k] * 0 - 8.0                # decays that hardly forget
        c.path = R.save_checkpoint(tmp / f"far-{kind}", c.cfg, c.w)
        toks = [7] + [t if t != 7 else 8 for t in c.tokens(159)]
        want, other = c.oracle(toks), c.oracle([9] + toks[1:])
        assert position_errors(other, want).min() > 5 * F32_TOL
        eng = c.engine(256)
        for cuts in ((160,), (100, 1), (1, 63, 1, 1), (2,)):
            s = eng.open_request()
            assert_logits(run(eng, s, toks, cuts), want, dtype, f"{kind} {cuts}")
            eng.close_request(s)


MODELS = [check_layers, check_portions, check_long_decode, check_batches, check_slots, check_sampling, check_far_token]


def planted(cfg, w):
    """(what, config, weights) with one mistake each, for the oracle: the comparison must notice every one."""
    def changed(f):
        c, v = copy.deepcopy(cfg), dict(w)
        f(c, v)
        return c, v

    def weights(end, fn):
        return lambda c, v: v.update({k: fn(t) for k, t in v.items() if k.endswith(end)})

    def entries(kind, fn):
        return lambda c, v: [fn(lc) for lc in c["layers"] if lc["type"] == kind]
    yield ("embedding scale",) + changed(lambda c, v: c["embedding"].update(scale=1.0))
    yield ("eps",) + changed(lambda c, v: c["norm"].update(eps=0.02))
    for n in ("norm1", "final.norm", "q.norm", "k.norm", "mix.norm", "right.norm", "temp"):
        yield (n,) + changed(weights(n, lambda t: t * 0 + 1.0))
    yield ("sink left out",) + changed(weights("sink", lambda t: t * 0 - 60.0))
    yield ("oldest tap left out",) + changed(weights(".conv", lambda t: t * (torch.arange(t.shape[1]) > 0)))
    yield ("taps turned around",) + changed(weights(".conv", lambda t: t.flip(1)))
    yield ("strengths",) + changed(weights(".b", lambda t: t * 0))
    yield ("decay rate",) + changed(weights("A_log", lambda t: t * 0))
    yield ("decay bias",) + changed(weights("dt_bias", lambda t: t * 0))
    yield ("decay of one channel for all",) + changed(weights("right.a2", lambda t: t[:1].expand_as(t)))
    yield ("no output gate",) + changed(weights("mix.g", lambda t: t * 0))
    yield ("no thin output gate",) + changed(weights("right.g2", lambda t: t * 0))
    yield ("left scale",) + changed(entries("parallel", lambda x: x["mixer"].update(left_scale=1.0)))
    yield ("right scale",) + changed(entries("parallel", lambda x: x["mixer"].update(right_scale=1.0)))
    yield ("score scale",) + changed(entries("parallel", lambda x: x["mixer"]["left"].update(scale=0.5)))
    yield ("rotation base",) + changed(entries("parallel", lambda x: x["mixer"]["left"]["rot"].update(base=90.0)))
    yield ("rotated dimensions",) + changed(entries("retention", lambda x: x["mixer"]["rot"].update(dims=10)))
    yield ("retention rotation base",) + changed(entries("retention", lambda x: x["mixer"]["rot"].update(base=300.0)))
    yield ("decays in another order",) + changed(entries("retention", lambda x: x["mixer"].update(decay=x["mixer"]["decay"][::-1])))
    yield ("no feed-forward",) + changed(weights("mlp.up", lambda t: t * 0))
    yield ("weights of another layer",) + changed(lambda c, v: (c["layers"][3].pop("weights_of"), v.update(
        {"l3" + k[2:]: t.flip(0) if k.endswith("left.q") else t for k, t in w.items() if k.startswith("l0.")})))
