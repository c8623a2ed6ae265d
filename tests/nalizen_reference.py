"""Plain, slow fp64 implementation of the Nalizen decoder, one function per mechanism, written from the model's equations.
Shares no code with ``shai_amd``: tests compare the framework with it.

``cfg`` is the parsed config.json, ``w`` a dict of full tensors under their checkpoint names.  A whole sequence is
recomputed from its first token, so there is no cache, no batch and no state to get wrong."""
import json
import math
import os

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def embed(tokens, cfg, w):
    return w["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]


def token_shift(h, s):
    """Every row moved towards the row before it (zeros before the first) by the shares ``s``."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * s


def frequencies(rot):
    """Rotation frequency of every pair."""
    out, sc = [], rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        if sc:
            turn = 2.0 * math.pi / f                    # tokens of a full turn
            if turn > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif turn >= sc["original"] / sc["high"]:
                s = (sc["original"] / turn - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate_half(x, rot, first=0):
    """x [n, ..., dim], row t at position ``first`` + t: dimension i < dims / 2 pairs with i + dims / 2."""
    n, half = x.shape[0], rot["dims"] // 2
    out = x.clone()
    for i, f in enumerate(frequencies(rot)):
        a = ((torch.arange(n, dtype=x.dtype) + first) * f).reshape([n] + [1] * (x.dim() - 2))
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., i + half] = v * torch.cos(a) + u * torch.sin(a)
    return out


def window_attend(q, k, v, scale, size):
    """q [n, H, dk], k [n, G, dk], v [n, G, dv] -> [n, H, dv]: softmax over a token and the size - 1 tokens before it."""
    n, H, G = q.shape[0], q.shape[1], k.shape[1]
    back = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    see = (back >= 0) & (back < size)
    outs = []
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(~see, float("-inf"))
        outs.append(torch.softmax(s, -1) @ v[:, g])
    return torch.stack(outs, 1)


def attention(h, mc, eps, get, kv=None):
    """h [n, width] -> ([n, width], (keys, values)); ``kv``: another layer's keys and values instead of own ones."""
    n, H, G = h.shape[0], mc["heads"], mc["kv_heads"]
    turn = lambda x: rms(rotate_half(x, mc["rot"]), eps)
    q = turn((h @ get("q").T).view(n, H, mc["dim"]))
    if kv is None:
        kv = turn((h @ get("k").T).view(n, G, mc["dim"])), (h @ get("v").T).view(n, G, mc["vdim"])
    o = window_attend(q, *kv, mc["scale"], mc["mask"]["size"]).reshape(n, -1)
    return (o * torch.sigmoid(h @ get("g").T)) @ get("o").T, kv


def hgrn2_rows(q, z, lower, v):
    """q, z [n, H, dk] (activated queries, forget logits with bias), lower [H, dk], v [n, H, dv] -> o [n, H, dv]."""
    f = lower + (1.0 - lower) * torch.sigmoid(z)
    S = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype)
    out = []
    for t in range(q.shape[0]):
        S = f[t][:, :, None] * S + (1.0 - f[t])[:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def hgrn2(h, mc, eps, get):
    n, H, dk, dv = h.shape[0], mc["heads"], mc["dim"], mc["vdim"]
    q = h @ get("q").T
    q = (q * torch.sigmoid(q)).view(n, H, dk)
    z = (h @ get("f").T + get("f.b")).view(n, H, dk)
    o = hgrn2_rows(q, z, get("lower").view(H, dk), (h @ get("v").T).view(n, H, dv))
    return (rms(o, eps) * get("norm")).reshape(n, -1) @ get("o").T


def dense_ff(h, get):
    return (gelu_tanh(h @ get("gate").T) * (h @ get("up").T)) @ get("down").T


def route(z, top):
    """[(expert, weight)] of one token from its router logits."""
    ids = torch.topk(z, top).indices
    return list(zip(ids.tolist(), torch.softmax(z[ids], 0)))


def moe_ff(h, top, get):
    z = h @ get("router").T + get("router.b")
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in route(z[t], top):
            out[t] += p * ((torch.relu(h[t] @ get(f"e{e}.up").T) ** 2) @ get(f"e{e}.down").T)
    return out


def side_input(x, e, eps, gate, proj, gain):
    """x [n, width] and the tokens' rows e [n, dim] of one layer -> what is added to x."""
    return rms((gelu_tanh(x @ gate.T) * e) @ proj.T, eps) * gain


def forward(tokens, cfg, w, dtype=torch.float64):
    """(logits [n, vocab], [residual stream after every layer])."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps, tokens = cfg["norm"]["eps"], list(tokens)
    x = embed(tokens, cfg, w)
    trail, kvs, sd = [], {}, cfg["token_side"]["dim"]
    for i, lc in enumerate(cfg["layers"]):
        p, mc = f"l{i}.", lc["mixer"]
        get = lambda n: w[p + "mix." + n]
        h = token_shift(x, w[p + "shift"])
        if lc["type"] == "attention":
            y, kvs[i] = attention(h, mc, eps, get, kvs[mc["kv_from"]] if mc.get("kv_from") is not None else None)
        else:
            y = hgrn2(h, mc, eps, get)
        x = x + layer_norm(y, w[p + "norm1"], w[p + "norm1.b"], eps)
        if lc.get("mlp"):
            ff = lambda n: w[p + "mlp." + n]
            y = dense_ff(x, ff) if lc["mlp"]["kind"] == "dense" else moe_ff(x, lc["mlp"]["router"]["top"], ff)
            x = x + layer_norm(y, w[p + "norm2"], w[p + "norm2.b"], eps)
        e = w["side.embed"][torch.tensor(tokens), i * sd:(i + 1) * sd]
        x = x + side_input(x, e, eps, w[p + "side.gate"], w[p + "side.proj"], w[p + "side.norm"])
        trail.append(x)
    return layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["embed"].T, trail


# ---------------------------------------------------------------------------------------------- random models
def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def experts(n=5, top=2, ff=24):
    return {"kind": "moe", "router": {"experts": n, "top": top}, "expert": {"ff": ff}}


def scaling(factor=6.0, low=0.7, high=3.0, original=90):
    return {"factor": factor, "low": low, "high": high, "original": original}


def attention_layer(heads=6, kv_heads=2, dim=20, vdim=28, window=37, base=60.0, dims=12, scale=0.4, stretch=scaling(),
                    kv_from=None, mlp=dense()):
    rot = {"base": base, "dims": dims}
    if stretch:
        rot["scaling"] = dict(stretch)
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window}, "rot": rot, "scale": scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp and dict(mlp)}


def hgrn2_layer(heads=3, dim=20, vdim=36, mlp=experts()):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}, "mlp": mlp and dict(mlp)}


def random_config(layers=None, vocab=97, width=56, side=10, embed_scale=2.5, eps=1e-4):
    layers = layers or [attention_layer(), hgrn2_layer(), attention_layer(kv_from=0, window=51, scale=0.3, mlp=experts()),
                        hgrn2_layer(2, 70, 24, dense(50))]
    return {"architecture": "Nalizen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "token_side": {"dim": side},
            "embedding": {"scale": embed_scale}, "layers": layers}


def random_weights(cfg, seed=0):
    """bfloat16-exact random weights under their checkpoint names (fp32 tensors)."""
    g = torch.Generator().manual_seed(seed)
    b = lambda t: t.bfloat16().float()
    r = lambda *s, std=None: b(torch.randn(*s, generator=g) * (s[-1] ** -0.5 if std is None else std))
    gain = lambda n: b(1.0 + 0.3 * torch.randn(n, generator=g))
    D, L, S = cfg["width"], len(cfg["layers"]), cfg["token_side"]["dim"]
    w = {"embed": r(cfg["vocab"], D, std=0.5), "side.embed": r(cfg["vocab"], L * S, std=1.0),
         "final.norm": gain(D), "final.norm.b": r(D, std=0.3)}
    for i, lc in enumerate(cfg["layers"]):
        m, p, ff = lc["mixer"], f"l{i}.", lc.get("mlp")
        w[p + "norm1"], w[p + "norm1.b"], w[p + "shift"] = gain(D), r(D, std=0.3), b(torch.rand(D, generator=g) * 1.2 - 0.1)
        w[p + "side.gate"], w[p + "side.proj"], w[p + "side.norm"] = r(S, D), r(D, S), b(0.5 * gain(D))
        H, d, vd = m["heads"], m["dim"], m["vdim"]
        w[p + "mix.q"], w[p + "mix.o"] = r(H * d, D), r(D, H * vd)
        if lc["type"] == "attention":
            w[p + "mix.g"] = r(H * vd, D)
            if m.get("kv_from") is None:
                w[p + "mix.k"], w[p + "mix.v"] = r(m["kv_heads"] * d, D), r(m["kv_heads"] * vd, D)
        else:
            w[p + "mix.f"], w[p + "mix.f.b"], w[p + "mix.v"] = r(H * d, D), r(H * d, std=1.0), r(H * vd, D)
            w[p + "mix.lower"] = b(torch.rand(H * d, generator=g) ** 0.3 * 0.98)       # many channels reach far back
            w[p + "mix.norm"] = gain(vd)
        if ff:
            w[p + "norm2"], w[p + "norm2.b"] = gain(D), r(D, std=0.3)
        if ff and ff["kind"] == "dense":
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = r(ff["ff"], D), r(ff["ff"], D), r(D, ff["ff"])
        elif ff:
            E, F = ff["router"]["experts"], ff["expert"]["ff"]
            w[p + "mlp.router"], w[p + "mlp.router.b"] = r(E, D, std=2 * D ** -0.5), r(E, std=1.0)
            for e in range(E):
                w[p + f"mlp.e{e}.up"], w[p + f"mlp.e{e}.down"] = r(F, D), r(D, F)
    return w


def save_checkpoint(path, cfg, w):
    """config.json + model.safetensors (bfloat16) in ``path``."""
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.bfloat16().contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
    return str(path)
