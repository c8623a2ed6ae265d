"""Plain, slow fp64 implementation of the Pugozen decoder, one function per mechanism, written from the model's equations.
Shares no code with ``shai_amd``: tests compare the framework with it.

``cfg`` is the parsed config.json, ``w`` a dict of full tensors under their checkpoint names.  A whole sequence is
recomputed from its first token, so there is no cache, no batch and no state to get wrong."""
import copy
import json
import os

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def rotate_half(x, rot, first=0):
    """x [n, heads, dim], row t at position ``first`` + t: dimension i < dims / 2 pairs with i + dims / 2."""
    n, half = x.shape[0], rot["dims"] // 2
    out = x.clone()
    for i in range(half):
        a = ((torch.arange(n, dtype=x.dtype) + first) * rot["base"] ** (-2.0 * i / rot["dims"]))[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., i + half] = v * torch.cos(a) + u * torch.sin(a)
    return out


def short_conv(x, taps):
    """x [n, channels], taps [channels, number]: each channel's last inputs, the newest under the last tap, then silu."""
    n, k = x.shape[0], taps.shape[1]
    out = torch.zeros_like(x)
    for j in range(k):
        age = k - 1 - j
        if age < n:
            out[age:] += taps[:, j] * x[:n - age]
    return silu(out)


def sink_attend(q, k, v, scale, sink):
    """q [n, H, d], k [n, G, d], v [n, G, dv], scale and sink [H] -> [n, H, dv]: softmax over a token and all before it,
    with exp(sink) in the denominator."""
    n, H, G = q.shape[0], q.shape[1], k.shape[1]
    later = torch.arange(n)[None, :] > torch.arange(n)[:, None]
    outs = []
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale[h]).masked_fill(later, float("-inf"))
        top = torch.maximum(s.max(-1, keepdim=True).values, sink[h])
        e = torch.exp(s - top)
        outs.append((e @ v[:, g]) / (e.sum(-1, keepdim=True) + torch.exp(sink[h] - top)))
    return torch.stack(outs, 1)


def attention(h, mc, eps, get):
    """The values are the projected keys, before norm and rotation."""
    n, H, G, d = h.shape[0], mc["heads"], mc["kv_heads"], mc["dim"]
    q, k = (h @ get("q").T).view(n, H, d), (h @ get("k").T).view(n, G, d)
    turn = lambda x, name: rotate_half(rms(x, eps) * get(name), mc["rot"])
    o = sink_attend(turn(q, "q.norm"), turn(k, "k.norm"), k, mc["scale"] * get("temp"), get("sink"))
    return o.reshape(n, -1) @ get("o").T


def delta_rows(q, k, v, g, beta):
    """q, k [n, H, dk], v [n, H, dv], g [n, H, dk] (decay of every row of S), beta [n, H] -> o [n, H, dv]."""
    S = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype)
    out = []
    for t in range(q.shape[0]):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def delta_inputs(h, mc, get):
    """Queries, keys (both per head), values and write strengths of the delta rule."""
    n, H, G = h.shape[0], mc["heads"], mc["kv_heads"]
    conv = lambda name: short_conv(h @ get(name).T, get(name + ".conv"))
    spread = lambda x: x.repeat_interleave(H // G, 1)
    q = spread(unit(conv("q").view(n, G, mc["dim"]))) * mc["dim"] ** -0.5
    k = spread(unit(conv("k").view(n, G, mc["dim"])))
    return q, k, conv("v").view(n, H, mc["vdim"]), torch.sigmoid(h @ get("b").T)


def delta(h, mc, eps, get):
    """One decay per head, silu gate."""
    n, H = h.shape[0], mc["heads"]
    q, k, v, beta = delta_inputs(h, mc, get)
    g = torch.exp(-torch.exp(get("A_log")) * softplus(h @ get("a").T + get("dt_bias")))
    o = delta_rows(q, k, v, g[:, :, None].expand(n, H, mc["dim"]), beta)
    o = rms(o, eps) * get("norm") * silu(h @ get("g").T).view(n, H, -1)
    return o.reshape(n, -1) @ get("o").T


def channel_delta(h, mc, eps, get):
    """One decay per head and key channel, sigmoid gate, both through two thin products."""
    n, H, d = h.shape[0], mc["heads"], mc["dim"]
    q, k, v, beta = delta_inputs(h, mc, get)
    z = ((h @ get("a1").T) @ get("a2").T + get("dt_bias")).view(n, H, d)
    o = delta_rows(q, k, v, torch.exp(-torch.exp(get("A_log"))[:, None] * softplus(z)), beta)
    gate = torch.sigmoid((h @ get("g1").T) @ get("g2").T).view(n, H, -1)
    return (rms(o, eps) * get("norm") * gate).reshape(n, -1) @ get("o").T


def parallel(h, mc, eps, get):
    left = attention(h, mc["left"], eps, lambda k: get("left." + k))
    right = channel_delta(h, mc["right"], eps, lambda k: get("right." + k))
    return mc["left_scale"] * left + mc["right_scale"] * right


def retention_rows(q, k, v, decay):
    """q, k [n, H, dk], v [n, H, dv], decay [H] -> o [n, H, dv]."""
    S = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype)
    out = []
    for t in range(q.shape[0]):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def retention(h, mc, eps, get):
    n, H, d = h.shape[0], mc["heads"], mc["dim"]
    q = rotate_half((h @ get("q").T).view(n, H, d), mc["rot"])
    k = rotate_half((h @ get("k").T).view(n, H, d), mc["rot"]) * d ** -0.5
    o = rms(retention_rows(q, k, (h @ get("v").T).view(n, H, -1), torch.tensor(mc["decay"], dtype=h.dtype)), eps)
    return (o.reshape(n, -1) * silu(h @ get("g").T)) @ get("o").T


MIXERS = {"retention": retention, "delta": delta, "parallel": parallel}


def feed_forward(h, get):
    return (torch.relu(h @ get("up").T) ** 2) @ get("down").T


def weights_layer(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(tokens, cfg, w, dtype=torch.float64):
    """(logits [n, vocab], [residual stream after every layer])."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(list(tokens))] * cfg["embedding"]["scale"]
    trail = []
    for i, lc in enumerate(cfg["layers"]):
        p = f"l{weights_layer(cfg, i)}."
        h = rms(x, eps) * w[p + "norm1"]
        y = MIXERS[lc["type"]](h, lc["mixer"], eps, lambda n: w[p + "mix." + n])
        if lc.get("mlp"):
            y = y + feed_forward(h, lambda n: w[p + "mlp." + n])
        x = x + y
        trail.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T, trail


# ---------------------------------------------------------------------------------------------- random models
def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def delta_layer(heads=6, kv_heads=3, dim=20, vdim=36, conv=3, mlp=dense()):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}
    return {"type": "delta", "mixer": m, "mlp": mlp and dict(mlp)}


def retention_layer(decay=(0.5, 0.97, 0.998), dim=28, vdim=20, base=200.0, dims=12, mlp=dense(72)):
    m = {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay), "rot": {"base": base, "dims": dims}}
    return {"type": "retention", "mixer": m, "mlp": mlp and dict(mlp)}


def parallel_layer(heads=6, kv_heads=2, dim=20, base=60.0, dims=12, scale=0.3, right_heads=4, right_kv=2, right_dim=12,
                   right_vdim=28, conv=5, left_scale=0.7, right_scale=1.3, mlp=dense()):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale, "rot": {"base": base, "dims": dims}}
    right = {"heads": right_heads, "kv_heads": right_kv, "dim": right_dim, "vdim": right_vdim, "conv": conv}
    m = {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}
    return {"type": "parallel", "mixer": m, "mlp": mlp and dict(mlp)}


def again(layer, j):
    """A layer like ``layer``, layer j, with its weights."""
    return dict(copy.deepcopy(layer), weights_of=j)


def random_config(layers=None, vocab=97, width=56, embed_scale=2.5, eps=1e-4):
    if layers is None:
        layers = [parallel_layer(), delta_layer(), retention_layer()]
        layers += [again(layers[0], 0), again(layers[1], 1)]
    return {"architecture": "Pugozen", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": embed_scale}, "layers": layers}


def random_weights(cfg, seed=0, ranks=(10, 14)):
    """bfloat16-exact random weights under their checkpoint names (fp32 tensors)."""
    g = torch.Generator().manual_seed(seed)
    b = lambda t: t.bfloat16().float()
    r = lambda *s, std=None: b(torch.randn(*s, generator=g) * (s[-1] ** -0.5 if std is None else std))
    gain = lambda n: b(1.0 + 0.3 * torch.randn(n, generator=g))
    D = cfg["width"]
    w = {"embed": r(cfg["vocab"], D, std=0.5), "head": r(cfg["vocab"], D), "final.norm": gain(D)}

    def rule(p, m, channels):
        n, kv, H, d, vd = m["heads"] * m["dim"], m["kv_heads"] * m["dim"], m["heads"], m["dim"], m["vdim"]
        for name, c in (("q", kv), ("k", kv), ("v", H * vd)):
            w[p + name], w[p + name + ".conv"] = r(c, D), r(c, m["conv"])
        w[p + "b"], w[p + "A_log"], w[p + "norm"] = r(H, D, std=2 * D ** -0.5), r(H, std=1.5), gain(vd)
        w[p + "o"] = r(D, H * vd)
        if channels:
            w[p + "a1"], w[p + "a2"] = r(ranks[0], D), r(n, ranks[0], std=1.0)
            w[p + "g1"], w[p + "g2"] = r(ranks[1], D), r(H * vd, ranks[1])
        else:
            w[p + "a"], w[p + "g"] = r(H, D), r(H * vd, D)
        w[p + "dt_bias"] = b(-3.0 + 2.0 * torch.randn(n if channels else H, generator=g))   # many channels reach far back
    for i, lc in enumerate(cfg["layers"]):
        if lc.get("weights_of") is not None:
            continue
        m, p, ff = lc["mixer"], f"l{i}.", lc.get("mlp")
        w[p + "norm1"] = gain(D)
        if lc["type"] == "delta":
            rule(p + "mix.", m, False)
        elif lc["type"] == "retention":
            for name, d in (("q", m["dim"]), ("k", m["dim"]), ("v", m["vdim"]), ("g", m["vdim"])):
                w[p + "mix." + name] = r(m["heads"] * d, D)
            w[p + "mix.o"] = r(D, m["heads"] * m["vdim"])
        else:
            a, s = m["left"], p + "mix.left."
            w[s + "q"], w[s + "k"] = r(a["heads"] * a["dim"], D), r(a["kv_heads"] * a["dim"], D)
            w[s + "q.norm"], w[s + "k.norm"], w[s + "o"] = gain(a["dim"]), gain(a["dim"]), r(D, a["heads"] * a["dim"])
            w[s + "temp"], w[s + "sink"] = gain(a["heads"]), r(a["heads"], std=1.5)
            rule(p + "mix.right.", m["right"], True)
        if ff:
            w[p + "mlp.up"], w[p + "mlp.down"] = r(ff["ff"], D), r(D, ff["ff"])
    return w


def save_checkpoint(path, cfg, w):
    """config.json + model.safetensors (bfloat16) in ``path``."""
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.bfloat16().contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
    return str(path)
