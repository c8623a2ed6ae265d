"""Plain, slow fp64 implementation of the Faledra decoder, one function per mechanism, written from the model's equations.
Shares no code with ``shai_amd``: tests compare the framework with it.

``cfg`` is the parsed config.json, ``w`` a dict of full tensors under their checkpoint names.  A whole sequence is
recomputed from its first token, so there is no cache, no batch and no state to get wrong."""
import json
import os

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def embed(tokens, cfg, w):
    return w["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]


def causal_conv(h, w):
    """Channel by channel: sum over j of w[:, j] * h at the position (taps - 1 - j) before; h [n, D], w [D, taps]."""
    n, taps = h.shape[0], w.shape[1]
    out = torch.zeros_like(h)
    for t in range(n):
        for j in range(taps):
            if t - (taps - 1 - j) >= 0:
                out[t] += w[:, j] * h[t - (taps - 1 - j)]
    return out


def rotate(x, base, first=0):
    """Interleaved pairs of the last axis turned by position * base^(-2 i / dims); x [n, ..., dims], row t is position
    ``first`` + t."""
    n, dims = x.shape[0], x.shape[-1]
    out = torch.empty_like(x)
    for i in range(dims // 2):
        a = (torch.arange(n, dtype=x.dtype) + first) * base ** (-2.0 * i / dims)
        a = a.reshape([n] + [1] * (x.dim() - 2))
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return out


def attend(q, k, v, sink, scale):
    """q [n, H, dk], k [n, H, dk], v [n, H, dv], sink [H] -> [n, H * dv]: causal, a constant term in the denominator."""
    n, H = q.shape[:2]
    see = torch.tril(torch.ones(n, n, dtype=torch.bool))
    outs = []
    for hd in range(H):
        s = ((q[:, hd] @ k[:, hd].T) * scale).masked_fill(~see, float("-inf"))
        top = torch.maximum(s.amax(-1, keepdim=True), sink[hd])
        e = torch.exp(s - top)
        outs.append((e @ v[:, hd]) / (e.sum(-1, keepdim=True) + torch.exp(sink[hd] - top)))
    return torch.cat(outs, -1)


def latent_attention(h, mc, eps, get):
    """h [n, width] -> [n, width]; ``get(name)`` returns the mixer's tensor."""
    n, H, d, r, R = h.shape[0], mc["heads"], mc["dim"], mc["rot_dim"], mc["kv_rank"]
    base = mc["rot"]["base"]
    q = (rms_norm(h @ get("dq").T, get("dq.norm"), eps) @ get("uq").T).view(n, H, d + r)
    q = torch.cat([q[..., :d], rotate(q[..., d:], base)], -1)
    low = h @ get("dkv").T
    c = rms_norm(low[:, :R], get("dkv.norm"), eps)
    turn = rotate(low[:, R:], base)
    k = torch.cat([(c @ get("uk").T).view(n, H, d), turn[:, None, :].expand(n, H, r)], -1)
    v = (c @ get("uv").T).view(n, H, mc["vdim"])
    return attend(q, k, v, get("sink"), mc["scale"]) @ get("o").T


def mingru_states(z, u):
    """S of every position from gate logits z and candidate inputs u, both [n, width]."""
    keep = 1.0 / (1.0 + torch.exp(z))
    cand = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    S, out = torch.zeros_like(z[0]), []
    for t in range(z.shape[0]):
        S = keep[t] * S + (1.0 - keep[t]) * cand[t]
        out.append(S)
    return torch.stack(out)


def mingru(h, get):
    S = mingru_states(h @ get("z").T + get("z.b"), h @ get("x").T + get("x.b"))
    g = h @ get("g").T
    return (S * g * torch.sigmoid(g)) @ get("o").T


def xielu(z, p, q):
    sp = lambda t: torch.log1p(torch.exp(t))
    return torch.where(z > 0, sp(p) * z * z, (0.5 + sp(q)) * (torch.expm1(z) - z)) + 0.5 * z


def feed_forward(h, get):
    p, q = get("act")
    return xielu(h @ get("up").T, p, q) @ get("down").T


def layer_order(cfg):
    """[(layer index, pass whose step vector is added before it, or None)] in execution order."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    order = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        order += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return order + [(i, None) for i in range(lp["stop"], n)]


def forward(tokens, cfg, w, dtype=torch.float64):
    """(logits [n, vocab], [residual stream after every layer run])."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = embed(list(tokens), cfg, w)
    trail = []
    for i, turn in layer_order(cfg):
        lc, p = cfg["layers"][i], f"l{i}."
        get = lambda n, b: w[p + b + "." + n]
        if turn is not None:
            x = x + w["loop.step"][turn]
        h = rms_norm(x, w[p + "norm1"], eps)
        h = h + causal_conv(h, w[p + "canon1"])
        if lc["type"] == "latent_attention":
            y = latent_attention(h, lc["mixer"], eps, lambda n: get(n, "mix"))
        else:
            y = mingru(h, lambda n: get(n, "mix"))
        x = x + m * rms_norm(y, w[p + "norm1b"], eps)
        if lc.get("mlp"):
            y = feed_forward(rms_norm(x, w[p + "norm2"], eps), lambda n: get(n, "mlp"))
            x = x + m * rms_norm(y, w[p + "norm2b"], eps)
        trail.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T, trail


def attention_layer(heads=3, dim=20, rot_dim=6, vdim=28, q_rank=36, kv_rank=44, base=300.0, scale=0.2, ff=40):
    return {"type": "latent_attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank,
                      "kv_rank": kv_rank, "rot": {"base": base, "dims": rot_dim}, "scale": scale}}


def mingru_layer(width=52, ff=40):
    return {"type": "mingru", "mixer": {"width": width}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def random_config(layers=None, vocab=97, width=56, taps=3, embed_scale=2.5, eps=1e-4, mult=0.6, loop=(1, 3, 2)):
    layers = layers or [mingru_layer(), attention_layer(), mingru_layer(36, 24), attention_layer(heads=2, kv_rank=70)]
    c = {"architecture": "Faledra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "canon": {"taps": taps},
         "embedding": {"scale": embed_scale}, "residual_mult": mult, "layers": layers}
    if loop:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


def random_weights(cfg, seed=0):
    """bfloat16-exact random weights under their checkpoint names (fp32 tensors)."""
    g = torch.Generator().manual_seed(seed)
    b = lambda t: t.bfloat16().float()
    r = lambda *s, std=None: b(torch.randn(*s, generator=g) * (s[-1] ** -0.5 if std is None else std))
    gain = lambda n: b(1.0 + 0.3 * torch.randn(n, generator=g))
    D = cfg["width"]
    w = {"embed": r(cfg["vocab"], D, std=0.5), "final.norm": gain(D), "head": r(cfg["vocab"], D)}
    if cfg.get("loop"):
        w["loop.step"] = r(cfg["loop"]["times"], D, std=0.7)
    for i, lc in enumerate(cfg["layers"]):
        m, p = lc["mixer"], f"l{i}."
        w[p + "norm1"], w[p + "norm1b"] = gain(D), gain(D)
        w[p + "canon1"] = r(D, cfg["canon"]["taps"], std=0.5)
        if lc["type"] == "latent_attention":
            H, d, rd, vd, Q, R = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"))
            w[p + "mix.dq"], w[p + "mix.dq.norm"], w[p + "mix.uq"] = r(Q, D), gain(Q), r(H * (d + rd), Q, std=2 * Q ** -0.5)
            w[p + "mix.dkv"], w[p + "mix.dkv.norm"] = r(R + rd, D), gain(R)
            w[p + "mix.uk"], w[p + "mix.uv"] = r(H * d, R), r(H * vd, R)
            w[p + "mix.sink"], w[p + "mix.o"] = r(H, std=1.5), r(D, H * vd)
        else:
            W = m["width"]
            for n in ("z", "x"):
                w[p + f"mix.{n}"], w[p + f"mix.{n}.b"] = r(W, D), r(W, std=0.7)
            w[p + "mix.z.b"] = w[p + "mix.z.b"] - 1.0           # slow gates: the state reaches far back
            w[p + "mix.z.b"] = b(w[p + "mix.z.b"])
            w[p + "mix.g"], w[p + "mix.o"] = r(W, D), r(D, W)
        if lc.get("mlp"):
            F = lc["mlp"]["ff"]
            w[p + "norm2"], w[p + "norm2b"] = gain(D), gain(D)
            w[p + "mlp.up"], w[p + "mlp.down"], w[p + "mlp.act"] = r(F, D, std=1.5 * D ** -0.5), r(D, F), r(2, std=0.8)
    return w


def save_checkpoint(path, cfg, w):
    """config.json + model.safetensors (bfloat16) in ``path``."""
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.bfloat16().contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
    return str(path)
