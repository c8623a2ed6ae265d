"""Plain, slow fp32 / fp64 implementation of the Golulix decoder, one function per mechanism, written from the model's
equations.  Shares no code with ``shai_amd``: tests compare the framework with it.

``cfg`` is the parsed config.json, ``w`` a dict of full tensors under their checkpoint names.  A whole sequence is
recomputed from its first token, so there is no cache, no batch and no state to get wrong."""
import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * (1.0 + w)


def bigram_rows(tokens, big):
    """Row of the bigram table for every token; the row after the last bucket for the first one."""
    rows = [big["buckets"]]
    for a, b in zip(tokens[:-1], tokens[1:]):
        rows.append((a * big["mul_prev"] + b * big["mul_cur"]) % big["buckets"])
    return rows


def embed(tokens, cfg, w):
    x = w["embed"][torch.tensor(tokens)]
    big = (cfg.get("embedding") or {}).get("bigram")
    if big:
        x = x + w["bigram"][torch.tensor(bigram_rows(tokens, big))]
    return x


def chunk_visible(n, size):
    """[n, n] bool: query i sees key j."""
    i = torch.arange(n)
    return (i[None, :] <= i[:, None]) & (i[None, :] // size == i[:, None] // size)


def attend(q, k, v, gate, chunk, scale):
    """q [n, H, dk], k [n, G, dk], v [n, G, dv], gate logits [n, H] -> [n, H * dv]."""
    n, H, G = q.shape[0], q.shape[1], k.shape[1]
    see = chunk_visible(n, chunk)
    outs = []
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * scale
        p = torch.softmax(s.masked_fill(~see, float("-inf")), -1)
        outs.append((p @ v[:, g]) * torch.sigmoid(gate[:, hd:hd + 1]))
    return torch.cat(outs, -1)


def attention(h, mc, get):
    """h [n, width] -> [n, width]; ``get(name)`` returns the mixer's tensor."""
    n = h.shape[0]
    H, G, dk, dv = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    q = (h @ get("q").T).view(n, H, dk)
    k = (h @ get("k").T).view(n, G, dk)
    v = (h @ get("v").T).view(n, G, dv)
    return attend(q, k, v, h @ get("g").T, mc["mask"]["size"], mc["scale"]) @ get("o").T


def expert(h, gate, up, down, limit):
    g = torch.clamp(h @ gate.T, max=limit)
    u = torch.clamp(h @ up.T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def route(h, rw, rc):
    """Per token: list of (expert, weight)."""
    s = torch.softmax(h @ rw.T, -1)
    E, n_groups = rc["experts"], (rc.get("groups") or {}).get("count", 1)
    keep = (rc.get("groups") or {}).get("keep", n_groups)
    per = E // n_groups
    out = []
    for row in s.tolist():
        best = sorted(range(n_groups), key=lambda i: -max(row[i * per:(i + 1) * per]))[:keep]
        allowed = [e for e in range(E) if e // per in best]
        top = sorted(allowed, key=lambda e: -row[e])[:rc["top"]]
        out.append([(e, row[e]) for e in top])
    return out


def moe(h, mlp, get):
    y = torch.zeros_like(h)
    for t, picks in enumerate(route(h, get("router"), mlp["router"])):
        for e, s in picks:
            y[t] += s * expert(h[t:t + 1], get(f"e{e}.gate"), get(f"e{e}.up"), get(f"e{e}.down"),
                               mlp["expert"]["limit"])[0]
    if mlp.get("shared"):
        y = y + expert(h, get("shared.gate"), get("shared.up"), get("shared.down"), mlp["shared"]["limit"])
    return y


def layer_order(cfg):
    """[(layer index, whether the embedding output is added before it)] in execution order."""
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    order = [(i, False) for i in range(lp["start"])]
    for t in range(lp["times"]):
        order += [(i, t > 0 and i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return order + [(i, False) for i in range(lp["stop"], n)]


def forward(tokens, cfg, w, dtype=torch.float64):
    """(logits [n, vocab], [residual stream after every layer run])."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x0 = x = embed(list(tokens), cfg, w)
    trail = []
    for i, inject in layer_order(cfg):
        lc = cfg["layers"][i]
        if inject:
            x = x + x0
        x = x + attention(rms_norm(x, w[f"l{i}.norm1"], eps), lc["mixer"], lambda n: w[f"l{i}.mix.{n}"])
        if lc.get("mlp"):
            x = x + moe(rms_norm(x, w[f"l{i}.norm2"], eps), lc["mlp"], lambda n: w[f"l{i}.mlp.{n}"])
        trail.append(x)
    logits = rms_norm(x, w["final.norm"], eps) @ w["head"].T
    cap = cfg.get("logit_softcap")
    if cap:
        logits = cap * torch.tanh(logits / cap)
    return logits, trail


def random_config(vocab=96, width=48, layers=3, heads=4, kv_heads=2, dim=16, vdim=24, chunk=20, scale=0.3, ff=24,
                  limit=1.5, experts=12, top=2, groups=3, keep=1, shared_ff=40, shared_limit=0.75, eps=1e-5, cap=9.0,
                  loop=(1, 2, 3), bigram=(61, 29, 5), no_mlp=()):
    layer = lambda i: {
        "type": "attention",
        "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                  "mask": {"size": chunk if isinstance(chunk, int) else chunk[i % len(chunk)]}},
        "mlp": None if i in no_mlp else {
            "kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}},
            "shared": {"ff": shared_ff, "limit": shared_limit}}}
    c = {"architecture": "Golulix", "vocab": vocab, "width": width, "norm": {"eps": eps},
         "layers": [layer(i) for i in range(layers)], "logit_softcap": cap,
         "embedding": {"bigram": {"buckets": bigram[0], "mul_prev": bigram[1], "mul_cur": bigram[2]}}}
    if loop:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


def random_weights(cfg, seed=0, gain=1.0):
    """bfloat16-exact random weights under their checkpoint names (fp32 tensors)."""
    g = torch.Generator().manual_seed(seed)
    r = lambda *s, std: (torch.randn(*s, generator=g) * std).bfloat16().float()
    D = cfg["width"]
    w = {"embed": r(cfg["vocab"], D, std=1.0), "final.norm": r(D, std=0.2), "head": r(cfg["vocab"], D, std=D ** -0.5)}
    big = cfg["embedding"]["bigram"]
    w["bigram"] = r(big["buckets"] + 1, D, std=0.7)
    for i, lc in enumerate(cfg["layers"]):
        m, p = lc["mixer"], f"l{i}."
        w[p + "norm1"] = r(D, std=0.2)
        s = gain * D ** -0.5
        w[p + "mix.q"], w[p + "mix.k"] = r(m["heads"] * m["dim"], D, std=s), r(m["kv_heads"] * m["dim"], D, std=s)
        w[p + "mix.v"], w[p + "mix.g"] = r(m["kv_heads"] * m["vdim"], D, std=s), r(m["heads"], D, std=s)
        w[p + "mix.o"] = r(D, m["heads"] * m["vdim"], std=(m["heads"] * m["vdim"]) ** -0.5)
        if not lc.get("mlp"):
            continue
        w[p + "norm2"] = r(D, std=0.2)
        mlp = lc["mlp"]
        w[p + "mlp.router"] = r(mlp["router"]["experts"], D, std=2 * s)
        blocks = [(f"e{e}", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
        if mlp.get("shared"):
            blocks.append(("shared", mlp["shared"]["ff"]))
        for name, ff in blocks:
            w[p + f"mlp.{name}.gate"], w[p + f"mlp.{name}.up"] = r(ff, D, std=2 * s), r(ff, D, std=2 * s)
            w[p + f"mlp.{name}.down"] = r(D, ff, std=ff ** -0.5)
    return w


def save_checkpoint(path, cfg, w):
    """config.json + model.safetensors (bfloat16) in ``path``."""
    import json
    import os
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.bfloat16().contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
    return str(path)
