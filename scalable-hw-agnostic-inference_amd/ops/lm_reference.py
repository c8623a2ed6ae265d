"""CPU implementations of :mod:`shai_amd.ops.lm` (fp32 math, outputs in the op's dtype) for tests without a GPU."""
from __future__ import annotations

import torch


def _norm(x, w, eps, width):
    return x * torch.rsqrt(x.pow(2).sum(-1, keepdim=True) / width + eps) * (1.0 + w.float())


def embed_norm(ids, prev, table, bigram, mul_prev, mul_cur, w, eps, width):
    ids = ids.long()
    x = table[ids].float()
    if bigram is not None:
        buckets = bigram.shape[0] - 1
        row = (prev.long() * mul_prev + ids * mul_cur) % buckets
        x = x + bigram[torch.where(prev < 0, torch.full_like(row, buckets), row)].float()
    return x, _norm(x, w, eps, width).to(table.dtype)


def add_norm(x, delta, inject, w, eps, width, dtype, rows=None):
    from .lm import Experts
    y = x if rows is None else x.clone()
    if isinstance(delta, Experts):
        y += (delta.y.float()[delta.slot_of.long()] * delta.weights[..., None]).sum(1)
        delta = delta.dense
    if delta is not None:
        y += delta.float()
    if inject is not None:
        y += inject
    if w is None:
        return None
    if rows is not None:
        y = y[rows.long()]
    return _norm(y, w, eps, width).to(dtype)


def _gelu_tanh(z):
    return torch.nn.functional.gelu(z, approximate="tanh")


def _epilogue(c, epi, param, vec=None, rope=None, head=0, rot0=0, ids=None, table=None):
    from .lm import EPI_CLAMP_GLU, EPI_GELU_GLU, EPI_GELU_ROWS, EPI_RELU2, EPI_ROTARY, EPI_SOFTCAP, EPI_XIELU
    if epi == EPI_GELU_GLU:
        return _gelu_tanh(c[..., 0::2]) * c[..., 1::2]
    if epi == EPI_RELU2:
        return torch.relu(c) ** 2
    if epi == EPI_GELU_ROWS:
        return _gelu_tanh(c) * table[ids.long()].float()
    if epi == EPI_CLAMP_GLU:
        g = c[..., 0::2].clamp(max=param)
        u = c[..., 1::2].clamp(-param, param)
        return g * torch.sigmoid(1.702 * g) * (u + 1.0)
    if epi == EPI_SOFTCAP:
        return param * torch.tanh(c / param)
    if epi == EPI_XIELU:
        return torch.where(c > 0, vec[0] * c * c, vec[1] * (torch.expm1(c) - c)) + 0.5 * c
    if epi == EPI_ROTARY:
        c = c.view(c.shape[0], -1, head).clone()
        rot = rope.shape[1]
        c[..., rot0:rot0 + rot] = _turn(c[..., rot0:rot0 + rot], rope[:, None, :])
        return c.view(c.shape[0], -1)
    return c


def _turn(x, rope):
    u, v, cs, sn = x[..., 0::2], x[..., 1::2], rope[..., 0::2], rope[..., 1::2]
    return torch.stack([u * cs - v * sn, v * cs + u * sn], -1).flatten(-2)


def matmul(a, w, out_dtype, epi, param, plan=None, gather=False, vec=None, rope=None, head=0, rot0=0, ids=None, table=None):
    if plan is None:
        return _epilogue(a.float() @ w.float().T, epi, param, vec, rope, head, rot0, ids, table).to(out_dtype)
    rows = a[plan.token_of.long()] if gather else a
    off = plan.offsets.tolist()
    parts = [_epilogue(rows[off[e]:off[e + 1]].float() @ w[e].float().T, epi, param)
             for e in range(w.shape[0]) if off[e + 1] > off[e]]
    return torch.cat(parts, 0).to(out_dtype)


def route(logits, top, groups, keep, bias=None, renorm=False):
    logits = logits.float() if bias is None else logits.float() + bias
    s = torch.softmax(logits, -1)
    T, E = s.shape
    best = s.view(T, groups, E // groups).amax(-1)
    ok = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, best.topk(keep, -1).indices, True)
    w, ids = s.masked_fill(~ok.repeat_interleave(E // groups, 1), -1.0).topk(top, -1)
    if renorm:
        w = torch.softmax(logits.gather(1, ids), -1)
    return ids.int(), w


def plan_experts(ids, experts, bm):
    from .lm import Plan
    T, top = ids.shape
    flat = ids.reshape(-1).long()
    order = torch.argsort(flat, stable=True)
    slot_of = torch.empty(T * top, dtype=torch.int32)
    slot_of[order] = torch.arange(T * top, dtype=torch.int32)
    off = torch.zeros(experts + 1, dtype=torch.int32)
    off[1:] = torch.bincount(flat, minlength=experts).cumsum(0).int()
    return Plan(off, (order // top).int(), slot_of.view(T, top), torch.empty(0, 2, dtype=torch.int32), bm)


def _turn_heads(x, dim_pad, turn, gain=None):
    """Rotation (dimension i with i + rot / 2) and rms norm of every head of x [T, heads * dim_pad]; with a gain the norm
    comes first."""
    x = x.float().reshape(x.shape[0], -1, dim_pad).clone()
    rms = lambda x: x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) / turn.dim + turn.eps)
    if gain is not None:
        x = rms(x) * gain
    x = _rotate_half(x, turn.rope)
    return rms(x) if gain is None else x


def _rotate_half(x, rope):
    x, half = x.clone(), rope.shape[1] // 2
    cs, sn = rope[:, None, 0::2], rope[:, None, 1::2]
    u, v = x[..., :half].clone(), x[..., half:2 * half].clone()
    x[..., :half], x[..., half:2 * half] = u * cs - v * sn, v * cs + u * sn
    return x


def gated_attention(qkvg, k_cache, v_cache, batch, heads, size, scale, window, per_element, own_kv, turn, plain=None):
    G, dk, dv = k_cache.shape[1], k_cache.shape[3], v_cache.shape[3]
    T = qkvg.shape[0]
    if plain is not None:
        q, k = qkvg[:, :(heads + G) * dk].split([heads * dk, G * dk], -1)
        v = k
    else:
        n_gate, kv = heads * (dv if per_element else 1), (G * dk, G * dv) if own_kv else (0, 0)
        q, k, v, gate = qkvg[:, :heads * dk + sum(kv) + n_gate].split([heads * dk, *kv, n_gate], -1)
    if turn is not None:
        q = _turn_heads(q, dk, turn, turn.q_gain).to(qkvg.dtype).view(T, -1)
        k = _turn_heads(k, dk, turn, turn.k_gain).to(qkvg.dtype).view(T, -1) if own_kv else k
    scale = torch.full((heads,), scale) if plain is None else scale * plain.temp
    for t, slot in enumerate(batch.slots[:T].tolist()):
        if slot >= 0 and own_kv:
            k_cache[slot // 64, :, slot % 64] = k[t].reshape(G, dk)
            v_cache[slot // 64, :, slot % 64] = v[t].reshape(G, dv)
    o = torch.zeros(T, heads, dv)
    for b in range(batch.B):
        n_q = int(batch.q_lens[b]) if batch.is_prefill else 1
        row0 = int(batch.q_start[b]) if batch.is_prefill else b
        ctx = int(batch.ctx_lens[b])
        bt = batch.block_table[b].long()
        for i in range(n_q):
            pos = ctx - n_q + i
            key = torch.arange(max(0, pos - size + 1) if window else pos // size * size, pos + 1)
            kk = k_cache[bt[key // 64], :, key % 64].float().repeat_interleave(heads // G, 1)   # [n, H, dk]
            vv = v_cache[bt[key // 64], :, key % 64].float().repeat_interleave(heads // G, 1)
            s = torch.einsum("hd,nhd->hn", q[row0 + i].float().reshape(heads, dk), kk) * scale[:, None]
            p = torch.softmax(s, -1) if plain is None else _sink_softmax(s, plain.sink)
            o[row0 + i] = torch.einsum("hn,nhd->hd", p, vv)
    if plain is not None:
        plain.out.copy_((o * plain.out_scale).view(T, heads * dv))
        return plain.out
    return (o * torch.sigmoid(gate.float()).view(T, heads, -1)).reshape(T, heads * dv).to(qkvg.dtype)


def _sequences(batch):
    """(first row, rows, first position, state slot, sequence) of every sequence of a step."""
    for b in range(batch.B):
        row0 = int(batch.q_start[b]) if batch.is_prefill else b
        n = int(batch.q_lens[b]) if batch.is_prefill else 1
        yield row0, n, int(batch.positions[row0]), int(batch.state_slots[b]), b


def residual_norm(source, delta, wb, mult, step, w, eps, width, dtype, conv, batch, rows, keep):
    from .lm import PLAIN, Affine, Embedding, Experts

    def rms(t, w):
        gain, bias = w if isinstance(w, Affine) else (w, None)
        if w is None or w is PLAIN:
            return t
        if bias is not None:
            mean = t.sum(-1, keepdim=True) / width
            t = torch.where(torch.arange(t.shape[-1]) < width, t - mean, torch.zeros(()))
        y = t / torch.sqrt(t.pow(2).sum(-1, keepdim=True) / width + eps) * gain
        return y if bias is None else y + bias
    if isinstance(delta, Experts):
        delta = (delta.y.float()[delta.slot_of.long()] * delta.weights[..., None]).sum(1)
    x = source.table[source.ids.long()].float() * source.scale if isinstance(source, Embedding) else source.clone()
    if delta is not None:
        x = x + mult * rms(delta.float(), wb)
    if step is not None:
        x = x + step
    if w is None:
        return x, None
    if rows is not None:
        return (x if keep else None), rms(x[rows.long()], w).to(dtype)
    h = rms(x, w)
    if conv is not None:
        y, k = h.clone(), conv.weight.shape[0] - 1
        for row0, n, pos, slot, b in _sequences(batch):
            past = conv.state[slot] if slot >= 0 else torch.zeros(k, h.shape[1])
            past = past * (torch.arange(k) >= k - pos)[:, None] if pos < k else past
            line = torch.cat([past, h[row0:row0 + n]])
            for j in range(k + 1):
                y[row0:row0 + n] += conv.weight[j] * line[j:j + n]
            if conv.tail is not None:
                conv.tail[b, k - min(n, k):] = line[n + k - min(n, k):]
            elif slot >= 0:
                conv.state[slot] = line[n:]
        h = y
    return x, h.to(dtype)


def conv_commit(state, tail, batch):
    k = state.shape[2]
    for _, n, _, slot, b in _sequences(batch):
        if slot >= 0:
            state[:, slot] = torch.cat([state[:, slot], tail[:, b, k - min(n, k):]], 1)[:, -k:] if k else state[:, slot]


def rope_rows(positions, freq):
    a = positions.double()[:, None] * freq.double().sum(1)
    return torch.stack([a.cos(), a.sin()], -1).flatten(1).float()


def latent_prep(d, wq, wkv, rope, batch, cache, eps, q_rank, kv_rank):
    qp, rp = wq.shape[0], wkv.shape[0]
    rms = lambda t, n, gain: t / torch.sqrt(t.pow(2).sum(-1, keepdim=True) / n + eps) * gain
    turn = d[:, qp + rp:].clone()
    turn[:, :rope.shape[1]] = _turn(turn[:, :rope.shape[1]], rope)
    row = torch.cat([rms(d[:, qp:qp + rp], kv_rank, wkv), turn], 1).to(cache.dtype)
    for t, slot in enumerate(batch.slots[:d.shape[0]].tolist()):
        if slot >= 0:
            cache[slot // 64, slot % 64] = row[t]
    return rms(d[:, :qp], q_rank, wq).to(cache.dtype)


def _sink_softmax(s, sink):
    return torch.softmax(torch.cat([s, sink[:, None]], 1), 1)[:, :-1]


def latent_rows(ql, q, cache, block_table, plan, sink, np_, rot, scale):
    n, H, rp = ql.shape
    qr = q.view(n, H, -1)[..., np_:np_ + rot].float()
    o = torch.zeros(n, H, rp)
    for i, ctx in enumerate(plan.ctx[:n].tolist()):
        key = torch.arange(ctx)
        bt = block_table[int(plan.seqs[i]) if plan.seqs is not None else i].long()
        row = cache[bt[key // 64], key % 64].float()
        s = (ql[i].float() @ row[:, :rp].T + qr[i] @ row[:, rp:rp + rot].T) * scale
        o[i] = _sink_softmax(s, sink) @ row[:, :rp]
    return o.to(ql.dtype)


def latent_gather(cache, block_table, g):
    key = lambda n: torch.arange(n)
    return torch.cat([cache[block_table[b].long()[key(n) // 64], key(n) % 64]
                      for b, n in zip(g.seqs.tolist(), g.ctx.tolist())])


def latent_prefill(q, kv, lat, o, g, sink, heads, np_, rot, rank, scale):
    ov = o.view(o.shape[0], heads, -1)
    for ctx, n, row0, k0 in zip(*(t.tolist() for t in (g.ctx, g.q_lens, g.q_start, g.kv_start))):
        qs = q[row0:row0 + n].view(n, heads, -1).float()
        kvs = kv[k0:k0 + ctx].view(ctx, heads, -1).float()
        turn = lat[k0:k0 + ctx, rank:rank + rot].float()
        hide = torch.arange(ctx)[None, :] > torch.arange(ctx - n, ctx)[:, None]
        for h in range(heads):
            s = qs[:, h, :np_] @ kvs[:, h, :np_].T + qs[:, h, np_:np_ + rot] @ turn.T
            p = _sink_softmax((s * scale).masked_fill(hide, float("-inf")), sink[h].expand(n))
            ov[row0:row0 + n, h] = (p @ kvs[:, h, np_:]).to(o.dtype)


def mingru_scan(zx, g, bias, state, batch):
    z, u = (zx + bias).chunk(2, 1)
    keep, cand = torch.sigmoid(-z), torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    add, S = torch.sigmoid(z) * cand, torch.zeros_like(z)
    for row0, n, pos, slot, _ in _sequences(batch):
        s = state[slot].clone() if slot >= 0 and pos > 0 else torch.zeros_like(z[0])
        for t in range(row0, row0 + n):
            s = keep[t] * s + add[t]
            S[t] = s
        if slot >= 0:
            state[slot] = s
    return (S * torch.nn.functional.silu(g.float())).to(g.dtype)


def hgrn2(qv, z, bias, lower, gain, state, batch, vdim, eps):
    _, H, dk, dv = state.shape
    T = qv.shape[0]
    q = torch.nn.functional.silu(qv[:, :H * dk].float()).view(T, H, dk)
    v = qv[:, H * dk:].float().view(T, H, dv)
    f = (lower + (1 - lower) * torch.sigmoid(z + bias)).view(T, H, dk)
    k = ((1 - lower) * torch.sigmoid(-(z + bias))).view(T, H, dk)
    o = torch.zeros(T, H, dv)
    for row0, n, pos, slot, _ in _sequences(batch):
        S = state[slot].clone() if slot >= 0 and pos > 0 else torch.zeros(H, dk, dv)
        for t in range(row0, row0 + n):
            S = f[t][..., None] * S + k[t][..., None] * v[t][:, None]
            o[t] = (S * q[t][..., None]).sum(1)
        if slot >= 0:
            state[slot] = S
    return (o / torch.sqrt(o.pow(2).sum(-1, keepdim=True) / vdim + eps) * gain).reshape(T, H * dv).to(qv.dtype)


def _gate(z, kind):
    return torch.nn.functional.silu(z) if kind == 0 else torch.sigmoid(z)


def _rule_out(o, gain, gate, out, shape, eps):
    T, H, dv = o.shape
    o = o / torch.sqrt(o.pow(2).sum(-1, keepdim=True) / shape.vdim + eps)
    if gain is not None:
        o = o * gain
    out.copy_(o.reshape(T, H * dv) * _gate(gate.float(), shape.gate))


def delta_rule(x, gate, decay, beta, conv, rate, bias, gain, state, ring, batch, out, shape, eps):
    _, H, dk, dv = state.shape
    T, G, taps, C = x.shape[0], shape.kv_heads, conv.shape[0], conv.shape[1]
    x = x.float()
    y = torch.zeros(T, C)
    for row0, n, pos, slot, _ in _sequences(batch):
        past = torch.zeros(taps - 1, C)
        for j in range(1, taps):
            if pos - j >= 0 and slot >= 0:
                past[-j] = ring[slot, (pos - j) % taps].float()
        line = torch.cat([past, x[row0:row0 + n]])
        for j in range(taps):
            y[row0:row0 + n] += conv[j] * line[j:j + n]
        if slot >= 0:
            for t in range(max(0, n - taps), n):
                ring[slot, (pos + t) % taps] = x[row0 + t].to(ring.dtype)
    y = torch.nn.functional.silu(y)
    unit = lambda t: t / torch.sqrt(t.pow(2).sum(-1, keepdim=True) + 1e-6)
    q, k, v = y.split([G * dk, G * dk, H * dv], 1)
    q = (unit(q.reshape(T, G, dk)) * shape.dim ** -0.5).repeat_interleave(H // G, 1)
    k, v = unit(k.reshape(T, G, dk)).repeat_interleave(H // G, 1), v.reshape(T, H, dv)
    g = torch.exp(-rate[:, None] * torch.nn.functional.softplus(decay.float() + bias).reshape(T, H, -1))
    b, o = torch.sigmoid(beta.float()), torch.zeros(T, H, dv)
    for row0, n, pos, slot, _ in _sequences(batch):
        S = state[slot].clone() if slot >= 0 and pos > 0 else torch.zeros(H, dk, dv)
        for t in range(row0, row0 + n):
            S = g[t][..., None] * S
            u = b[t][:, None] * (v[t] - (S * k[t][..., None]).sum(1))
            S = S + k[t][..., None] * u[:, None]
            o[t] = (S * q[t][..., None]).sum(1)
        if slot >= 0:
            state[slot] = S
    _rule_out(o, gain, gate, out, shape, eps)


def retention(x, gate, decay, rope, state, batch, out, shape, eps):
    _, H, dk, dv = state.shape
    T = x.shape[0]
    q, k, v = x.float().split([H * dk, H * dk, H * dv], 1)
    q = _rotate_half(q.reshape(T, H, dk), rope)
    k, v = _rotate_half(k.reshape(T, H, dk), rope) * shape.dim ** -0.5, v.reshape(T, H, dv)
    o = torch.zeros(T, H, dv)
    for row0, n, pos, slot, _ in _sequences(batch):
        S = state[slot].clone() if slot >= 0 and pos > 0 else torch.zeros(H, dk, dv)
        for t in range(row0, row0 + n):
            S = decay[0][:, None, None] * S + k[t][..., None] * v[t][:, None]
            o[t] = (S * q[t][..., None]).sum(1)
        if slot >= 0:
            state[slot] = S
    _rule_out(o, None, gate, out, shape, eps)
