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


def _epilogue(c, epi, param):
    from .lm import EPI_CLAMP_GLU, EPI_SOFTCAP
    if epi == EPI_CLAMP_GLU:
        g = c[..., 0::2].clamp(max=param)
        u = c[..., 1::2].clamp(-param, param)
        return g * torch.sigmoid(1.702 * g) * (u + 1.0)
    if epi == EPI_SOFTCAP:
        return param * torch.tanh(c / param)
    return c


def matmul(a, w, out_dtype, epi, param, plan=None, gather=False):
    if plan is None:
        return _epilogue(a.float() @ w.float().T, epi, param).to(out_dtype)
    rows = a[plan.token_of.long()] if gather else a
    off = plan.offsets.tolist()
    parts = [_epilogue(rows[off[e]:off[e + 1]].float() @ w[e].float().T, epi, param)
             for e in range(w.shape[0]) if off[e + 1] > off[e]]
    return torch.cat(parts, 0).to(out_dtype)


def route(logits, top, groups, keep):
    s = torch.softmax(logits.float(), -1)
    T, E = s.shape
    best = s.view(T, groups, E // groups).amax(-1)
    ok = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, best.topk(keep, -1).indices, True)
    w, ids = s.masked_fill(~ok.repeat_interleave(E // groups, 1), -1.0).topk(top, -1)
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


def chunk_attention(qkvg, k_cache, v_cache, batch, heads, chunk, scale):
    G, dk, dv = k_cache.shape[1], k_cache.shape[3], v_cache.shape[3]
    T = qkvg.shape[0]
    q, k, v, gate = qkvg[:, :heads * dk + G * (dk + dv) + heads].split([heads * dk, G * dk, G * dv, heads], -1)
    for t, slot in enumerate(batch.slots[:T].tolist()):
        if slot >= 0:
            k_cache[slot // 64, :, slot % 64] = k[t].view(G, dk)
            v_cache[slot // 64, :, slot % 64] = v[t].view(G, dv)
    o = torch.zeros(T, heads, dv)
    for b in range(batch.B):
        n_q = int(batch.q_lens[b]) if batch.is_prefill else 1
        row0 = int(batch.q_start[b]) if batch.is_prefill else b
        ctx = int(batch.ctx_lens[b])
        bt = batch.block_table[b].long()
        for i in range(n_q):
            pos = ctx - n_q + i
            key = torch.arange(pos // chunk * chunk, pos + 1)
            kk = k_cache[bt[key // 64], :, key % 64].float().repeat_interleave(heads // G, 1)   # [n, H, dk]
            vv = v_cache[bt[key // 64], :, key % 64].float().repeat_interleave(heads // G, 1)
            s = torch.einsum("hd,nhd->hn", q[row0 + i].float().view(heads, dk), kk) * scale
            o[row0 + i] = torch.einsum("hn,nhd->hd", torch.softmax(s, -1), vv)
    return (o * torch.sigmoid(gate.float())[..., None]).reshape(T, heads * dv).to(qkvg.dtype)
