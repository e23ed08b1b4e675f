"""Plain-PyTorch implementations of the head-mixing attention's and parallel layers' ops (``ops/mixed.py``): the CPU data
path.  Token by token; math in fp32, outputs in the activation dtype (bf16 or fp32).
"""
from __future__ import annotations

import torch

from . import reference as ref
from .reference_mixers import clamped_glu, norm, turn


def put_columns(out, y, col, K, packed):
    """Columns [col, col + n) of ``out`` [T, K], row-major or packed."""
    T, n = y.shape
    if not packed:
        out.view(-1)[: T * K].view(T, K)[:, col:col + n] = y.to(out.dtype)
        return out
    x = ref.unpack_act(out, T, K).clone()
    x[:, col:col + n] = y.to(out.dtype)
    return ref.pack_act(x, out=out)


def ffn_act(z, kind, F, block, limit):
    z = z.float()
    if kind == "gelu":
        u = z[:, :F]
        return 0.5 * u * (1.0 + torch.erf(u * 0.5 ** 0.5))
    y = clamped_glu(z[:, : 2 * F], block, limit)
    return y * torch.sigmoid(z[:, 2 * F: 2 * F + 1]) if kind == "gated_glu" else y


def pairs(x):
    """[.., V] -> the cache's column order: pair m in columns 2 m, 2 m + 1."""
    return torch.stack(x.chunk(2, -1), -1).flatten(-2)


def unpairs(x):
    return torch.cat([x[..., 0::2], x[..., 1::2]], -1)


def _views(cache, D, V):
    """Key rows [pages, G, page, D] and value columns [pages, G, page / B, V, B] of a cache [pages, G, page, D + V]."""
    P, G, page, _ = cache.shape
    B = min(32, page)
    flat = cache.view(P, G, page * (D + V))
    return flat[..., : page * D].view(P, G, page, D), flat[..., page * D:].view(P, G, page // B, V, B)


def mixed_prep(z, q_gain, k_gain, qn, cache, slots, q_ctx, rope, vrope, eps):
    T, D, V, G = z.shape[0], q_gain.numel(), vrope.shape[1], cache.shape[1]
    H = qn.shape[1] // D
    z = z.float()
    pos = (q_ctx.long() - 1).clamp(min=0)
    cs = rope[pos][:, None]
    q = turn(norm(z[:, : H * D].reshape(T, H, D), q_gain, eps, False), cs)
    k = turn(norm(z[:, H * D:(H + G) * D].reshape(T, G, D), k_gain, eps, False), cs)
    v = turn(z[:, (H + G) * D:(H + G) * D + G * V].reshape(T, G, V), vrope[pos][:, None])
    qn.copy_(q.reshape(T, H * D))
    kc, vc = _views(cache, D, V)
    page, B = cache.shape[2], vc.shape[-1]
    ok = slots >= 0
    s = slots[ok]
    pg, off = s // page, s % page
    kc[pg, :, off] = k[ok].to(cache.dtype)
    vc[pg, :, off // B, :, off % B] = pairs(v[ok]).to(cache.dtype)


def mixed_attention(z, qn, talk, cache, table, q_seq, q_ctx, vrope, scale, cap):
    H, G, V, T = talk.shape[0], cache.shape[1], vrope.shape[1], z.shape[0]
    D = cache.shape[3] - V
    kc, vc = _views(cache, D, V)
    page, B, rep = cache.shape[2], vc.shape[-1], H // G
    q = qn.float().view(T, H, D)
    gate = torch.sigmoid(z[:, H * D + G * (D + V):][:, :H].float())
    out = torch.zeros(T, H, V, device=z.device)
    for t in range(T):
        n = int(q_ctx[t])
        if n <= 0:
            continue
        j = torch.arange(n, device=z.device)
        pg, off = table[int(q_seq[t])][j // page].long(), j % page
        k = kc[pg, :, off].float().repeat_interleave(rep, 1)
        v = vc[pg, :, off // B, :, off % B].float().repeat_interleave(rep, 1)
        s = torch.einsum("hd,jhd->hj", q[t], k) * scale
        if cap > 0:
            s = cap * torch.tanh(s / cap)
        p = torch.softmax(torch.cat([s, s.new_zeros(H, 1)], 1), -1)[:, :n]  # (a sink of score 0)
        o = unpairs(torch.einsum("hj,jhv->hv", talk @ p, v))
        cs = vrope[n - 1].clone()
        cs[V // 2:] *= -1.0
        out[t] = turn(o, cs) * gate[t][:, None]
    return out.reshape(T, H * V)
