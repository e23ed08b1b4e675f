"""Plain-PyTorch implementations of the hybrid decoders' ops: the CPU data path.

Token by token; math in fp32, outputs in the activation dtype (bf16 or fp32).
"""
from __future__ import annotations

import torch


def sinusoid(positions, inv, width):
    a = positions.double()[:, None] * inv[None, :]
    out = torch.empty(positions.numel(), width, dtype=torch.float32, device=positions.device)
    out[:, 0::2] = torch.sin(a).float()
    out[:, 1::2] = torch.cos(a).float()[:, : width // 2]
    return out


def embed_pos(ids, table, positions, inv, res):
    res.copy_(table[ids.long()].float() + sinusoid(positions, inv, table.shape[1]))


def _unit(x, eps):
    x = x.float()
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def residual_norm(y, res, w, eps):
    res.add_(_unit(y, eps) * w)


def rows_norm(res, rows, w, eps):
    return _unit(res.index_select(0, rows.long()), eps) * w


def relu2(x):
    a = torch.clamp(x.float(), min=0)
    return a * a


def hgrn2(z, bias, lower, norm, state, q_seq, q_ctx, eps):
    """z [T, H (2 D + V)] in flat token order (a session's tokens in sequence); ``state`` is updated."""
    T = z.shape[0]
    _, H, D, V = state.shape
    z = z.float()
    q = torch.nn.functional.silu(z[:, : H * D]).view(T, H, D)
    f = (lower + (1 - lower) * torch.sigmoid(z[:, H * D: 2 * H * D] + bias)).view(T, H, D)
    v = z[:, 2 * H * D:].view(T, H, V)
    o = torch.zeros(T, H, V, device=z.device)
    for t in range(T):
        if int(q_ctx[t]) <= 0:
            continue
        S = state[int(q_seq[t])]
        if int(q_ctx[t]) == 1:
            S.zero_()
        S.mul_(f[t].unsqueeze(-1)).add_((1 - f[t]).unsqueeze(-1) * v[t].unsqueeze(1))
        o[t] = torch.einsum("hd,hdv->hv", q[t], S)
    return (_unit(o, eps) * norm).reshape(T, H * V)


def talk_prep(z, wqk, qn, cache, rk, slots, eps):
    T, HD = qn.shape
    P, G, ps, D = cache.shape
    k = z[:, HD: HD + G * D]
    qn.copy_((_unit(z[:, :HD], eps) * wqk).to(qn.dtype))
    r = 1.0 / torch.sqrt(k.float().pow(2).mean(-1) + eps)
    ok = slots >= 0
    s = slots[ok]
    cache[s // ps, :, s % ps, :] = k[ok].reshape(-1, G, D).to(cache.dtype)
    rk[s // ps, s % ps] = r[ok]


def talk_attention(z, qn, talk, cache, rk, table, q_seq, q_ctx, chunk, scale):
    T, HD = qn.shape
    P, G, ps, D = cache.shape
    H = HD // D
    rep = H // G
    slope = torch.exp2(-8.0 * torch.arange(1, H + 1, dtype=torch.float32, device=z.device) / H)
    gate = torch.sigmoid(z[:, HD + G * D:].float())
    out = torch.zeros(T, HD, device=z.device)
    for t in range(T):
        n = int(q_ctx[t])
        if n <= 0:
            continue
        i = n - 1
        j = torch.arange(i // chunk * chunk, n, device=z.device)
        pg = table[int(q_seq[t])][j // ps].long()
        kv = cache[pg, :, j % ps, :].float()                     # [n, G, D]
        r = rk[pg, j % ps]
        q = qn[t].float().view(G, rep, D)
        s = torch.einsum("gad,ngd->gan", q, kv).reshape(H, -1) * (scale * r) - slope[:, None] * (i - j).float()
        p = torch.softmax(talk @ s, -1).view(G, rep, -1)
        out[t] = torch.einsum("gan,ngd->gad", p, kv).reshape(HD)
    return out * gate
