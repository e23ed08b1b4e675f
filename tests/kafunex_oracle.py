"""Plain fp32 / fp64 implementation of the Kafunex decoder, one function per mechanism.

Works on the checkpoint's own tensors (a dict name -> tensor) and the config dict, one sequence at a time, token
by token where the mechanism is recurrent.  Shares no code with the framework: this is what the tests compare it to.
"""
import math

import torch


def rms(x, eps):
    """x over its root mean square (last axis), eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def scalar_norm(x, g, eps):
    return rms(x, eps) * g


def sinusoid(n, width, dt=torch.float64, start=0):
    """[n, width]: sin at even entries, cos at odd ones, frequency 10000^(-2i/width) for the pair i."""
    p = torch.arange(start, start + n, dtype=torch.float64)[:, None]
    i = torch.arange((width + 1) // 2, dtype=torch.float64)[None, :]
    a = p * torch.pow(torch.tensor(10000.0, dtype=torch.float64), -2.0 * i / width)
    out = torch.zeros(n, width, dtype=torch.float64)
    out[:, 0::2] = torch.sin(a)
    out[:, 1::2] = torch.cos(a)[:, : width // 2]
    return out.to(dt)


def forget_gate(zf, b, lower):
    """lower + (1 - lower) sigmoid(zf + b)."""
    return lower + (1 - lower) / (1 + torch.exp(-(zf + b)))


def hgrn2_scan(q, f, v, state=None):
    """q, f [L, H, D], v [L, H, V] -> o [L, H, V], final state [H, D, V]: one token after the other."""
    L, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    o = torch.zeros(L, H, v.shape[-1], dtype=q.dtype)
    for t in range(L):
        S = f[t][:, :, None] * S + (1 - f[t])[:, :, None] * v[t][:, None, :]
        o[t] = (q[t][:, :, None] * S).sum(1)
    return o, S


def hgrn2(w, p, h, m, eps):
    L, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    zq = h @ w[p + "q"].t()
    q = zq / (1 + torch.exp(-zq))
    f = forget_gate(h @ w[p + "f"].t(), w[p + "f.b"], w[p + "lower"])
    v = h @ w[p + "v"].t()
    o, _ = hgrn2_scan(q.view(L, H, D), f.view(L, H, D), v.view(L, H, V))
    o = rms(o, eps) * w[p + "norm"]
    return o.reshape(L, H * V) @ w[p + "o"].t()


def slopes(H, dt=torch.float64):
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], dtype=dt)


def chunk_mask(L, size):
    """[L, L] bool: query i (row) sees key j (column)."""
    i = torch.arange(L)
    return (i[None, :] <= i[:, None]) & (i[None, :] // size == i[:, None] // size)


def talking_scores(q, k, scale, talk):
    """q [L, H, D], k [L, G, D] -> mixed scores [H, L, L] before the mask."""
    L, H, _ = q.shape
    G = k.shape[1]
    i = torch.arange(L, dtype=q.dtype)
    sl = slopes(H, q.dtype)
    raw = torch.stack([q[:, h] @ k[:, h // (H // G)].t() * scale - sl[h] * (i[:, None] - i[None, :])
                       for h in range(H)])
    return torch.stack([sum(talk[h, g] * raw[g] for g in range(H)) for h in range(H)])


def attention_core(q, k, v, scale, talk, size):
    """softmax over the visible keys of the mixed scores; values of kv head floor(h G / H)."""
    L, H, _ = q.shape
    G = k.shape[1]
    s = talking_scores(q, k, scale, talk).masked_fill(~chunk_mask(L, size)[None], -math.inf)
    p = torch.exp(s - s.max(-1, keepdim=True).values)
    p = p / p.sum(-1, keepdim=True)
    return torch.stack([p[h] @ v[:, h // (H // G)] for h in range(H)], 1)


def attention(w, p, h, m, eps):
    L, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = rms(h @ w[p + "q"].t(), eps) * w[p + "q.norm"]
    kr = h @ w[p + "k"].t()
    k = rms(kr, eps) * w[p + "k.norm"]
    o = attention_core(q.view(L, H, D), k.view(L, G, D), kr.view(L, G, D), m["scale"], w[p + "talk"],
                       m["mask"]["size"]).reshape(L, H * D)
    o = o / (1 + torch.exp(-(h @ w[p + "g"].t())))
    return o @ w[p + "o"].t()


def relu2_mlp(w, p, h):
    return torch.clamp(h @ w[p + "up"].t(), min=0) ** 2 @ w[p + "down"].t()


MIXERS = {"hgrn2": hgrn2, "attention": attention}


def layer(w, spec, i, x, eps):
    p = f"l{i}."
    y = MIXERS[spec["type"]](w, p + "mix.", x, spec["mixer"], eps)
    x = x + scalar_norm(y, w[p + "norm1"], eps) * w[p + "ls1"]
    if spec.get("mlp") is not None:
        x = x + scalar_norm(relu2_mlp(w, p + "mlp.", x), w[p + "norm2"], eps) * w[p + "ls2"]
    return x


def embed(w, ids, dt):
    e = w["embed"][ids.long()]
    return e + sinusoid(ids.numel(), e.shape[1], dt)


def forward(cfg, tensors, ids, dt=torch.float64, residuals=None):
    """ids [L] -> logits [L, vocab]; ``residuals`` (a list) collects the stream after every layer."""
    w = {k: t.to(dt) for k, t in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = embed(w, ids, dt)
    for i, spec in enumerate(cfg["layers"]):
        x = layer(w, spec, i, x, eps)
        if residuals is not None:
            residuals.append(x)
    return scalar_norm(x, w["final.norm"], eps) @ w["head"].t()


def greedy(cfg, tensors, ids, n, dt=torch.float64):
    ids = ids.clone()
    out = []
    for _ in range(n):
        t = int(torch.argmax(forward(cfg, tensors, ids, dt)[-1]))
        out.append(t)
        ids = torch.cat([ids, torch.tensor([t])])
    return out
