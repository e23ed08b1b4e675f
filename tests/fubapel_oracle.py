"""Plain fp32 / fp64 implementation of the Fubapel decoder, one function per mechanism.

Works on the checkpoint's own tensors (a dict name -> tensor) and the config dict, one sequence at a time, token
by token where the mechanism is recurrent.  Shares no code with the framework: this is what the tests compare it to.
"""
import math

import torch


def rms(x, eps):
    """x over its root mean square (last axis), eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, eps):
    """Centred, divided by the standard deviation, times a weight; no bias."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def sigmoid(x):
    return 1 / (1 + torch.exp(-x))


def rotate(x, pos, dims, base):
    """x [L, heads, n]: the first ``dims`` entries of each head turn, entry i with entry i + dims / 2."""
    half = dims // 2
    out = x.clone()
    for i in range(half):
        a = pos.double() * float(base) ** (-2.0 * i / dims)
        c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def sink_softmax(s, sink):
    """s [H, L, n] scores (-inf: not seen), sink [H]: weights whose denominator also holds exp(sink)."""
    top = torch.maximum(s.max(-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink[:, None, None] - top))


def latent_core(qn, qr, kn, kr, v, sink, scale):
    """qn, kn [L, H, D], qr [L, H, R], kr [L, R] (one for all heads), v [L, H, V] -> [L, H, V], causal."""
    L = qn.shape[0]
    s = (torch.einsum("ihd,jhd->hij", qn, kn) + torch.einsum("ihr,jr->hij", qr, kr)) * scale
    i = torch.arange(L)
    s = s.masked_fill(i[None, None, :] > i[None, :, None], -math.inf)
    return torch.einsum("hij,jhv->ihv", sink_softmax(s, sink), v)


def latent_attention(w, p, h, m, eps):
    L, H, D, R, V, C = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(L)
    cq = rms(h @ w[p + "dq"].t(), eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].t()).view(L, H, D + R)
    ckr = h @ w[p + "dkv"].t()
    c = rms(ckr[:, :C], eps) * w[p + "dkv.norm"]
    turn = lambda x: rotate(x, pos, m["rot"]["dims"], m["rot"]["base"])  # noqa: E731
    qr, kr = turn(q[..., D:]), turn(ckr[:, None, C:])[:, 0]
    kn, v = (c @ w[p + "uk"].t()).view(L, H, D), (c @ w[p + "uv"].t()).view(L, H, V)
    o = latent_core(q[..., :D], qr, kn, kr, v, w[p + "sink"], m["scale"])
    return o.reshape(L, H * V) @ w[p + "o"].t()


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def log_sigmoid(x):
    return torch.minimum(x, torch.zeros_like(x)) - torch.log1p(torch.exp(-x.abs()))


def mlstm_scan(q, k, v, i, f, state=None):
    """q, k [L, H, D], v [L, H, V], log gates i, f [L, H] -> o [L, H, V], (S, n, m): one token after the other."""
    L, H, D = q.shape
    if state is None:
        S, n, m = torch.zeros(H, D, v.shape[-1], dtype=q.dtype), torch.zeros(H, D, dtype=q.dtype), \
            torch.zeros(H, dtype=q.dtype)
    else:
        S, n, m = (t.clone() for t in state)
    o = torch.zeros(L, H, v.shape[-1], dtype=q.dtype)
    for t in range(L):
        m1 = torch.maximum(f[t] + m, i[t])
        a, b = torch.exp(f[t] + m - m1), torch.exp(i[t] - m1)
        S = a[:, None, None] * S + b[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = a[:, None] * n + b[:, None] * k[t]
        m = m1
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        o[t] = (q[t][:, :, None] * S).sum(1) / den[:, None]
    return o, (S, n, m)


def mlstm(w, p, h, m, eps):
    L, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].t() * D ** -0.5).view(L, H, D)
    k = (h @ w[p + "k"].t()).view(L, H, D)
    v = (h @ w[p + "v"].t()).view(L, H, V)
    i = soft_cap(h @ w[p + "i"].t() + w[p + "i.b"], m["gate_cap"])
    f = log_sigmoid(soft_cap(h @ w[p + "f"].t() + w[p + "f.b"], m["gate_cap"]))
    o, _ = mlstm_scan(q, k, v, i, f)
    y = rms(o, eps).reshape(L, H * V) * w[p + "norm"] * sigmoid(h @ w[p + "g"].t())
    return y @ w[p + "o"].t()


def retention_scan(q, k, v, decay, state=None):
    """q, k [L, H, D], v [L, H, V], decay [H] -> o [L, H, V], final state [H, D, V]."""
    L, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    o = torch.zeros(L, H, v.shape[-1], dtype=q.dtype)
    for t in range(L):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (q[t][:, :, None] * S).sum(1)
    return o, S


def retention(w, p, h, m, eps):
    L, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    pos = torch.arange(L)
    turn = lambda x: rotate(x.view(L, H, D), pos, m["rot"]["dims"], m["rot"]["base"])  # noqa: E731
    q, k = turn(h @ w[p + "q"].t()), turn(h @ w[p + "k"].t()) * D ** -0.5
    v = (h @ w[p + "v"].t()).view(L, H, V)
    o, _ = retention_scan(q, k, v, torch.tensor(m["decay"], dtype=h.dtype))
    g = h @ w[p + "g"].t()
    return (rms(o, eps).reshape(L, H * V) * g * sigmoid(g)) @ w[p + "o"].t()


def clamped_glu(g, u, limit):
    """g below the limit, u inside +-limit: g sigmoid(1.702 g) (u + 1)."""
    g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1)


def mlp(w, p, h, m):
    return clamped_glu(h @ w[p + "gate"].t(), h @ w[p + "up"].t(), m["limit"]) @ w[p + "down"].t()


MIXERS = {"latent_attention": latent_attention, "mlstm": mlstm, "retention": retention}


def layer(w, spec, i, x, eps, mult):
    p = f"l{i}."
    x = x + mult * MIXERS[spec["type"]](w, p + "mix.", layer_norm(x, w[p + "norm1"], eps), spec["mixer"], eps)
    if spec.get("mlp") is not None:
        x = x + mult * mlp(w, p + "mlp.", layer_norm(x, w[p + "norm2"], eps), spec["mlp"])
    return x


def layer_runs(cfg):
    """Layer numbers in the order in which they run: start .. stop - 1 as often as the loop says."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if lp is None:
        return list(range(n))
    a, b = lp["start"], lp["stop"]
    return list(range(a)) + list(range(a, b)) * lp["times"] + list(range(b, n))


def forward(cfg, tensors, ids, dt=torch.float64, residuals=None):
    """ids [L] -> logits [L, vocab]; ``residuals`` (a list) collects the stream after every layer run."""
    w = {k: t.to(dt) for k, t in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][ids.long()]
    for i in layer_runs(cfg):
        x = layer(w, cfg["layers"][i], i, x, eps, cfg["residual_mult"])
        if residuals is not None:
            residuals.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["head"].t()


def greedy(cfg, tensors, ids, n, dt=torch.float64):
    ids = ids.clone()
    out = []
    for _ in range(n):
        t = int(torch.argmax(forward(cfg, tensors, ids, dt)[-1]))
        out.append(t)
        ids = torch.cat([ids, torch.tensor([t])])
    return out
