"""Plain fp32 / fp64 implementation of the Nuvorax decoder, one function per mechanism.

Works on the checkpoint's own tensors (a dict name -> tensor) and the config dict, one sequence at a time.  Shares no
code with the framework: this is what the tests compare it to.
"""
import math

import torch


def rms(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def layer_norm(x, w, eps):
    """Centred, divided by the standard deviation, times a weight; no bias."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def sigmoid(x):
    return 1 / (1 + torch.exp(-x))


def gelu(x):
    return 0.5 * x * (1 + torch.erf(x / math.sqrt(2.0)))


def frequencies(dims, base, scaling=None):
    """Turns per position (in radians) of every pair; ``scaling``: long wavelengths slowed by ``factor``."""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling is not None:
            n, a, b, c = (float(scaling[k]) for k in ("original", "low", "high", "factor"))
            wave = 2 * math.pi / f
            if wave > n / a:
                f = f / c
            elif not wave < n / b:
                s = (n / wave - a) / (b - a)
                f = (1 - s) * f / c + s * f
        out.append(f)
    return out


def rotate(x, pos, freqs, sign=1.0):
    """x [L, heads, n]: entry i turns with entry i + len(freqs), by sign * pos * freqs[i]; later entries pass."""
    half = len(freqs)
    out = x.clone()
    for i, f in enumerate(freqs):
        a = pos.double() * (sign * f)
        c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def scores(q, k, scale, cap):
    """q [L, H, D], k [L, G, D] -> soft-capped scores [H, L, L]."""
    H, G = q.shape[1], k.shape[1]
    kk = k[:, [h // (H // G) for h in range(H)]]
    s = torch.einsum("ihd,jhd->hij", q, kk) * scale
    return cap * torch.tanh(s / cap)


def causal_weights(s):
    """exp(s) over (1 + the sum of exp(s)) of the keys j <= i."""
    L = s.shape[-1]
    i = torch.arange(L)
    s = s.masked_fill(i[None, :] > i[:, None], -math.inf)
    top = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def mix_heads(p, talk):
    return torch.einsum("hg,gij->hij", talk, p)


def attention(w, p, h, m, eps):
    L, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(L)
    q = rms((h @ w[p + "q"].t()).view(L, H, D), w[p + "q.norm"], eps)
    k = rms((h @ w[p + "k"].t()).view(L, G, D), w[p + "k.norm"], eps)
    v = (h @ w[p + "v"].t()).view(L, G, V)
    f = frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"]["scaling"])
    q, k = rotate(q, pos, f), rotate(k, pos, f)
    fv = frequencies(V, m["rot"]["base"])
    v = rotate(v, pos, fv)
    a = mix_heads(causal_weights(scores(q, k, m["scale"], m["softcap"])), w[p + "talk"])
    o = torch.einsum("hij,jhv->ihv", a, v[:, [x // (H // G) for x in range(H)]])
    o = rotate(o, pos, fv, -1.0)
    o = o * sigmoid(h @ w[p + "g"].t())[:, :, None]
    return o.reshape(L, H * V) @ w[p + "o"].t()


def clamped_glu(g, u, limit):
    g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1)


def expert(w, p, h, limit):
    return clamped_glu(h @ w[p + "gate"].t(), h @ w[p + "up"].t(), limit) @ w[p + "down"].t()


def route(z, r):
    """Router logits [L, E] -> dense weights [L, E] (0: not chosen)."""
    E, n = r["experts"], r["groups"]["count"]
    s = torch.softmax(z, -1)
    out = torch.zeros_like(s)
    for t in range(z.shape[0]):
        best = [float(s[t, g * (E // n):(g + 1) * (E // n)].max()) for g in range(n)]
        keep = sorted(range(n), key=lambda g: -best[g])[:r["groups"]["keep"]]
        allowed = [e for e in range(E) if e // (E // n) in keep]
        top = sorted(allowed, key=lambda e: -float(s[t, e]))[:r["top"]]
        total = sum(s[t, e] for e in top) + 1e-20
        for e in top:
            out[t, e] = s[t, e] / total * r["scale"]
    return out


def experts(w, p, h, m):
    a = route(h @ w[p + "router"].t(), m["router"])
    y = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        y = y + a[:, e:e + 1] * expert(w, p + f"e{e}.", h, m["expert"]["limit"])
    if m.get("shared") is not None:
        y = y + sigmoid(h @ w[p + "shared.sg"].t()) * expert(w, p + "shared.", h, m["shared"]["limit"])
    return y


def feed_forward(w, p, h, m):
    if m["kind"] == "dense":
        return gelu(h @ w[p + "up"].t()) @ w[p + "down"].t()
    return experts(w, p, h, m)


def layer(w, spec, i, x, eps):
    """Both sublayers read one norm of the stream."""
    h = layer_norm(x, w[f"l{i}.norm1"], eps)
    y = attention(w, f"l{i}.mix.", h, spec["mixer"], eps)
    if spec.get("mlp") is not None:
        y = y + feed_forward(w, f"l{i}.mlp.", h, spec["mlp"])
    return x + y


def forward(cfg, tensors, ids, dt=torch.float64, residuals=None):
    """ids [L] -> logits [L, vocab]; ``residuals`` (a list) collects the stream after every layer."""
    w = {k: t.to(dt) for k, t in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][ids.long()] * cfg["embedding"]["scale"]
    for i, spec in enumerate(cfg["layers"]):
        x = layer(w, spec, i, x, eps)
        if residuals is not None:
            residuals.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["head"].t() * cfg["logit_scale"]


def greedy(cfg, tensors, ids, n, dt=torch.float64):
    ids = ids.clone()
    out = []
    for _ in range(n):
        t = int(torch.argmax(forward(cfg, tensors, ids, dt)[-1]))
        out.append(t)
        ids = torch.cat([ids, torch.tensor([t])])
    return out
