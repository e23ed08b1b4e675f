"""Small random Nuvorax models for the tests: config dict + checkpoint tensors, written as a model folder; and attention and
expert inputs made directly for the ops."""
import torch

from tests import nuvorax_oracle as O
from tests.kafunex_utils import executor, ids, write  # noqa: F401  (the same helpers)

SCALING = {"factor": 6.0, "low": 1.0, "high": 4.0, "original": 64}  # (small: all three ranges of wavelengths occur)


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=24, limit=1.5, count=3, keep=2, scale=1.7, shared=(20, 0.9)):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale, "groups": {"count": count, "keep": keep}},
            "expert": {"ff": ff, "limit": limit},
            "shared": {"ff": shared[0], "limit": shared[1]} if shared else None}


def att(heads=4, kv_heads=2, dim=16, vdim=12, rot=12, base=1000.0, scaling=SCALING, scale=None, cap=8.0, mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "softcap": cap,
                      "scale": dim ** -0.5 if scale is None else scale, "rot": {"dims": rot, "base": base, "scaling": scaling}}}


def config(layers, vocab=160, width=64, eps=1e-5, embed=2.5, logit=0.6):
    return {"architecture": "Nuvorax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed},
            "logit_scale": logit, "layers": layers}


def layer_tensors(e, W, g):
    m, mlp = e["mixer"], e["mlp"]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]

    def mat(n, k, gain=1.0):
        return gain * torch.randn(n, k, generator=g) / k ** 0.5

    def near(n, c=1.0, s=0.3):
        return c + s * torch.randn(n, generator=g)

    t = {"norm1": near(W), "mix.q": mat(H * D, W), "mix.k": mat(G * D, W), "mix.v": mat(G * V, W),
         "mix.q.norm": near(D, 1.6), "mix.k.norm": near(D, 1.6),
         "mix.talk": torch.eye(H) + 0.4 * torch.randn(H, H, generator=g), "mix.g": mat(H, W, 2.0), "mix.o": mat(W, H * V)}
    glu = lambda p, ff: {p + "gate": mat(ff, W, 1.5), p + "up": mat(ff, W, 1.5), p + "down": mat(W, ff)}  # noqa: E731
    if mlp is not None and mlp["kind"] == "dense":
        t.update({"mlp.up": mat(mlp["ff"], W, 1.5), "mlp.down": mat(W, mlp["ff"])})
    elif mlp is not None:
        t["mlp.router"] = mat(mlp["router"]["experts"], W, 3.0)
        for x in range(mlp["router"]["experts"]):
            t.update(glu(f"mlp.e{x}.", mlp["expert"]["ff"]))
        if mlp.get("shared"):
            t.update(glu("mlp.shared.", mlp["shared"]["ff"]))
            t["mlp.shared.sg"] = mat(1, W, 2.0)
    return t


def tensors(cfg, seed=0, dtype=torch.bfloat16):
    """Checkpoint tensors rounded to ``dtype``."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    out = {"embed": torch.randn(cfg["vocab"], W, generator=g) / 2, "head": torch.randn(cfg["vocab"], W, generator=g) / W ** 0.5,
           "final.norm": 1 + 0.3 * torch.randn(W, generator=g)}
    for i, e in enumerate(cfg["layers"]):
        out.update({f"l{i}.{k}": v for k, v in layer_tensors(e, W, g).items()})
    return {k: v.to(dtype).contiguous() for k, v in out.items()}


# sizes that differ in every place; the values a model could make equal or 1; layers without a feed-forward, a shared expert
# or a scaling
MODELS = {
    "mixed": config([att(mlp=moe()), att(6, 3, 20, 8, 16, 300.0, scale=0.4, mlp=dense()),
                     att(5, 1, 12, 14, 4, 5e4, dict(SCALING, factor=2.0, original=20), cap=3.0,
                         mlp=moe(10, 3, 16, 0.7, 5, 3, 0.8, (28, 2.0)))], width=72, vocab=157),
    "ones": config([att(1, 1, 2, 2, 2, mlp=moe(1, 1, 1, 1.0, 1, 1, 1.0, (1, 1.0))), att(2, 2, 4, 4, 0, mlp=dense(1)),
                    att(3, 1, 6, 6, 6, scaling=None, mlp=moe(4, 4, 5, 1.0, 1, 1, 1.0, None))], width=32, vocab=64, eps=1e-3,
                   embed=1.0, logit=1.0),
    "bare": config([att(4, 4, 8, 16, 8, mlp=None), att(4, 1, 8, 8, 8, mlp=moe(8, 2, 16, 1.2, 8, 3, 2.5, None)),
                    att(2, 1, 24, 10, 24, mlp=dense(32))], width=48, vocab=96, eps=1e-2, embed=5.0),
}


class Attn:
    """Sequences of projected rows [q | k | v | gate] on a paged cache whose pages are not in order; the first ``starts``
    tokens of each were cached by an earlier step.  ``spike`` (query, key): the two share a direction."""

    def __init__(self, ntoks, starts, H, G, D, V, rot=None, dt=torch.float32, device="cpu", page=16, cap=20.0, scale=None,
                 spike=None, gain=1.5, base=500.0, scaling=SCALING, seed=0, pad=0):
        from src.ops import mixed, mixers

        self.ops = mixed
        g = torch.Generator().manual_seed(seed)
        rn = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
        self.H, self.G, self.D, self.V, self.dt, self.dev, self.page, self.cap = H, G, D, V, dt, device, page, cap
        self.ntoks, self.starts, self.eps, self.base, self.scaling = ntoks, starts, 1e-4, base, scaling
        self.rot = D - D % 2 if rot is None else rot
        self.scale = D ** -0.5 if scale is None else scale
        self.rep = H // G
        cols = H * D + G * (D + V) + H
        self.z = [rn(n + s, cols).to(dt) for n, s in zip(ntoks, starts)]
        if spike is not None:
            i, j = spike
            d = torch.sign(rn(D))
            z = self.z[0]
            z[j, H * D:(H + G) * D] = (3 * d).repeat(G).to(dt)
            z[i, :H * D] = (3 * d).repeat(H).to(dt)
        self.qg, self.kg = gain + 0.3 * rn(D), gain + 0.3 * rn(D)
        if spike is not None:
            self.qg, self.kg = torch.full((D,), gain), torch.full((D,), gain)
        self.talk = (torch.eye(H) + 0.5 * rn(H, H)).bfloat16().float()
        npg = [-(-z.shape[0] // page) for z in self.z]
        perm = torch.randperm(sum(npg) + 3, generator=g)[:sum(npg)]
        self.cache = torch.full((sum(npg) + 3, G, page, D + V), 55.0, dtype=dt, device=device)
        self.table = torch.full((len(ntoks) + 1, max(npg)), -1, dtype=torch.int32)
        self.slots, at = [], 0
        for i, z in enumerate(self.z):
            pages = perm[at:at + npg[i]]
            self.table[i + 1, :npg[i]] = pages.int()
            at += npg[i]
            p = torch.arange(z.shape[0])
            self.slots.append(pages[p // page] * page + p % page)
        self.table = self.table.to(device)
        mx = max(z.shape[0] for z in self.z)
        sc = None if scaling is None else tuple(scaling[k] for k in ("factor", "low", "high", "original"))
        self.rope = mixers.rope_table(base, self.rot, mx, device, sc)
        self.vrope = mixers.rope_table(base, V, mx, device)
        self.K = H * V + pad
        self.prep([slice(0, s) for s in starts])
        self.q = self.prep([slice(s, None) for s in starts])
        self.zr = torch.cat([z[s:] for z, s in zip(self.z, starts)]).to(device)
        self.q_seq = torch.cat([torch.full((n,), i + 1) for i, n in enumerate(ntoks)]).int().to(device)
        self.q_ctx = torch.cat([torch.arange(s + 1, s + n + 1) for n, s in zip(ntoks, starts)]).int().to(device)

    def prep(self, parts):
        z = torch.cat([z[s] for z, s in zip(self.z, parts)]).to(self.dev)
        if not z.shape[0]:
            return None
        slots = torch.cat([x[s] for x, s in zip(self.slots, parts)]).to(self.dev)
        ctx = torch.cat([torch.arange(1, x.shape[0] + 1)[s] for x, s in zip(self.slots, parts)]).int().to(self.dev)
        qn = torch.zeros(z.shape[0], self.H * self.D, dtype=self.dt, device=self.dev)
        out = torch.zeros(z.shape[0] * self.K, dtype=self.dt, device=self.dev)
        self.ops.mixed_prep(z, self.qg.to(self.dev), self.kg.to(self.dev), qn, self.cache, slots, ctx, self.rope, self.vrope,
                            out, self.K, self.eps)
        return qn

    def run(self, out=None, packed=False, **kw):
        T = self.zr.shape[0]
        out = torch.zeros(T * self.K, dtype=self.dt, device=self.dev) if out is None else out
        return self.ops.mixed_attention(self.zr, self.q, self.talk.to(self.dev), self.cache, self.table, self.q_seq,
                                        self.q_ctx, self.vrope, out, self.K, self.scale, self.cap, packed=packed, **kw)

    def want(self, no_sink=False, gates=True):
        H, G, D, V = self.H, self.G, self.D, self.V
        out = []
        for z, n in zip(self.z, self.ntoks):
            z, L = z.double(), z.shape[0]
            pos = torch.arange(L)
            f, fv = O.frequencies(self.rot, self.base, self.scaling), O.frequencies(V, self.base)
            q = O.rotate(O.rms(z[:, :H * D].reshape(L, H, D), self.qg.double(), self.eps), pos, f)
            k = O.rotate(O.rms(z[:, H * D:(H + G) * D].reshape(L, G, D), self.kg.double(), self.eps), pos, f)
            v = O.rotate(z[:, (H + G) * D:(H + G) * D + G * V].reshape(L, G, V), pos, fv)
            s = O.scores(q, k, self.scale, self.cap) if self.cap > 0 else \
                torch.einsum("ihd,jhd->hij", q, k.repeat_interleave(self.rep, 1)) * self.scale
            p = O.causal_weights(s)
            if no_sink:
                p = p / p.sum(-1, keepdim=True)
            a = O.mix_heads(p, self.talk.double())
            o = O.rotate(torch.einsum("hij,jhv->ihv", a, v.repeat_interleave(self.rep, 1)), pos, fv, -1.0)
            if gates:
                o = o * O.sigmoid(z[:, -H:])[:, :, None]
            out.append(o.reshape(L, H * V)[L - n:])
        return torch.cat(out)
