"""Small random Fubapel models for the tests: config dict + checkpoint tensors, written as a model folder."""
import torch

from tests.kafunex_utils import executor, ids, write  # noqa: F401  (the same helpers)


def glu(ff, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit} if ff else None


def mla(heads=3, dim=8, vdim=12, rot=4, q_rank=20, kv_rank=24, scale=None, base=10000.0, ff=40, limit=1.5):
    return {"type": "latent_attention", "mlp": glu(ff, limit),
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                      "scale": (dim + rot) ** -0.5 if scale is None else scale, "rot": {"dims": rot, "base": base}}}


def mem(heads=2, dim=16, vdim=24, cap=9.0, ff=0, limit=1.5):
    return {"type": "mlstm", "mlp": glu(ff, limit), "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def ret(heads=2, dim=16, vdim=24, rot=None, base=5000.0, decay=None, ff=0, limit=1.5):
    if decay is None:
        decay = [1 - 2.0 ** (-3 - 2 * h) for h in range(heads)]
    return {"type": "retention", "mlp": glu(ff, limit),
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay,
                      "rot": {"dims": dim if rot is None else rot, "base": base}}}


def config(layers, vocab=160, width=64, eps=1e-5, mult=0.6, loop=None):
    return {"architecture": "Fubapel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
            "loop": loop, "layers": layers}


def layer_tensors(e, W, g):
    m = e["mixer"]
    H, D, V = m["heads"], m["dim"], m["vdim"]

    def mat(n, k, gain=1.0):
        return gain * torch.randn(n, k, generator=g) / k ** 0.5

    def near(n, c=1.0, s=0.3):
        return c + s * torch.randn(n, generator=g)

    t = {"norm1": near(W), "mix.o": mat(W, H * V)}
    if e["type"] == "latent_attention":
        R, Q, C = m["rot_dim"], m["q_rank"], m["kv_rank"]
        t.update({"mix.dq": mat(Q, W), "mix.dq.norm": near(Q), "mix.uq": mat(H * (D + R), Q, 2.0),
                  "mix.dkv": mat(C + R, W), "mix.dkv.norm": near(C), "mix.uk": mat(H * D, C, 2.0),
                  "mix.uv": mat(H * V, C), "mix.sink": near(H, 0.5, 1.5)})
    else:
        t.update({"mix.q": mat(H * D, W), "mix.k": mat(H * D, W), "mix.v": mat(H * V, W), "mix.g": mat(H * V, W)})
    if e["type"] == "mlstm":
        t.update({"mix.norm": near(H * V), "mix.i": mat(H, W), "mix.i.b": near(H, -1.0, 2.0), "mix.f": mat(H, W),
                  "mix.f.b": near(H, 3.0, 1.5)})
    if e["mlp"] is not None:
        ff = e["mlp"]["ff"]
        t.update({"mlp.gate": mat(ff, W, 1.5), "mlp.up": mat(ff, W, 1.5), "mlp.down": mat(W, ff), "norm2": near(W)})
    return t


def tensors(cfg, seed=0, dtype=torch.bfloat16):
    """Checkpoint tensors rounded to ``dtype``."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    out = {"embed": torch.randn(cfg["vocab"], W, generator=g), "head": torch.randn(cfg["vocab"], W, generator=g) / W ** 0.5,
           "final.norm": 1 + 0.3 * torch.randn(W, generator=g)}
    for i, e in enumerate(cfg["layers"]):
        out.update({f"l{i}.{k}": v for k, v in layer_tensors(e, W, g).items()})
    return {k: v.to(dtype).contiguous() for k, v in out.items()}


# sizes that differ in every place, with and without a loop; one with the values a model could make equal or 1
MODELS = {
    "mixed": config([ret(), mla(), mem(3, 12, 8), mla(5, 16, 8, 8, 36, 40, 0.21, 700.0, 24, 0.8), ret(3, 20, 8, 12)],
                    width=72, vocab=157, loop={"start": 1, "stop": 4, "times": 2}),
    "ones": config([mla(1, 1, 1, 2, 1, 1, 1.0, ff=1), mem(1, 1, 1), ret(1, 2, 1, decay=[0.0]), mla(2, 2, 3, 2, 3, 4),
                    ret(2, 4, 4, 0, decay=[1.0, 0.5])], width=32, vocab=64, eps=1e-3, mult=1.0,
                   loop={"start": 0, "stop": 2, "times": 3}),
    "ffs": config([mem(2, 8, 8, 4.0, ff=48), ret(2, 8, 16, ff=32, limit=0.7), mla(4, 12, 8, 6, ff=0)], width=48,
                  vocab=96, eps=1e-2, mult=0.3),
}
