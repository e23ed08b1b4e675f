"""Small random Kafunex models for the tests: config dict + checkpoint tensors, written as a model folder."""
import json
import os

import torch


def rec(heads=2, dim=16, vdim=24, ff=48):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def att(heads=4, kv_heads=2, dim=16, size=20, scale=None, ff=48):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim,
                                           "scale": dim ** -0.5 if scale is None else scale, "mask": {"size": size}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, vocab=160, width=64, eps=1e-5):
    return {"architecture": "Kafunex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def tensors(cfg, seed=0, dtype=torch.bfloat16, gain=1.0):
    """Checkpoint tensors rounded to ``dtype``; ``gain`` sharpens the query / key norms (peaky attention)."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def mat(n, k):
        return torch.randn(n, k, generator=g) / k ** 0.5

    def near(n, c=1.0, s=0.3):
        return c + s * torch.randn(n, generator=g)

    out = {"embed": torch.randn(cfg["vocab"], W, generator=g), "head": mat(cfg["vocab"], W),
           "final.norm": near(1).reshape(())}
    for i, e in enumerate(cfg["layers"]):
        m, p = e["mixer"], f"l{i}."
        H, D = m["heads"], m["dim"]
        t = {"norm1": near(1).reshape(()), "ls1": near(W, 0.7, 0.2)}
        if e["type"] == "hgrn2":
            V = m["vdim"]
            t.update({"mix.q": mat(H * D, W), "mix.f": mat(H * D, W), "mix.f.b": near(H * D, 2.0, 1.5),
                      "mix.lower": torch.rand(H * D, generator=g) * 0.9, "mix.v": mat(H * V, W), "mix.norm": near(V),
                      "mix.o": mat(W, H * V)})
            t["mix.lower"][:: 5] = 0.0
        else:
            G = m["kv_heads"]
            t.update({"mix.q": mat(H * D, W), "mix.k": mat(G * D, W), "mix.q.norm": near(H * D) * gain,
                      "mix.k.norm": near(G * D) * gain, "mix.talk": torch.eye(H) + 0.4 * torch.randn(H, H, generator=g),
                      "mix.g": mat(H * D, W), "mix.o": mat(W, H * D)})
        if e["mlp"] is not None:
            ff = e["mlp"]["ff"]
            t.update({"mlp.up": mat(ff, W), "mlp.down": mat(W, ff), "norm2": near(1).reshape(()),
                      "ls2": near(W, 0.7, 0.2)})
        out.update({p + k: v for k, v in t.items()})
    return {k: v.to(dtype).contiguous() for k, v in out.items()}


def write(folder, cfg, w):
    from safetensors.torch import save_file

    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(w, os.path.join(folder, "model.safetensors"))
    return str(folder)


def executor(folder, device, dtype, **kw):
    from src.llama_partition import load_stage_model
    from src.runtime.executor import StageExecutor

    full = load_stage_model(folder, device, kw.pop("role", "full"), dtype=dtype, start=kw.pop("start", 0),
                            end=kw.pop("end", None))
    kw.setdefault("max_sessions", 6)
    kw.setdefault("max_seq_len", 512)
    kw.setdefault("kv_cache_bytes", 32 << 20)
    return StageExecutor(full.cfg, full.weights, device, dtype=full.dtype, warmup=False, **kw)


def ids(n, vocab, seed=1):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed))


# sizes that differ in every place, one of them with the values a model could make equal or 1
MODELS = {
    "mixed": config([rec(), att(), rec(3, 12, 8, 40), att(6, 3, 8, 9, 0.4, 32), rec(1, 20, 33)], width=72, vocab=157),
    "ones": config([att(1, 1, 8, 1, 1.0), rec(1, 1, 1), att(2, 1, 8, 7), att(3, 3, 16, 33)], width=32, vocab=64,
                   eps=1e-3),
    "no_mlp": config([att(4, 4, 8, 5, 0.2, 0), rec(2, 8, 8, 0), rec(2, 8, 16, 24)], width=48, vocab=96, eps=1e-2),
}
