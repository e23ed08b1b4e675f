"""Nuvorax on the CPU data path: configuration, loading, every mechanism alone, the executor, the scheduler and the command
line, against the plain oracle (tests/nuvorax_oracle.py)."""
import dataclasses
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from src.models.config import LayerSpec, MoESpec, hybrid_config, resolve_model
from src.ops import mixed as xops
from src.ops import mixers as mops
from src.ops import moe as eops
from tests import nuvorax_oracle as O
from tests import nuvorax_utils as U
from tests.test_kafunex import serve

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = dict(atol=2e-4, rtol=2e-4)


@pytest.fixture(scope="module", params=sorted(U.MODELS))
def model(request, tmp_path_factory):
    cfg = U.MODELS[request.param]
    w = U.tensors(cfg, seed=3)
    return cfg, w, U.write(tmp_path_factory.mktemp(request.param), cfg, w)


def ref(cfg, w, ids):
    return O.forward(cfg, w, ids).float()


# ------------------------------------------------------------------ configuration and weights
@pytest.mark.parametrize("name", sorted(U.MODELS))
def test_registry_reads_every_size(tmp_path, name):
    cfg = U.MODELS[name]
    c = resolve_model(U.write(tmp_path, cfg, U.tensors(cfg)))
    assert (c.model_type, c.hybrid, c.num_hidden_layers) == ("nuvorax", True, len(cfg["layers"]))
    assert (c.vocab_size, c.hidden_size, c.rms_norm_eps) == (cfg["vocab"], cfg["width"], cfg["norm"]["eps"])
    assert (c.embed_scale, c.logit_scale) == (cfg["embedding"]["scale"], cfg["logit_scale"])
    assert (c.stream, c.norm, c.embed_positions, c.residual_mult) == ("pre", "layer", False, 1.0)
    for sp, e in zip(c.layers, cfg["layers"]):
        m, mlp = e["mixer"], e["mlp"]
        assert (sp.heads, sp.kv_heads, sp.dim, sp.vdim) == (m["heads"], m["kv_heads"], m["dim"], m["vdim"])
        assert (sp.scale, sp.softcap, sp.rot_dims, sp.rot_base) == (m["scale"], m["softcap"], m["rot"]["dims"], m["rot"]["base"])
        sc = m["rot"]["scaling"]
        assert sp.rot_scaling == (None if sc is None else (sc["factor"], sc["low"], sc["high"], sc["original"]))
        assert sp.parallel and (sp.moe is not None) == (mlp is not None and mlp["kind"] == "moe")
        if sp.moe:
            r = mlp["router"]
            assert sp.moe == MoESpec(r["experts"], r["top"], mlp["expert"]["ff"], mlp["expert"]["limit"],
                                     r["groups"]["count"], r["groups"]["keep"], r["scale"])
            assert (sp.ff, sp.limit) == ((mlp["shared"]["ff"], mlp["shared"]["limit"]) if mlp["shared"] else (0, 0.0))
        else:
            assert sp.ff == (mlp["ff"] if mlp else 0)
    assert type(c).from_hf_dict(json.loads(json.dumps(cfg))).layers == c.layers
    n = sum(t.numel() for k, t in U.tensors(cfg).items() if k.startswith("l"))
    assert abs(sum(sp.param_count(c.hidden_size) for sp in c.layers) - n) < 0.1 * n + 1200  # (padding rows, spare norms)
    assert c.kv_bytes_per_token_per_layer() > 0 and c.layer_param_bytes() > 0


@pytest.mark.parametrize("change,match", [
    (lambda c: c["layers"][0].update(type="other"), "unsupported mixer"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "multiple of kv_heads"),
    (lambda c: c["layers"][0]["mixer"].update(vdim=7), "even vdim"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "at most"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(scaling=dict(U.SCALING, high=1.0)), "scaling"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "top"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4), "equal groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "equal groups"),
    (lambda c: c["layers"][0]["mlp"]["expert"].update(limit=0.0), "experts"),
    (lambda c: c["layers"][1]["mlp"].update(kind="other"), "feed-forward kind")])
def test_bad_configurations_are_refused(tmp_path, change, match):
    cfg = json.loads(json.dumps(U.MODELS["mixed"]))
    change(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(ValueError, match=match):
        resolve_model(str(tmp_path))


@pytest.mark.parametrize("name", ["l0.mix.talk", "l2.mlp.e7.down", "l0.mlp.shared.sg", "l1.mlp.up"])
def test_wrong_tensor_shape_is_refused(tmp_path, name):
    cfg = U.MODELS["mixed"]
    w = U.tensors(cfg)
    w[name] = torch.cat([w[name], w[name][:, :1]], 1).contiguous()
    with pytest.raises(ValueError, match=name[3:]):
        U.executor(U.write(tmp_path, cfg, w), "cpu", "fp32")


def test_preset_runs_with_random_weights():
    ex = U.executor("tiny-nuvorax", "cpu", "fp32")
    assert torch.isfinite(ex.forward([("a", 50)], U.ids(50, 640))).all()
    c = resolve_model("nuvorax-7b")
    c.validate()
    assert 5e9 < sum(sp.param_count(c.hidden_size) for sp in c.layers) < 9e9


# ------------------------------------------------------------------ mechanisms
@pytest.mark.parametrize("dims,base,scaling", [(16, 1000.0, U.SCALING), (2, 1e6, None), (10, 10.0, U.SCALING),
                                               (12, 300.0, dict(factor=3.0, low=2.0, high=2.5, original=100))])
def test_rotation_and_frequency_scaling(dims, base, scaling):
    from src.ops.reference_mixers import turn

    x, pos = torch.randn(7, 3, 18), torch.tensor([0, 1, 2, 50, 999, 1000, 3])
    sc = None if scaling is None else tuple(scaling[k] for k in ("factor", "low", "high", "original"))
    f = O.frequencies(dims, base, scaling)
    got = turn(x, mops.rope_table(base, dims, 1001, "cpu", sc)[pos][:, None])
    torch.testing.assert_close(got, O.rotate(x.double(), pos, f).float(), **TOL)
    torch.testing.assert_close(O.rotate(O.rotate(x.double(), pos, f), pos, f, -1.0).float(), x, **TOL)
    assert torch.equal(got[..., dims:], x[..., dims:])
    if dims == 16:  # kept, divided and blended frequencies all occur
        r = torch.tensor(f) / torch.tensor(O.frequencies(dims, base))
        assert (r == 1).any() and (r - 1 / scaling["factor"]).abs().min() < 1e-12 and ((r < 0.99) & (r > 0.2)).any()


@pytest.mark.parametrize("H,G,D,V,rot,page", [(4, 2, 16, 12, 12, 16), (1, 1, 1, 2, 0, 8), (6, 3, 10, 6, 4, 64),
                                             (5, 1, 8, 8, 8, 32), (3, 3, 5, 4, 4, 64)])
@pytest.mark.parametrize("cap", [20.0, 1.5, 0.0])
def test_attention_alone(H, G, D, V, rot, page, cap):
    a = U.Attn([33, 1, 2, 17], [0, 30, 15, 63], H, G, D, V, rot, page=page, cap=cap)
    want = a.want()
    got = a.run().view(-1, H * V)
    torch.testing.assert_close(got, want.float(), **TOL)
    assert (a.want(no_sink=True)[:4] - want[:4]).abs().max() > 0.02  # the first tokens show a sink that is left out
    assert (a.want(gates=False) - want).abs().max() > 0.02
    if H > 1:
        b = U.Attn([33, 1, 2, 17], [0, 30, 15, 63], H, G, D, V, rot, page=page, cap=cap)
        b.talk = b.talk.t().contiguous()
        assert (b.want() - want).abs().max() > 0.02  # which way the mixing goes


@pytest.mark.parametrize("i,j", [(39, 0), (39, 7), (39, 8), (16, 15), (16, 16), (8, 7), (31, 24), (32, 31), (32, 32)])
def test_a_far_key_stands_out(i, j):
    res = []
    for sign in (1, -1):
        a = U.Attn([40], [0], 4, 2, 16, 12, 4, page=8, spike=(i, j), gain=2.0)
        at = slice((a.H + a.G) * a.D, (a.H + a.G) * a.D + a.G * a.V)
        a.z[0][j, at] *= sign
        a.prep([slice(0, None)])
        got = a.run().view(40, -1)[i]
        torch.testing.assert_close(got, a.want()[i].float(), **TOL)
        res.append(got)
    assert (res[0] - res[1]).abs().max() > 0.3


def test_values_are_rotated_by_their_own_place():
    """One key takes all the weight: its value comes out turned by the distance, at any vdim pair."""
    a = U.Attn([40], [0], 2, 1, 16, 6, 4, spike=(39, 3), gain=3.0, cap=0.0)
    a.talk = torch.eye(2)
    v = a.z[0][3, 3 * 16:3 * 16 + 6].double()
    d = O.rotate(v[None, None], torch.tensor([3 - 39]), O.frequencies(6, 500.0))[0, 0]
    got = (a.run().view(40, 2, 6)[39].double() / O.sigmoid(a.z[0][39, -2:].double())[:, None])
    torch.testing.assert_close(got, d.expand(2, 6), atol=2e-3, rtol=2e-3)
    assert (d - v).abs().max() > 0.1


@pytest.mark.parametrize("kind,F,block", [("gelu", 24, 1), ("clamped_glu", 24, 8), ("gated_glu", 20, 20)])
def test_feed_forward_activations(kind, F, block):
    z = 3 * torch.randn(9, 2 * F + 8)
    got = xops.ffn_act(z, torch.empty(9, F), kind, F, block, 1.25)
    if kind == "gelu":
        want = O.gelu(z[:, :F].double())
    else:
        v = z[:, :2 * F].double().view(9, F // block, 2, block)
        want = O.clamped_glu(v[:, :, 0].reshape(9, F), v[:, :, 1].reshape(9, F), 1.25)
        if kind == "gated_glu":
            want = want * O.sigmoid(z[:, 2 * F:2 * F + 1].double())
    torch.testing.assert_close(got, want.float(), **TOL)


def scratch():
    bufs = {}

    def e(name, shape, dtype=torch.float32):
        return bufs.setdefault(name, torch.empty(shape, dtype=dtype))
    return e


ROUTERS = [(6, 2, 3, 2), (8, 1, 1, 1), (8, 8, 1, 1), (12, 3, 12, 5), (5, 2, 5, 2), (1, 1, 1, 1), (16, 4, 2, 1)]


@pytest.mark.parametrize("E,top,count,keep", ROUTERS)
def test_choice_of_experts(E, top, count, keep):
    x, w = torch.randn(40, 24), torch.randn(E, 24)
    ctx = torch.ones(40, dtype=torch.int32)
    ctx[[3, 17]] = 0  # padding rows
    c = eops.choose(x, w, ctx, MoESpec(E, top, 8, 1.0, count, keep, 1.9), scratch())
    r = {"experts": E, "top": top, "scale": 1.9, "groups": {"count": count, "keep": keep}}
    want = O.route(x.double() @ w.double().t(), r)
    got, at = torch.zeros(40, E), 0
    for e, n in enumerate(c.lists.tolist()):
        for row in range(at, at + n):
            t = int(c.tok[row])
            got[t, e] = c.weights[t][c.slot[t] == row]
        at += n
    want[[3, 17]] = 0
    torch.testing.assert_close(got, want.float(), **TOL)
    assert (c.slot[[3, 17]] == -1).all() and at == 38 * top
    if keep < count and count < E:  # the group limit matters somewhere
        free = O.route(x.double() @ w.double().t(), dict(r, groups={"count": 1, "keep": 1}))
        assert ((free > 0) != (want > 0)).any()


def test_experts_and_their_sum():
    cfg = U.config([U.att(mlp=U.moe(shared=None))])
    w = {k[len("l0.mlp."):]: t.float() for k, t in U.tensors(cfg).items() if k.startswith("l0.mlp.")}
    m = cfg["layers"][0]["mlp"]
    x, res = torch.randn(21, 64), torch.randn(21, 64)
    up = torch.stack([torch.cat([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(6)])
    down = torch.stack([w[f"e{e}.down"] for e in range(6)])
    e = scratch()
    c = eops.choose(x, w["router"], torch.ones(21, dtype=torch.int32), MoESpec(6, 2, 24, 1.5, 3, 2, 1.7), e)
    y = eops.experts(x, c, up, down, None, None, 24, e)
    want = res.double() + O.experts({k: t.double() for k, t in w.items()}, "", x.double(), m)
    mops.add_norm(None, res, 1.0, None, 1e-5, None, experts=(y, c.slot, c.weights))
    torch.testing.assert_close(res, want.float(), **TOL)


# ------------------------------------------------------------------ executor
def test_whole_prompts(model):
    cfg, w, d = model
    ex = U.executor(d, "cpu", "fp32")
    for n in (1, 2, 3, 64, 65, 130):
        t = U.ids(n, cfg["vocab"], n)
        got = ex.forward([("a", n)], t, reset=[True], logit_rows=range(n))
        torch.testing.assert_close(got, ref(cfg, w, t), **TOL)


def test_prefill_equals_decoding_and_portions(model):
    cfg, w, d = model
    n = 90
    t = U.ids(n, cfg["vocab"])
    want = ref(cfg, w, t)
    ex = U.executor(d, "cpu", "fp32")
    for name, sizes in (("decode", [1] * n), ("pairs", [2] * (n // 2)), ("odd", [2, 3, 5, 7, 11, 13, 17, 19, 2, 11]),
                        ("head", [67, 1, 1, 2, 19])):
        assert sum(sizes) == n
        at, got = 0, []
        for k in sizes:
            got.append(ex.forward([(name, k)], t[at:at + k], logit_rows=range(k)))
            at += k
        torch.testing.assert_close(torch.cat(got), want, **TOL)
        ex.sessions.close(name)


def test_unequal_batches_equal_each_alone(model):
    cfg, w, d = model
    ex = U.executor(d, "cpu", "fp32")
    lens = {"a": 70, "b": 3, "c": 41, "d": 1}
    toks = {k: U.ids(n + 12, cfg["vocab"], n) for k, n in lens.items()}
    at = {k: 0 for k in lens}
    steps = [{"a": 30, "b": 2}, {"a": 1, "c": 20, "b": 1}, {"d": 1, "c": 21, "a": 39}, {"a": 1, "b": 1, "c": 1, "d": 1},
             {"d": 1, "b": 1}, {"c": 2, "a": 1}, {"b": 1, "d": 5}]
    for s in steps:
        x = torch.cat([toks[k][at[k]:at[k] + n] for k, n in s.items()])
        got = ex.forward(list(s.items()), x)
        for r, (k, n) in enumerate(s.items()):
            at[k] += n
            torch.testing.assert_close(got[r], ref(cfg, w, toks[k][:at[k]])[-1], **TOL)


def test_pages_are_used_again(model):
    cfg, w, d = model
    ex = U.executor(d, "cpu", "fp32", max_sessions=2, num_pages=3, page_size=64)
    for k in range(5):
        t, u = U.ids(100 + k, cfg["vocab"], k), U.ids(30, cfg["vocab"], 50 + k)
        torch.testing.assert_close(ex.forward([(f"s{k}", t.numel())], t)[0], ref(cfg, w, t)[-1], **TOL)
        torch.testing.assert_close(ex.forward([(f"u{k}", 30)], u)[0], ref(cfg, w, u)[-1], **TOL)
        with pytest.raises(Exception):
            ex.forward([(f"x{k}", 1)], t[:1])  # no third session
        ex.sessions.close(f"s{k}")
        ex.sessions.close(f"u{k}")
        for s in ex.cache.rows:  # whatever is left there must not be read
            s.fill_(1e6)
    assert ex.sessions.free_pages == 3


def test_long_decoding(model):
    cfg, w, d = model
    n = 200
    t = U.ids(n, cfg["vocab"], 9)
    ex = U.executor(d, "cpu", "fp32")
    ex.forward([("a", 10)], t[:10])
    got = torch.cat([ex.forward([("a", 1)], t[i:i + 1]) for i in range(10, n)])
    torch.testing.assert_close(got, ref(cfg, w, t)[10:], **TOL)


def test_chunked_prefill_of_a_long_step(model):
    cfg, w, d = model
    t = U.ids(150, cfg["vocab"], 4)
    ex = U.executor(d, "cpu", "fp32", max_tokens_per_step=37)
    got = ex.forward([("a", 120), ("b", 30)], t)
    torch.testing.assert_close(got[0], ref(cfg, w, t[:120])[-1], **TOL)
    torch.testing.assert_close(got[1], ref(cfg, w, t[120:])[-1], **TOL)


def test_stage_split_equals_full(model):
    cfg, w, d = model
    s0 = U.executor(d, "cpu", "bf16", role="stage0", end=1)
    s1 = U.executor(d, "cpu", "bf16", role="segment", start=1, end=2)
    s2 = U.executor(d, "cpu", "bf16", role="last", start=2, end=len(cfg["layers"]))
    full = U.executor(d, "cpu", "bf16")
    t = U.ids(40, cfg["vocab"])
    h = s0.forward([("a", 40)], t)
    assert h.dtype == torch.float32 == s0.hidden_dtype  # the stream between stages stays 32-bit
    torch.testing.assert_close(s2.forward([("a", 40)], s1.forward([("a", 40)], h)), full.forward([("a", 40)], t))


def test_fork_and_rewind(model):
    cfg, w, d = model
    ex = U.executor(d, "cpu", "fp32")
    t = U.ids(30, cfg["vocab"])
    ex.forward([("a", 25)], t[:25])
    ex.sessions.fork("a", "b")
    ex.forward([("a", 3)], t[:3])
    torch.testing.assert_close(ex.forward([("b", 5)], t[25:])[0], ref(cfg, w, t)[-1], **TOL)
    got = ex.forward([("b", 20)], t[10:], starts=[10])
    torch.testing.assert_close(got[0], ref(cfg, w, t)[-1], **TOL)


def test_bf16_path_is_close(model):
    cfg, w, d = model
    t = U.ids(120, cfg["vocab"], 2)
    want = ref(cfg, w, t)
    got = U.executor(d, "cpu", "bf16").forward([("a", 120)], t, logit_rows=range(120)).float()
    err = (got - want).pow(2).mean(-1).sqrt() / want.std()
    assert err.quantile(0.9) < 0.1  # (a close call of a router goes either way)


def sequential(parallel=False):
    """The same mechanisms in layers whose feed-forward reads a norm of its own."""
    kw = dict(kv_heads=2, scale=0.3, softcap=9.0, rot_dims=8, rot_base=200.0)
    return hybrid_config("nuvorax", 90, 48, 1e-5, [
        LayerSpec("mixed_attention", 4, 8, 6, 32, ffn="gelu", **kw),
        LayerSpec("mixed_attention", 4, 8, 6, 20, ffn="clamped_glu", limit=1.1, moe=MoESpec(6, 2, 16, 1.3, 2, 1, 1.4), **kw),
        LayerSpec("mixed_attention", 4, 8, 6, ffn="clamped_glu", moe=MoESpec(4, 2, 12, 1.3), **kw)], "seq", stream="pre",
        norm="layer", residual_mult=0.7, embed_positions=False)


def sequential_oracle(c, w, ids):
    from src.models.weights import random_hybrid_tensors

    x = w.embed.double()[ids]
    for i, sp in enumerate(c.layers):
        t = {k: v.double() for k, v in random_hybrid_tensors(c, i, dtype=torch.float32).items()}
        m = {"heads": 4, "kv_heads": 2, "dim": 8, "vdim": 6, "scale": 0.3, "softcap": 9.0,
             "rot": {"dims": 8, "base": 200.0, "scaling": None}}
        x = x + 0.7 * O.attention(t, "mix.", O.layer_norm(x, t["norm1"], 1e-5), m, 1e-5)
        h = O.layer_norm(x, t["norm2"], 1e-5)
        if sp.moe:
            r = {"experts": sp.moe.experts, "top": sp.moe.top, "scale": sp.moe.scale,
                 "groups": {"count": sp.moe.groups, "keep": sp.moe.keep}}
            y = O.experts(t, "mlp.", h, {"router": r, "expert": {"limit": sp.moe.limit},
                                         "shared": {"limit": sp.limit} if sp.ff else None})
        else:
            y = O.gelu(h @ t["mlp.up"].t()) @ t["mlp.down"].t()
        x = x + 0.7 * y
    return (O.layer_norm(x, w.final_norm.double(), 1e-5) @ w.lm_head[:90].double().t()).float()


@pytest.mark.parametrize("device", ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)])
def test_sequential_layers_take_the_same_mechanisms(device):
    from src.models.weights import random_stage_weights
    from src.runtime.executor import StageExecutor

    c = sequential()
    cpu = random_stage_weights(c, 0, 3, has_embed=True, has_head=True, device="cpu", dtype=torch.float32)
    w = dataclasses.replace(cpu, layers=[dataclasses.replace(lay, **{
        f.name: getattr(lay, f.name).to(device) for f in dataclasses.fields(lay)
        if isinstance(getattr(lay, f.name), torch.Tensor)}) for lay in cpu.layers],
        **{k: getattr(cpu, k).to(device) for k in ("embed", "final_norm", "lm_head")})
    ex = StageExecutor(c, w, device, dtype=torch.float32, max_sessions=2, max_seq_len=128, kv_cache_bytes=8 << 20, warmup=False)
    t = U.ids(50, 90)
    want = sequential_oracle(c, cpu, t)
    got = [ex.forward([("a", 40)], t[:40].to(device), logit_rows=range(40)).cpu()]
    got += [ex.forward([("a", 1)], t[i:i + 1].to(device)).cpu() for i in range(40, 50)]  # (a replay's output is reused)
    torch.testing.assert_close(torch.cat(got).float(), want, **TOL)


def test_a_post_norm_stream_refuses_them():
    c = dataclasses.replace(sequential(), stream="post")
    with pytest.raises(ValueError, match="pre-norm"):
        c.validate()


# ------------------------------------------------------------------ scheduler, sampling, command line
def test_greedy_generation_through_the_scheduler(model):
    cfg, w, d = model
    reqs = [(U.ids(n, cfg["vocab"], n).tolist(), 5 + n % 3) for n in (1, 2, 9, 40, 71, 5, 18)]
    want = [O.greedy(cfg, w, torch.tensor(p), n) for p, n in reqs]
    ex = U.executor(d, "cpu", "fp32")
    assert serve(ex, reqs, batch=3, n_slots=2) == want
    assert serve(ex, reqs, batch=6, prefill_chunk=4, max_step_tokens=11) == want
    assert not ex.sessions.sessions


def test_trace_run_program(model, tmp_path):
    cfg, w, d = model
    a, b = U.ids(20, cfg["vocab"], 1), U.ids(9, cfg["vocab"], 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:11].tolist(), "want": [0, 10]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:8].tolist(), "want": []},
                                     {"id": "a", "tokens": a[11:12].tolist(), "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[8:].tolist(), "want": []}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[12:].tolist(), "want": [7, 2]},
                                     {"id": "c", "tokens": b.tolist(), "want": [8]}], "end": ["a", "c"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype", "float32", "--out",
                        str(tmp_path), "--max-tokens", "128", "--device", "cpu"], text=True, capture_output=True,
                       input="".join(json.dumps(s) + "\n" for s in steps), timeout=240)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {k}" for k in range(4)]
    A, B = ref(cfg, w, a), ref(cfg, w, b)
    want = {0: A[[0, 10]], 1: A[[11]], 3: torch.stack([A[19], A[14], B[8]])}
    assert sorted(os.listdir(tmp_path)) == [f"{k}.f32" for k in sorted(want)]
    for k, y in want.items():
        got = torch.from_numpy(np.fromfile(tmp_path / f"{k}.f32", "<f4").reshape(-1, cfg["vocab"]))
        torch.testing.assert_close(got, y, **TOL)


def test_cli_generates(tmp_path):
    """Client (stage 0) and tail server from ``python -m src.main`` over TCP, greedy, against the oracle."""
    from tests.test_engine_gloo import _free_port

    cfg = U.config([U.att(mlp=U.dense()), U.att(mlp=U.moe()), U.att(2, 2, 8, 8, 8)], vocab=300)
    w = U.tensors(cfg, seed=8)
    d = U.write(tmp_path / "m", cfg, w)
    reg, p1, p0, pr = (_free_port() for _ in range(4))
    env = dict(os.environ, OMP_NUM_THREADS="1")
    common = [sys.executable, "-m", "src.main", "--model", d, "--splits", "2", "--dtype", "fp32", "--device", "cpu",
              "--host", "127.0.0.1", "--device_channel", "off", "--max_seq_len", "128", "--max_sessions", "4",
              "--temperature", "0", "--kv_cache_gb", "0.05"]
    srv = subprocess.Popen(common + ["--stage", "1", "--dht_port", str(reg), "--rpc_port", str(p1)], cwd=ROOT, env=env,
                           stdout=subprocess.DEVNULL, stderr=subprocess.DEVNULL)
    try:
        r = subprocess.run(common + ["--stage", "0", "--dht_port", str(p0), "--rpc_port", str(pr),
                                     "--dht_initial_peers", f"127.0.0.1:{reg}", "--max_new_tokens", "6", "--prompt",
                                     "hello there"], cwd=ROOT, env=env, capture_output=True, text=True, timeout=150)
        assert r.returncode == 0, r.stderr[-3000:]
    finally:
        srv.kill()
        srv.wait()
    from src.models.tokenizer import load_tokenizer

    tok = load_tokenizer(d, resolve_model(d))
    want = O.greedy(cfg, w, torch.tensor(tok(("hello there")).input_ids[0]), 6)
    if tok.eos_token_id in want:
        want = want[:want.index(tok.eos_token_id)]
    assert f"GENERATED: {tok.decode(want, skip_special_tokens=True)}" in r.stdout
