"""Fubapel on the CPU data path: configuration, loading, every mechanism alone, the executor, the scheduler and the
command line, against the plain oracle (tests/fubapel_oracle.py)."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from src.models.config import looped, resolve_model
from src.ops import mixers as mops
from tests import fubapel_oracle as O
from tests import fubapel_utils as U
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
def test_registry_reads_every_size(tmp_path):
    cfg = U.MODELS["mixed"]
    c = resolve_model(U.write(tmp_path, cfg, U.tensors(cfg)))
    runs = O.layer_runs(cfg)
    assert (c.model_type, c.hybrid, c.num_hidden_layers) == ("fubapel", True, len(runs))
    assert (c.vocab_size, c.hidden_size, c.rms_norm_eps, c.residual_mult) == (157, 72, 1e-5, 0.6)
    assert (c.stream, c.norm, c.embed_positions) == ("pre", "layer", False)
    for sp, i in zip(c.layers, runs):
        e = cfg["layers"][i]
        m, mlp = e["mixer"], e["mlp"]
        assert (sp.mixer, sp.heads, sp.dim, sp.vdim, sp.source) == (e["type"], m["heads"], m["dim"], m["vdim"], i)
        assert (sp.ff, sp.limit) == ((mlp["ff"], mlp["limit"]) if mlp else (0, 0.0))
        if e["type"] != "mlstm":
            assert (sp.rot_dims, sp.rot_base) == (m["rot"]["dims"], m["rot"]["base"])
        if e["type"] == "latent_attention":
            assert (sp.q_rank, sp.kv_rank, sp.rot_dim, sp.scale) == (m["q_rank"], m["kv_rank"], m["rot_dim"], m["scale"])
        if e["type"] == "retention":
            assert sp.decay == tuple(m["decay"])
        if e["type"] == "mlstm":
            assert sp.gate_cap == m["gate_cap"]
    assert type(c).from_hf_dict(json.loads(json.dumps(cfg))).layers == c.layers
    assert c.layer_param_bytes(1.0) > 0 and c.kv_bytes_per_token_per_layer() > 0


def test_loops():
    sp = resolve_model("tiny-fubapel").layers[0]
    order = lambda *a: [x.source for x in looped([sp] * 4, *a)]  # noqa: E731
    assert order(None) == [0, 1, 2, 3]
    assert order({"start": 1, "stop": 3, "times": 3}) == [0, 1, 2, 1, 2, 1, 2, 3]
    assert order({"start": 0, "stop": 4, "times": 1}) == [0, 1, 2, 3]
    for bad in ({"start": 2, "stop": 1, "times": 1}, {"start": 0, "stop": 5, "times": 1}, {"start": 0, "stop": 1, "times": 0}):
        with pytest.raises(ValueError, match="loop"):
            order(bad)


@pytest.mark.parametrize("change,match", [
    (lambda c: c["layers"][0].update(type="other"), "unsupported mixer"),
    (lambda c: c["layers"][0]["mixer"]["decay"].pop(), "decay per head"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=2), "rot_dim"),
    (lambda c: c["layers"][1]["mlp"].update(kind="moe"), "feed-forward kind"),
    (lambda c: c["layers"][1]["mlp"].update(limit=0.0), "limit"),
    (lambda c: c["layers"][2]["mixer"].update(gate_cap=0), "gate_cap")])
def test_bad_configurations_are_refused(tmp_path, change, match):
    cfg = json.loads(json.dumps(U.MODELS["mixed"]))
    change(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(ValueError, match=match):
        resolve_model(str(tmp_path))


def test_wrong_tensor_shape_is_refused(tmp_path):
    cfg = U.MODELS["ffs"]
    w = U.tensors(cfg)
    w["l2.mix.uk"] = w["l2.mix.uk"][:-1].contiguous()
    with pytest.raises(ValueError, match="mix.uk"):
        U.executor(U.write(tmp_path, cfg, w), "cpu", "fp32")


def test_a_loop_holds_its_weights_once_and_its_states_apart(tmp_path):
    cfg = U.MODELS["mixed"]
    ex = U.executor(U.write(tmp_path, cfg, U.tensors(cfg)), "cpu", "fp32")
    lay = ex.w.layers
    assert lay[1] is lay[4] and lay[2] is lay[5] and lay[1] is not lay[3]
    assert len(ex.cache.rows) == 4 and len(ex.state.states) == 2 + 2 * 2  # (mLSTM: the matrix, normalizer and maximum)
    one = resolve_model(U.write(tmp_path / "n", dict(cfg, loop=None), U.tensors(cfg)))
    assert ex.w.nbytes() == U.executor(one.name, "cpu", "fp32").w.nbytes()


def test_preset_runs_with_random_weights():
    ex = U.executor("tiny-fubapel", "cpu", "fp32")
    assert torch.isfinite(ex.forward([("a", 50)], U.ids(50, 640))).all()
    c = resolve_model("fubapel-7b")
    assert c.num_hidden_layers == 36 and c.state_bytes_per_session_per_layer() > 0


# ------------------------------------------------------------------ mechanisms
@pytest.mark.parametrize("center", [True, False])
def test_stream_norms(center):
    y, res, w = torch.randn(4, 20), torch.randn(4, 20) + 1, torch.randn(20)
    norm = (lambda x: O.layer_norm(x, w.double(), 1e-2)) if center else (lambda x: O.rms(x, 1e-2) * w.double())
    x, got = torch.empty(4, 20), res.clone()
    mops.add_norm(y, got, 0.3, w, 1e-2, x, center)
    want = res.double() + 0.3 * y.double()
    torch.testing.assert_close(got, want.float(), **TOL)
    torch.testing.assert_close(x, norm(want).float(), **TOL)
    out = mops.rows_norm(res, torch.tensor([2, 0], dtype=torch.int32), w, 1e-2, torch.empty(2, 20), center)
    torch.testing.assert_close(out, norm(res.double())[[2, 0]].float(), **TOL)


@pytest.mark.parametrize("block", [4, 12])
def test_clamped_feed_forward(block):
    g, u = 3 * torch.randn(5, 12), 3 * torch.randn(5, 12)
    x = torch.stack([g.view(5, -1, block), u.view(5, -1, block)], 2).reshape(5, 24)
    got = mops.clamped_glu(x, torch.empty(5, 12), block, 1.25)
    torch.testing.assert_close(got, O.clamped_glu(g.double(), u.double(), 1.25).float(), **TOL)
    assert ((g > 1.25) | (u.abs() > 1.25)).any()


@pytest.mark.parametrize("dims,base", [(6, 700.0), (2, 1e6), (10, 10.0)])
def test_rotation(dims, base):
    x, pos = torch.randn(7, 3, 10), torch.tensor([0, 1, 2, 50, 999, 1000, 3])
    from src.ops.reference_mixers import turn

    got = turn(x, mops.rope_table(base, dims, 1001, "cpu")[pos][:, None])
    torch.testing.assert_close(got, O.rotate(x.double(), pos, dims, base).float(), **TOL)
    assert torch.equal(got[0], x[0]) and torch.equal(got[..., dims:], x[..., dims:])


@pytest.mark.parametrize("kind", ["retention", "mlstm"])
def test_recurrences_and_their_states(kind):
    H, D, V, L = 3, 6, 7, 23
    g = torch.Generator().manual_seed(0)
    z = torch.randn(L, 2 * H * (D + V + 1), generator=g)
    q, k, v, gate, zi, zf = z.double().split([H * D, H * D, H * V, H * V, H, H], 1)
    q, k, v = q.reshape(L, H, D), k.reshape(L, H, D), v.reshape(L, H, V)
    state = torch.full((2, H, D, V), 1e9)  # what a slot's last user left
    seq, ctx, out = torch.ones(L, dtype=torch.int32), torch.arange(1, L + 1, dtype=torch.int32), torch.empty(L, H * V)
    if kind == "retention":
        decay = torch.tensor([0.0, 0.6, 1.0], dtype=torch.float64)
        pos = torch.arange(L)
        o, S = O.retention_scan(O.rotate(q, pos, 4, 90.0), O.rotate(k, pos, 4, 90.0) * D ** -0.5, v, decay)
        want = O.rms(o, 1e-3).reshape(L, -1) * gate * O.sigmoid(gate)
        mops.retention(z[:, : 2 * H * (D + V)], mops.rope_table(90.0, 4, L, "cpu"), torch.log2(decay).clamp(min=-1e30).float(),
                       state, seq, ctx, out, 1e-3)
    else:
        z[:, -2 * H:] *= 8
        zi, zf = z[:, -2 * H:-H].double(), z[:, -H:].double()
        b, nw = torch.randn(2, H, generator=g), torch.randn(H * V, generator=g)
        li, lf = O.soft_cap(zi + b[0].double(), 5.0), O.log_sigmoid(O.soft_cap(zf + b[1].double(), 5.0))
        o, (S, n, m) = O.mlstm_scan(q * D ** -0.5, k, v, li, lf)
        want = O.rms(o, 1e-3).reshape(L, -1) * nw.double() * O.sigmoid(gate)
        aux = torch.full((2, H, D + 1), -1e9)
        mops.mlstm(z, b, 5.0, nw, state, aux, seq, ctx, out, 1e-3)
        torch.testing.assert_close(aux[1], torch.cat([n, m[:, None]], 1).float(), **TOL)
    torch.testing.assert_close(out, want.float(), **TOL)
    torch.testing.assert_close(state[1], S.float(), **TOL)
    assert (state[0] == 1e9).all()


def latent_case(L, H, D, R, V, C, seed=0, spike=None):
    g = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    c, kr, q = rnd(L, C), rnd(L, R), rnd(L, H, D + R)
    uk, uv, sink = rnd(H, D, C) / C ** 0.5, rnd(H, V, C) / C ** 0.5, rnd(H)
    if spike is not None:  # one query and one key share a direction no other token has much of
        i, j = spike
        d = torch.sign(rnd(C))
        c[j] = 2 * d
        q[i] = 0
        q[i, :, :D] = (uk @ d) * 6 / (uk @ d).norm(dim=-1, keepdim=True)
    return c, kr, q, uk, uv, sink


def latent_oracle(c, kr, q, uk, uv, sink, scale, D, base=90.0):
    c, kr, q, uk, uv, sink = (t.double() for t in (c, kr, q, uk, uv, sink))
    pos = torch.arange(c.shape[0])
    R = kr.shape[1]
    kr = O.rotate(kr[:, None], pos, R, base)[:, 0]
    o = O.latent_core(q[..., :D], O.rotate(q[..., D:], pos, R, base), torch.einsum("lc,hdc->lhd", c, uk), kr,
                      torch.einsum("lc,hvc->lhv", c, uv), sink, scale)
    return o.flatten(1).float()


def latent_product(c, kr, q, uk, uv, sink, scale, D, base=90.0, page=8):
    """The ops on a paged cache whose pages are not in order."""
    L, C, R = c.shape[0], c.shape[1], kr.shape[1]
    n = (L + page - 1) // page
    pages = torch.randperm(n + 2, generator=torch.Generator().manual_seed(1))[:n]
    cache = torch.full((n + 2, 1, page, C + R), 7.0)
    table = torch.full((2, n), -1, dtype=torch.int32)
    table[1] = pages.int()
    pos = torch.arange(L)
    rope = mops.rope_table(base, R, L, "cpu")
    ctx = (pos + 1).int()
    z = torch.cat([torch.randn(L, 3), c, kr], 1)
    mops.latent_prep(z, torch.ones(3), torch.ones(C), torch.empty(L, 3), cache, pages[pos // page] * page + pos % page, ctx,
                     rope, 1e-6)
    return mops.latent_attention(q.flatten(1), uk.transpose(1, 2).contiguous(), uv, sink, rope, cache, table,
                                 torch.ones(L, dtype=torch.int32), ctx, torch.empty(L, uv.shape[0] * uv.shape[1]), scale)


@pytest.mark.parametrize("L,H,D,R,V,C", [(40, 3, 8, 4, 6, 10), (9, 1, 1, 2, 1, 1), (33, 2, 5, 6, 9, 16)])
def test_latent_attention_alone(L, H, D, R, V, C):
    a = latent_case(L, H, D, R, V, C)
    want = latent_oracle(O.rms(a[0].double(), 1e-6), *a[1:], 0.3, D)
    torch.testing.assert_close(latent_product(*a, 0.3, D), want, **TOL)
    off = list(a)
    off[5] = torch.full((H,), -1e30)  # an oracle without the sink must show at the first tokens
    assert (latent_oracle(O.rms(a[0].double(), 1e-6), *off[1:], 0.3, D)[:4] - want[:4]).abs().max() > 0.05


@pytest.mark.parametrize("i,j", [(39, 0), (39, 7), (39, 8), (16, 15), (16, 16), (8, 7), (31, 24)])
def test_a_far_key_stands_out(i, j):
    a = latent_case(40, 3, 8, 4, 6, 24, spike=(i, j))
    res = []
    for sign in (1, -1):
        c = a[0].clone()
        c[j] *= sign
        got = latent_product(c, *a[1:], 1.0, 8)[i]
        torch.testing.assert_close(got, latent_oracle(O.rms(c.double(), 1e-6), *a[1:], 1.0, 8)[i], **TOL)
        res.append(got)
    assert (res[0] - res[1]).abs().max() > 0.3


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


def leftovers(ex, value):
    """Fill every page and slot: whatever is left there must not be read."""
    for s in ([] if ex.state is None else ex.state.states) + ex.cache.rows + ex.cache.rk:
        s.fill_(value)


def test_pages_and_slots_are_used_again(model):
    cfg, w, d = model
    ex = U.executor(d, "cpu", "fp32", max_sessions=2, num_pages=3, page_size=64)
    for k in range(5):
        t, u = U.ids(100 + k, cfg["vocab"], k), U.ids(30, cfg["vocab"], 50 + k)
        torch.testing.assert_close(ex.forward([(f"s{k}", t.numel())], t)[0], ref(cfg, w, t)[-1], **TOL)
        torch.testing.assert_close(ex.forward([(f"u{k}", 30)], u)[0], ref(cfg, w, u)[-1], **TOL)
        with pytest.raises(Exception):
            ex.forward([(f"x{k}", 1)], t[:1])  # no third slot
        ex.sessions.close(f"s{k}")
        ex.sessions.close(f"u{k}")
        leftovers(ex, 1e6)
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
    """Stages may be cut inside a loop: every run is a layer of its own."""
    cfg, w, d = model
    L = len(O.layer_runs(cfg))
    s0 = U.executor(d, "cpu", "bf16", role="stage0", end=1)
    s1 = U.executor(d, "cpu", "bf16", role="segment", start=1, end=2)
    s2 = U.executor(d, "cpu", "bf16", role="last", start=2, end=L)
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
    with pytest.raises(ValueError, match="rewound"):
        ex.forward([("b", 1)], t[:1], starts=[10])
    got = ex.forward([("b", 30)], t, starts=[0])  # from the first token it can always start over
    torch.testing.assert_close(got[0], ref(cfg, w, t)[-1], **TOL)


def test_bf16_path_is_close(model):
    cfg, w, d = model
    t = U.ids(120, cfg["vocab"], 2)
    want = ref(cfg, w, t)
    got = U.executor(d, "cpu", "bf16").forward([("a", 120)], t, logit_rows=range(120)).float()
    err = (got - want).pow(2).mean(-1).sqrt() / want.std()
    # (a head of one value is normed to its sign, which rounding can flip: not every position can be close)
    assert err.quantile(0.95) < 0.1


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

    cfg = U.config([U.ret(), U.mla(), U.mem()], vocab=300, loop={"start": 0, "stop": 2, "times": 2})
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
