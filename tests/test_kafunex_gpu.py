"""Kafunex on the GPU: every HIP kernel against the plain oracle (tests/kafunex_oracle.py), then the executor, its
graphs and the scheduler end to end, in bf16 and in 32-bit."""
import pytest
import torch

from src import ops
from src.ops import hybrid as hops
from tests import kafunex_oracle as O
from tests import kafunex_utils as U

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = {"bf16": torch.bfloat16, "fp32": torch.float32}
TOL = {"bf16": dict(atol=3e-2, rtol=2e-2), "fp32": dict(atol=1e-4, rtol=1e-4)}
FP32 = dict(atol=2e-5, rtol=2e-5)


def close(got, want, tol):
    torch.testing.assert_close(got.float().cpu(), want.float().cpu(), **tol)


# ------------------------------------------------------------------ small kernels
@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("W", [64, 70, 33, 1024, 4096])
def test_embedding_and_positions(dt, W):
    table = torch.randn(50, W).to(DTYPES[dt])
    ids, pos = torch.randint(0, 50, (9,)), torch.tensor([0, 1, 2, 3, 100, 4095, 32000, 7, 8])
    res, xb = torch.empty(9, W, device=DEV), torch.empty(9, W, dtype=DTYPES[dt], device=DEV)
    hops.embed_pos(ids.to(DEV), table.to(DEV), pos.to(DEV), hops.position_frequencies(W, DEV), res, xb)
    want = torch.cat([O.sinusoid(1, W, start=int(p)) for p in pos]) + table[ids].double()
    close(res, want, FP32)
    assert torch.equal(xb, res.to(DTYPES[dt]))


@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("n,W", [(1, 64), (300, 70), (5, 4096), (300, 4096), (3, 33), (2, 6144)])
def test_residual_and_row_norms(dt, n, W):
    y, res, w = torch.randn(n, W).to(DTYPES[dt]), torch.randn(n, W), torch.randn(W)
    want = res.double() + O.rms(y.double(), 1e-5) * w.double()
    r, xb = res.to(DEV), torch.empty(n, W, dtype=DTYPES[dt], device=DEV)
    hops.residual_norm(y.to(DEV), r, w.to(DEV), 1e-5, xb)
    close(r, want, FP32)
    assert torch.equal(xb, r.to(DTYPES[dt]))
    rows = torch.tensor([n - 1, 0], dtype=torch.int32)
    out = hops.rows_norm(res.to(DEV), rows.to(DEV), w.to(DEV), 1e-5, torch.empty(2, W, dtype=DTYPES[dt], device=DEV))
    close(out, (O.rms(res.double(), 1e-5) * w.double())[rows.long()], TOL[dt])


def test_residual_norm_of_slabs_and_packed_copy():
    n, W = 21, 512
    part, res, w = torch.randn(5, n, W), torch.randn(n, W), torch.randn(W)
    r, xb = res.to(DEV), torch.zeros(ops.packed_numel(n, W), dtype=torch.bfloat16, device=DEV)
    hops.residual_norm(part.to(DEV), r, w.to(DEV), 1e-5, xb, packed=True)
    close(r, res.double() + O.rms(part.double().sum(0), 1e-5) * w.double(), FP32)
    assert torch.equal(ops.unpack_act(xb, n, W), r.bfloat16())


@pytest.mark.parametrize("dt", sorted(DTYPES))
def test_squared_relu(dt):
    x = torch.randn(37, 72).to(DTYPES[dt])
    out = hops.relu2(x.to(DEV), torch.empty(37, 72, dtype=DTYPES[dt], device=DEV))
    close(out, x.double().clamp(min=0) ** 2, TOL[dt])


@pytest.mark.parametrize("kern", ["pk", "sk", "lds22", "lds24", "lds42", "rw"])
@pytest.mark.parametrize("M", [1, 7, 33, 64])
def test_squared_relu_epilogue(kern, M):
    K, N = 1024, 2048
    x, w = torch.randn(M, K).bfloat16(), (torch.randn(N, K) / 32).bfloat16()
    want = (x.double() @ w.double().t()).clamp(min=0) ** 2
    wp = ops.pack_weight(w.to(DEV))
    ops.set_gemm_sk(kern)
    ops.gemm_workspace(DEV)
    for packed in (False, True):
        out = torch.zeros(ops.packed_numel(M, N), dtype=torch.bfloat16, device=DEV) if packed else \
            torch.zeros(M, N, dtype=torch.bfloat16, device=DEV)
        ops.linear(ops.pack_act(x.to(DEV)), None, wp=wp, a_rows=M, out=out, epilogue=4, out_packed=packed)
        close(ops.unpack_act(out, M, N) if packed else out, want, dict(atol=3e-2, rtol=2e-2))


def test_fp32_greedy_and_sampling():
    x = torch.randn(5, 176, device=DEV)[:, :171]
    assert torch.equal(ops.argmax(x).cpu(), x.cpu().argmax(-1))
    n = 5
    out = ops.sample(x, torch.full((n,), 1.0, device=DEV), torch.ones(n, device=DEV),
                     torch.ones(n, dtype=torch.int32, device=DEV), torch.ones(n, device=DEV),
                     torch.zeros(n, 50, dtype=torch.int32, device=DEV), torch.zeros(n, dtype=torch.int32, device=DEV),
                     torch.arange(n, device=DEV))
    assert torch.equal(out.cpu(), x.bfloat16().float().cpu().argmax(-1))  # top-1


# ------------------------------------------------------------------ recurrence
def rec_case(ntoks, H, D, V, dt, starts, seed=0):
    g = torch.Generator().manual_seed(seed)
    T, S = sum(ntoks), len(ntoks)
    z = torch.randn(T, H * (2 * D + V), generator=g)
    z[:, H * D: 2 * H * D] *= 3
    z[::7, H * D: 2 * H * D] = -60.0  # gates at their lower bound (0 for some channels): the past is dropped
    z[3::11, H * D: 2 * H * D] = 40.0  # and gates of exactly 1
    z = z.to(DTYPES[dt])
    b, lo, nw = torch.randn(H * D, generator=g), torch.rand(H * D, generator=g), torch.randn(V, generator=g)
    lo[::3] = 0.0
    state = torch.randn(S + 1, H, D, V, generator=g)
    outs, states, at = [], state.double().clone(), 0
    for i, n in enumerate(ntoks):
        zq, zf, v = z[at:at + n].double().split([H * D, H * D, H * V], 1)
        f = O.forget_gate(zf, b.double(), lo.double()).view(n, H, D)
        o, states[i + 1] = O.hgrn2_scan((zq * torch.sigmoid(zq)).view(n, H, D), f, v.view(n, H, V),
                                        states[i + 1] if starts[i] else None)
        outs.append((O.rms(o, 1e-6) * nw.double()).reshape(n, -1))
        at += n
    q_seq = torch.cat([torch.full((n,), i + 1) for i, n in enumerate(ntoks)]).int()
    q_ctx = torch.cat([torch.arange(s + 1, s + n + 1) for n, s in zip(ntoks, starts)]).int()
    return z, b, lo, nw, state, q_seq, q_ctx, torch.cat(outs), states


def run_rec(case, dt, plan, packed=False):
    z, b, lo, nw, state, q_seq, q_ctx, _, _ = case
    T, HV = z.shape[0], state.shape[1] * state.shape[3]
    st = state.to(DEV)
    out = torch.zeros(ops.packed_numel(T, HV) if packed else T * HV, dtype=DTYPES[dt], device=DEV)
    hops.hgrn2(z.to(DEV), b.to(DEV), lo.to(DEV), nw.to(DEV), st, q_seq.to(DEV), q_ctx.to(DEV), out, 1e-6, plan=plan,
               packed=packed)
    return (ops.unpack_act(out, T, HV) if packed else out.view(T, HV)), st


def device_plan(ntoks, heads, seg_tokens=None, scan=False):
    p = hops.hgrn2_plan(ntoks, heads, seg_tokens=seg_tokens)
    up = lambda a: torch.from_numpy(a).to(DEV)  # noqa: E731
    return {"seqs": up(p["seqs"]), "seg": up(p["seg"]), "multi": up(p["multi"]) if p["slots"] else None,
            "slots": p["slots"], "scan": scan}


REC_TOL = {"bf16": dict(atol=4e-2, rtol=2e-2), "fp32": dict(atol=3e-4, rtol=3e-4)}


@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("H,D,V", [(2, 16, 16), (3, 40, 32), (2, 20, 33), (1, 1, 1), (2, 64, 128), (2, 128, 128),
                                   (1, 100, 200), (1, 256, 64), (1, 200, 256)])
@pytest.mark.parametrize("form", ["chunk", "segments", "scan"])
def test_recurrence_prompts(dt, H, D, V, form):
    ntoks, starts = [33, 1, 2, 150, 16, 17], [0, 5, 0, 9, 1, 0]
    case = rec_case(ntoks, H, D, V, dt, starts)
    plan = device_plan(ntoks, H, 32 if form == "segments" else None, form == "scan")
    out, st = run_rec(case, dt, plan)
    if V > 1:
        close(out, case[7], REC_TOL[dt])
    close(st[1:], case[8][1:], dict(atol=2e-4, rtol=2e-4))
    assert torch.equal(st[0].cpu(), case[4][0])  # nobody's slot


@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("H,D,V", [(2, 16, 16), (3, 40, 32), (2, 20, 33), (2, 128, 128), (1, 300, 64)])
def test_recurrence_decode(dt, H, D, V):
    n, starts = 9, [0, 3, 0, 1, 7, 20, 1, 1, 2]
    case = rec_case([1] * n, H, D, V, dt, starts)
    out, st = run_rec(case, dt, None)
    close(out, case[7], REC_TOL[dt])
    close(st[1:], case[8][1:], dict(atol=1e-4, rtol=1e-4))
    if dt == "bf16" and (H * V) % 32 == 0:
        close(run_rec(case, dt, None, packed=True)[0], case[7], REC_TOL[dt])
    case = list(case)
    case[6] = torch.zeros_like(case[6])  # padding rows: nothing is read or written
    assert torch.equal(run_rec(case, dt, None)[1].cpu(), case[4])


def test_larger_heads_fall_to_the_scan():
    case = rec_case([40, 3], 1, 300, 64, "fp32", [0, 2])
    out, st = run_rec(case, "fp32", device_plan([40, 3], 1))
    close(out, case[7], REC_TOL["fp32"])
    close(st[1:], case[8][1:], dict(atol=2e-4, rtol=2e-4))


# ------------------------------------------------------------------ attention
def att_case(ntoks, starts, H, G, D, dt, page=64, spike=None, seed=0):
    """Sequences whose first ``starts`` tokens are cached by an earlier step; returns everything on the device and
    the per-sequence fp64 inputs."""
    g = torch.Generator().manual_seed(seed)
    seqs, full = [], []
    for i, (n, s) in enumerate(zip(ntoks, starts)):
        L = n + s
        q, k = torch.randn(L, H * D, generator=g), torch.randn(L, G * D, generator=g)
        if spike is not None and spike[0] == i:
            d = torch.sign(torch.randn(D, generator=g))
            q[spike[1]], k[spike[2]] = 3 * d.repeat(H), 3 * d.repeat(G)
        seqs.append(torch.cat([q, k, torch.randn(L, H * D, generator=g)], 1).to(DTYPES[dt]))
    wq, wk = 1 + 0.3 * torch.randn(H * D, generator=g), 1 + 0.3 * torch.randn(G * D, generator=g)
    talk = (torch.eye(H) + 0.3 * torch.randn(H, H, generator=g)).bfloat16().float()
    npg = [(z.shape[0] + page - 1) // page for z in seqs]
    perm = torch.randperm(sum(npg) + 3, generator=g)[: sum(npg)]
    cache = torch.full((sum(npg) + 3, G, page, D), float("nan"), dtype=DTYPES[dt], device=DEV)
    cache.fill_(77.0)
    rk = torch.full((sum(npg) + 3, page), 5.0, device=DEV)
    table = torch.full((len(seqs) + 1, max(npg)), -1, dtype=torch.int32)
    at, slots = 0, []
    for i, z in enumerate(seqs):
        pages = perm[at:at + npg[i]]
        table[i + 1, : npg[i]] = pages.int()
        at += npg[i]
        p = torch.arange(z.shape[0])
        slots.append(pages[p // page] * page + p % page)
    wqk = (wq * wk.view(G, 1, D).expand(G, H // G, D).reshape(-1)).to(DEV)

    def prep(z, sl):
        qn = torch.zeros(z.shape[0], H * D, dtype=DTYPES[dt], device=DEV)
        hops.talk_prep(z.to(DEV), wqk, qn, cache, rk, sl.to(DEV), 1e-6)
        return qn

    past = [z[:s] for z, s in zip(seqs, starts)]
    if sum(starts):
        prep(torch.cat(past), torch.cat([sl[:s] for sl, s in zip(slots, starts)]))
    z = torch.cat([z[s:] for z, s in zip(seqs, starts)])
    qn = prep(z, torch.cat([sl[s:] for sl, s in zip(slots, starts)]))
    q_seq = torch.cat([torch.full((n,), i + 1) for i, n in enumerate(ntoks)]).int().to(DEV)
    q_ctx = torch.cat([torch.arange(s + 1, s + n + 1) for n, s in zip(ntoks, starts)]).int().to(DEV)
    return dict(z=z.to(DEV), qn=qn, talk=talk.to(DEV), cache=cache, rk=rk, table=table.to(DEV), q_seq=q_seq,
                q_ctx=q_ctx), seqs, wq, wk, talk


def att_oracle(seqs, ntoks, wq, wk, talk, H, G, D, chunk, scale):
    out = []
    for z, n in zip(seqs, ntoks):
        q, k, gate = z.double().split([H * D, G * D, H * D], 1)
        L = z.shape[0]
        o = O.attention_core((O.rms(q, 1e-6) * wq.double()).view(L, H, D), (O.rms(k, 1e-6) * wk.double()).view(L, G, D),
                             k.view(L, G, D), scale, talk.double(), chunk).reshape(L, H * D)
        out.append((o * torch.sigmoid(gate))[L - n:])
    return torch.cat(out)


def run_att(a, H, G, D, ntoks, chunk, scale, form, parts=None, packed=False):
    T = a["z"].shape[0]
    out = torch.zeros(ops.packed_numel(T, H * D) if packed else T * H * D, dtype=a["z"].dtype, device=DEV)
    kw = {}
    if form is not None:
        kw["sigma"] = hops.talk_sigma(a["talk"])
        if parts is not None:
            kw.update(parts=parts, ws=torch.full((parts[1] * T * H * (D + 2),), 3.0, device=DEV))
        else:
            tb = hops.talk_block(H, G, D)
            assert tb > 0
            kw["blocks"] = torch.from_numpy(hops.talk_blocks(ntoks, tb)).to(DEV)
    hops.talk_attention(**a, out=out, chunk=chunk, scale=scale, packed=packed, **kw)
    return ops.unpack_act(out, T, H * D) if packed else out.view(T, H * D)


@pytest.fixture(params=[1, 2])
def form(request, monkeypatch):
    monkeypatch.setattr(hops, "TALK_FORM", request.param)
    return request.param


SHAPES = [(4, 2, 80), (1, 1, 32), (2, 2, 64), (6, 3, 48), (8, 1, 128), (16, 4, 128), (32, 8, 128), (32, 4, 64), (12, 4, 96),
          (24, 8, 40), (10, 2, 8), (16, 16, 32), (20, 5, 64)]
PROMPTS = ([70, 2, 1, 130, 33], [0, 30, 63, 64, 100])


@pytest.mark.parametrize("H,G,D", SHAPES)
@pytest.mark.parametrize("chunk", [1, 50, 64, 1000])
def test_attention_prompts(H, G, D, chunk, form):
    ntoks, starts = PROMPTS
    a, *rest = att_case(ntoks, starts, H, G, D, "bf16")
    want = att_oracle(rest[0], ntoks, *rest[1:], H, G, D, chunk, D ** -0.5)
    close(run_att(a, H, G, D, ntoks, chunk, D ** -0.5, form), want, TOL["bf16"])


@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("H,G,D", [(4, 2, 80), (1, 1, 1), (6, 3, 20), (3, 1, 130), (32, 32, 128), (64, 8, 128)])
def test_attention_any_shape(dt, H, G, D):
    ntoks, starts = [20, 1, 2, 40], [0, 30, 63, 64]
    a, *rest = att_case(ntoks, starts, H, G, D, dt)
    want = att_oracle(rest[0], ntoks, *rest[1:], H, G, D, 37, 0.2)
    close(run_att(a, H, G, D, ntoks, 37, 0.2, None), want, TOL[dt])


@pytest.mark.parametrize("H,G,D", SHAPES)
@pytest.mark.parametrize("chunk", [50, 64, 300])
@pytest.mark.parametrize("split", [1, 3])
def test_attention_decode(H, G, D, chunk, split, form):
    starts = [0, 30, 49, 50, 63, 64, 200, 299, 300, 511]
    ntoks = [1] * len(starts)
    a, *rest = att_case(ntoks, starts, H, G, D, "bf16")
    want = att_oracle(rest[0], ntoks, *rest[1:], H, G, D, chunk, D ** -0.5)
    ps = 32 * -(-(chunk + 31) // (32 * split))
    parts = (ps, -(-(chunk + 31) // ps))
    close(run_att(a, H, G, D, ntoks, chunk, D ** -0.5, form, parts), want, TOL["bf16"])
    if (H * D) % 32 == 0:
        close(run_att(a, H, G, D, ntoks, chunk, D ** -0.5, form, parts, packed=True), want, TOL["bf16"])


@pytest.mark.parametrize("i,j,seen", [(99, 50, True), (100, 50, False), (100, 100, True), (100, 99, False),
                                      (149, 100, True), (150, 100, False), (127, 100, True), (128, 127, True)])
def test_a_standing_out_key_at_a_chunk_edge(i, j, seen, form):
    """Chunks of 50, pages and key tiles at 64 and 32: in a prompt and decoded, the key counts exactly in its chunk."""
    H, G, D, chunk = 4, 2, 80, 50
    for ntoks, starts in (([i + 1], [0]), ([1], [i])):
        res = []
        for flip in (1, -1):
            a, seqs, *rest = att_case(ntoks, starts, H, G, D, "bf16", spike=(0, i, j))
            if flip < 0:
                seqs = [seqs[0].clone()]
                seqs[0][j, H * D:(H + G) * D] *= -1
                if j >= starts[0]:
                    a["z"][j - starts[0], H * D:(H + G) * D] *= -1
                pg, off = int(a["table"][1, j // 64]), j % 64
                a["cache"][pg, :, off] *= -1
            parts = None if starts == [0] else hops.talk_parts(1, H, G, D, chunk)
            got = run_att(a, H, G, D, ntoks, chunk, 0.3, form, parts)[-1]
            close(got, att_oracle(seqs, ntoks, *rest, H, G, D, chunk, 0.3)[-1], TOL["bf16"])
            res.append(got.float())
        assert ((res[0] - res[1]).abs().max() > 0.2) == seen


# ------------------------------------------------------------------ executor
@pytest.fixture(scope="module", params=sorted(U.MODELS) + ["packed"])
def model(request, tmp_path_factory):
    if request.param == "packed":  # every GEMM has a decode form, the recurrence and attention fill their tiles
        cfg = U.config([U.rec(4, 64, 64, 512), U.att(8, 2, 64, 100, ff=384), U.rec(2, 128, 128, 256),
                        U.att(4, 4, 64, 33, ff=128)], vocab=333, width=256)
    else:
        cfg = U.MODELS[request.param]
    w = U.tensors(cfg, seed=3)
    return cfg, w, U.write(tmp_path_factory.mktemp(request.param), cfg, w), request.param


def check(got, want, dt, name, scale):
    if dt == "fp32":
        return torch.testing.assert_close(got.float().cpu(), want, atol=1e-3, rtol=1e-3)
    err = (got.float().cpu() - want).pow(2).mean(-1).sqrt() / scale
    # (heads of one value are normed to their sign, which rounding can flip)
    assert err.quantile(0.9 if name == "ones" else 1.0) < 0.12, err


@pytest.mark.parametrize("dt", sorted(DTYPES))
def test_prompts_decoding_portions_and_batches(model, dt):
    cfg, w, d, name = model
    n = 150
    toks = {k: U.ids(n, cfg["vocab"], s) for s, k in enumerate("abc")}
    want = {k: O.forward(cfg, w, t).float() for k, t in toks.items()}
    scale = want["a"].std()
    ex = U.executor(d, DEV, dt, max_sessions=4)
    check(ex.forward([("w", n)], toks["a"].to(DEV), logit_rows=range(n)), want["a"], dt, name, scale)
    ex.sessions.close("w")
    # one token at a time (graph replays), three sessions of different lengths together
    got = {k: [] for k in toks}
    ex.forward([("a", 5), ("b", 2), ("c", 64)], torch.cat([toks["a"][:5], toks["b"][:2], toks["c"][:64]]).to(DEV))
    at = {"a": 5, "b": 2, "c": 64}
    for _ in range(70):
        x = torch.cat([toks[k][at[k]:at[k] + 1] for k in toks]).to(DEV)
        y = ex.forward([(k, 1) for k in toks], x)
        assert ex.last_graphed
        for r, k in enumerate(toks):
            got[k].append(y[r].float().cpu())
            at[k] += 1
    for k, lo in (("a", 5), ("b", 2), ("c", 64)):
        check(torch.stack(got[k]), want[k][lo:lo + 70], dt, name, scale)
    # portions beside decoded tokens
    for step in ({"a": 2, "b": 1}, {"b": 30, "c": 1, "a": 1}, {"a": 17, "b": 3}, {"c": 2, "a": 40, "b": 1}):
        x = torch.cat([toks[k][at[k]:at[k] + m] for k, m in step.items()]).to(DEV)
        rows = list(range(x.numel()))
        y = ex.forward(list(step.items()), x, logit_rows=rows).cpu()
        off = 0
        for k, m in step.items():
            check(y[off:off + m], want[k][at[k]:at[k] + m], dt, name, scale)
            off += m
            at[k] += m
    # everything given back and used again, whatever it holds
    for k in toks:
        ex.sessions.close(k)
    for s in ([] if ex.state is None else ex.state.states) + ex.cache.rows + ex.cache.rk:
        s.fill_(1e4)
    check(ex.forward([("z", n)], toks["b"].to(DEV), logit_rows=range(n)), want["b"], dt, name, scale)


def test_wide_decode_batches(model):
    """65 and more rows take other GEMM forms."""
    cfg, w, d, name = model
    ex = U.executor(d, DEV, "bf16", max_sessions=80, max_seq_len=64, kv_cache_bytes=512 << 20)
    t = U.ids(80 * 6, cfg["vocab"], 5).view(80, 6)
    ex.forward([(f"s{i}", 5) for i in range(80)], t[:, :5].reshape(-1).to(DEV))
    y = ex.forward([(f"s{i}", 1) for i in range(80)], t[:, 5].to(DEV)).float().cpu()
    want = torch.stack([O.forward(cfg, w, t[i])[-1].float() for i in range(80)])
    check(y, want, "bf16", name, want.std())


def test_greedy_generation_through_the_scheduler(model):
    from tests.test_kafunex import serve

    cfg, w, d, name = model
    reqs = [(U.ids(n, cfg["vocab"], n).tolist(), 6 + n % 3) for n in (1, 2, 9, 40, 71)]
    want = [O.greedy(cfg, w, torch.tensor(p), n) for p, n in reqs]
    ex = U.executor(d, DEV, "fp32")
    assert serve(ex, reqs, batch=3, n_slots=2) == want
    assert serve(ex, reqs, batch=5, prefill_chunk=4, max_step_tokens=11) == want
    out = serve(U.executor(d, DEV, "bf16"), reqs, batch=4)  # bf16 may part from it at a near tie
    assert all(len(a) == len(b) for a, b in zip(out, want))
