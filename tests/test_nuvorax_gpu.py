"""Nuvorax on the GPU: every HIP kernel against the plain oracle (tests/nuvorax_oracle.py), then the executor, its graphs
and the scheduler end to end, in bf16 and in 32-bit."""
import pytest
import torch

from src import ops
from src.models.config import MoESpec
from src.ops import mixed as xops
from src.ops import mixers as mops
from src.ops import moe as eops
from tests import nuvorax_oracle as O
from tests import nuvorax_utils as U

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = {"bf16": torch.bfloat16, "fp32": torch.float32}
TOL = {"bf16": dict(atol=3e-2, rtol=2e-2), "fp32": dict(atol=1e-4, rtol=1e-4)}


def close(got, want, tol):
    torch.testing.assert_close(got.float().cpu(), want.float().cpu(), **tol)


def near(got, want):
    """bf16 attention: queries, keys, values and mixed weights are rounded, so an error has a size on the whole and a few
    outliers among a million."""
    d, want = got.double().cpu() - want.double(), want.double()
    assert d.pow(2).mean().sqrt() < 6e-3 * want.pow(2).mean().sqrt()
    assert (d.abs() < 0.12 + 0.02 * want.abs()).all()


# ------------------------------------------------------------------ residual stream, projections' ends
@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("n,W,top", [(1, 64, 1), (300, 70, 3), (5, 4096, 4), (3, 33, 6), (300, 4096, 5)])
def test_stream_norm_adds_the_experts_rows(dt, n, W, top):
    y, res, w = torch.randn(n, W).to(DTYPES[dt]), torch.randn(n, W), torch.randn(W)
    slot = torch.randperm(n * top).int().view(n, top)
    slot[0, 0] = -1
    ew = torch.rand(n, top)
    for ydt in {torch.float32, DTYPES[dt]}:
        ye = torch.randn(n * top, W).to(ydt)
        gone = int((set(range(n * top)) - set(slot[slot >= 0].tolist())).pop())
        ye[gone] = float("nan")  # a row that nobody chose is not read
        add = torch.where((slot >= 0)[..., None], ye[slot.clamp(min=0).long()].double(), 0.0) * ew[..., None].double()
        want = res.double() + 0.5 * (y.double() + add.sum(1))
        e = (ye.to(DEV), slot.to(DEV), ew.to(DEV))
        r, x = res.to(DEV), torch.empty(n, W, dtype=DTYPES[dt], device=DEV)
        mops.add_norm(y.to(DEV), r, 0.5, w.to(DEV), 1e-5, x, True, experts=e)
        close(r, want, dict(atol=3e-5, rtol=3e-5))
        close(x, O.layer_norm(want, w.double(), 1e-5), TOL[dt])
        r = res.to(DEV)
        mops.add_norm(None, r, 0.5, w.to(DEV), 1e-5, x, True, experts=e)
        close(r, want - 0.5 * y.double(), dict(atol=3e-5, rtol=3e-5))
    if dt == "bf16" and W % 4 == 0:  # split-K slabs and the last layer's sum alone
        part = torch.randn(3, n, W)
        r = res.to(DEV)
        mops.add_norm(part.to(DEV), r, 0.5, None, 1e-5, None, True, experts=e)
        close(r, want + 0.5 * (part.double().sum(0) - y.double()), dict(atol=3e-5, rtol=3e-5))


@pytest.mark.parametrize("dt", sorted(DTYPES))
def test_scaled_embedding(dt):
    table, ids, w = torch.randn(50, 96).to(DTYPES[dt]), torch.randint(0, 50, (9,)), torch.randn(96)
    r, x = torch.empty(9, 96, device=DEV), torch.empty(9, 96, dtype=DTYPES[dt], device=DEV)
    mops.embed_norm(ids.to(DEV), table.to(DEV), r, w.to(DEV), 1e-5, x, True, scale=3.7)
    close(r, 3.7 * table[ids].double(), dict(atol=1e-6, rtol=1e-6))
    close(x, O.layer_norm(3.7 * table[ids].double(), w.double(), 1e-5), TOL[dt])


@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("packed", [False, True])
@pytest.mark.parametrize("H,G,D,V,rot,kind,F,block", [
    (8, 4, 64, 32, 64, "gelu", 64, 1), (4, 2, 16, 32, 16, "gated_glu", 96, 16), (32, 8, 128, 128, 64, "gated_glu", 512, 16),
    (3, 1, 20, 6, 8, "clamped_glu", 12, 12), (6, 3, 40, 48, 16, "gelu", 40, 1), (2, 2, 8, 16, 0, None, 0, 1),
    (5, 1, 300, 14, 300, "gelu", 7, 1)])
def test_prep(dt, packed, H, G, D, V, rot, kind, F, block):
    """Norms, rotations, cache pages and the feed-forward's activation, against the plain forms."""
    T, K = 37, H * V + F
    if packed and (dt == "fp32" or K % 32):
        pytest.skip("not a packed shape")
    g = torch.Generator().manual_seed(1)
    rn = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    mr = 16 * -(-(H * (D + 1) + G * (D + V)) // 16)
    z = (2 * rn(T, mr + 16 * -(-((F if kind == "gelu" else 2 * F + 1) if kind else 0) // 16))).to(DTYPES[dt])
    qg, kg = 1 + 0.3 * rn(D), 1 + 0.3 * rn(D)
    cache = torch.full((3, G, 32, D + V), 9.0, dtype=DTYPES[dt])
    slots = torch.randperm(96, generator=g)[:T]
    slots[5] = -1  # a padding row
    ctx = torch.randint(1, 900, (T,), generator=g).int()
    rope, vrope = mops.rope_table(700.0, rot, 1000, "cpu", (6.0, 1.0, 4.0, 64.0)), mops.rope_table(700.0, V, 1000, "cpu")
    res = []
    for dev in ("cpu", DEV):
        qn, c = torch.zeros(T, H * D, dtype=DTYPES[dt], device=dev), cache.to(dev, copy=True)
        out = torch.zeros(ops.packed_numel(T, K), dtype=DTYPES[dt], device=dev)
        xops.mixed_prep(*(t.to(dev) for t in (z, qg, kg)), qn, c, slots.to(dev), ctx.to(dev), rope.to(dev), vrope.to(dev), out,
                        K, 1e-5, ff=(kind, F, block, mr, 1.4) if kind else None, packed=packed)
        o = ops.unpack_act(out, T, K) if packed else out[:T * K].view(T, K)
        live = torch.arange(T, device=dev) != 5
        res.append((qn[live].cpu(), c.cpu(), o[:, H * V:].cpu()))
    for a, b in zip(*res):
        close(b, a, dict(atol=2e-2, rtol=1e-2) if dt == "bf16" else dict(atol=2e-5, rtol=2e-5))


@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("kind,F,block", [("gelu", 48, 1), ("clamped_glu", 40, 8), ("gated_glu", 14, 14), ("gelu", 9, 1)])
def test_feed_forward_activation(dt, kind, F, block):
    z = (3 * torch.randn(33, 2 * F + 8)).to(DTYPES[dt])
    got = xops.ffn_act(z.to(DEV), torch.empty(33, F, dtype=DTYPES[dt], device=DEV), kind, F, block, 1.25)
    close(got, xops.ffn_act(z, torch.empty(33, F), kind, F, block, 1.25), TOL[dt])


# ------------------------------------------------------------------ attention
def run_attn(a, form, splits=1, packed=False, pad=0):
    """form: any / blocks / rows; ``splits``: of the contexts."""
    T, H, G, V = a.zr.shape[0], a.H, a.G, a.V
    kw = {}
    if form != "any":
        tb, dec = xops.mfma_ok(H, G, a.D, V, a.page, a.cap)
        assert tb and (dec or form == "blocks")
        span = int(a.q_ctx.max())
        parts = lambda n: (32 * -(-span // (32 * n)), -(-span // (32 * -(-span // (32 * n)))))  # noqa: E731
        kw = dict(parts=parts(splits), form=1 if form == "blocks" else 2)
        n = kw["parts"][1]
        if form == "blocks":
            kw.update(blocks=torch.from_numpy(xops.mixed_blocks(a.ntoks, a.starts, tb)).to(DEV), sum_parts=parts(splits + 1),
                      part=torch.full((n * T * H * V,), 3.0, device=DEV))
            n = kw["sum_parts"][1]
        else:
            kw["part"] = torch.full((n * T * G * H * V,), 3.0, device=DEV)
        kw["sums"] = torch.full((n * T * H,), 3.0, device=DEV)
    out = torch.zeros(ops.packed_numel(T, a.K), dtype=a.dt, device=DEV)
    a.run(out, packed, **kw)
    return (ops.unpack_act(out, T, a.K) if packed else out[:T * a.K].view(T, a.K))[:, :H * V]


PROMPT = ([70, 2, 1, 130, 33], [0, 30, 63, 64, 100])
SHAPES = [(4, 2, 64, 64), (32, 8, 128, 128), (16, 4, 128, 128), (8, 8, 64, 48), (12, 4, 40, 16), (20, 5, 128, 80), (32, 1, 64, 128),
          (1, 1, 8, 16), (18, 6, 72, 32), (24, 12, 96, 112), (7, 7, 16, 32), (10, 2, 80, 96)]


@pytest.mark.parametrize("H,G,D,V", SHAPES)
@pytest.mark.parametrize("splits", [1, 3])
def test_attention_prompts(H, G, D, V, splits):
    a = U.Attn(*PROMPT, H, G, D, V, dt=torch.bfloat16, device=DEV, page=64)
    near(run_attn(a, "blocks", splits), a.want())


@pytest.mark.parametrize("H,G,D,V", SHAPES)
@pytest.mark.parametrize("splits", [1, 3])
@pytest.mark.parametrize("page", [32, 128])
def test_attention_decode(H, G, D, V, splits, page):
    starts = [0, 30, 31, 32, 49, 63, 64, 200, 299, 511]
    pad = (-H * V) % 32
    a = U.Attn([1] * len(starts), starts, H, G, D, V, dt=torch.bfloat16, device=DEV, page=page, pad=pad)
    want = a.want()
    if xops.mfma_ok(H, G, D, V, page, a.cap)[1]:
        near(run_attn(a, "rows", splits), want)
        near(run_attn(a, "rows", splits, packed=True), want)
    near(run_attn(a, "blocks", splits), want)


@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("H,G,D,V", [(4, 2, 64, 64), (1, 1, 1, 2), (3, 1, 20, 6), (36, 6, 24, 10), (2, 2, 300, 200), (9, 3, 16, 14)])
@pytest.mark.parametrize("cap", [20.0, 0.0, 90.0])
def test_attention_any_shape(dt, H, G, D, V, cap):
    a = U.Attn([20, 1, 2, 90], [0, 30, 15, 64], H, G, D, V, dt=DTYPES[dt], device=DEV, page=16, cap=cap,
               gain=1.5 if D < 100 else 0.7)
    close(run_attn(a, "any"), a.want(), TOL[dt])


@pytest.mark.parametrize("form", ["any", "blocks", "rows"])
@pytest.mark.parametrize("cap", [0.5, 30.0, 64.0])
def test_soft_caps_and_the_sink(form, cap):
    """Scores far beyond the cap, both ways; the first tokens, where the sink decides."""
    ntoks, starts = ([1] * 4, [0, 1, 2, 130]) if form == "rows" else ([1, 3, 140], [0, 0, 0])
    a = U.Attn(ntoks, starts, 8, 2, 64, 64, dt=torch.bfloat16, device=DEV, page=64, cap=cap, scale=2.0, gain=2.0)
    for s in (1, 2) if form != "any" else (1,):
        # (a score's rounding counts as it is, and scores reach hundreds before the cap)
        close(run_attn(a, form, s), a.want(), dict(atol=0.1, rtol=5e-2))
    assert (a.want(no_sink=True) - a.want()).abs().max() > 0.1


@pytest.mark.parametrize("form", ["any", "blocks", "rows"])
@pytest.mark.parametrize("H,G,D,V", [(8, 2, 64, 64), (32, 8, 64, 32)])
@pytest.mark.parametrize("i,j", [(299, 0), (299, 63), (299, 64), (128, 127), (128, 128), (64, 63), (191, 64), (255, 191), (32, 31)])
def test_a_far_key_stands_out(form, H, G, D, V, i, j):
    """One key among hundreds is what the query asks for: it is found, in a prompt and decoded, wherever its page is."""
    ntoks, starts = ([1], [i]) if form == "rows" else ([i + 1], [0])
    res = []
    for sign in (1, -1):
        a = U.Attn(ntoks, starts, H, G, D, V, 32, dt=torch.bfloat16, device=DEV, page=64, spike=(i, j), gain=1.5)
        at = slice((H + G) * D, (H + G) * D + G * V)
        a.z[0][j, at] *= sign
        a.prep([slice(0, None)])
        got = run_attn(a, form, 2 if form != "any" else 1)[-1]
        close(got, a.want()[-1], TOL["bf16"])
        res.append(got.float())
    assert (res[0] - res[1]).abs().max() > 0.3


@pytest.mark.parametrize("form", ["blocks", "rows"])
def test_what_a_page_held_before_is_not_read(form):
    ntoks, starts = ([1] * 3, [0, 40, 65]) if form == "rows" else ([1, 41, 66], [0, 0, 0])
    a = U.Attn(ntoks, starts, 8, 2, 64, 64, dt=torch.bfloat16, device=DEV, page=64)
    a.cache.fill_(float("nan"))
    a.prep([slice(0, None)] * 3)
    close(run_attn(a, form, 2), a.want(), TOL["bf16"])


def test_blocks_cover_every_token_once():
    import numpy as np

    for ntoks, starts, tb in (([70, 0, 1, 130, 33], [0, 5, 63, 64, 100], 16), ([1], [9], 8), ([1024] * 8, [0] * 8, 8),
                              ([5000], [0], 16), ([3] * 50, [7] * 50, 8)):
        b = xops.mixed_blocks(ntoks, starts, tb)
        seen = np.concatenate([np.arange(t, t + n) for t, n in b.T])
        assert sorted(seen.tolist()) == list(range(sum(ntoks))) and b[1].max() <= tb
        edges = np.cumsum([0] + ntoks)
        assert all(np.searchsorted(edges, t, "right") == np.searchsorted(edges, t + n - 1, "right") for t, n in b.T if n)


# ------------------------------------------------------------------ experts
def scratch():
    bufs = {}

    def e(name, shape, dtype):
        return bufs.setdefault(name, torch.full(shape, 7, dtype=dtype, device=DEV))
    return e


def check_choice(c, want, live):
    """Dense weights, and that the rows by expert are what the slots say."""
    T, k = c.weights.shape
    E = want.shape[1]
    cnt, off = c.lists[:E].cpu(), c.lists[E:2 * E + 1].cpu()
    act, nact = c.lists[2 * E + 1:3 * E + 1].cpu(), int(c.lists[3 * E + 1])
    assert off[0] == 0 and torch.equal(off.diff(), cnt) and int(off[E]) == int(live.sum()) * k
    assert act[:nact].tolist() == [e for e in range(E) if cnt[e] > 0]
    slot, tok, w = c.slot.cpu().long(), c.tok.cpu(), c.weights.cpu()
    assert (slot[~live] == -1).all() and sorted(slot[live].flatten().tolist()) == list(range(int(off[E])))
    t = torch.arange(T)[live].repeat_interleave(k)
    assert torch.equal(tok[slot[live].flatten()].long(), t)
    e = torch.searchsorted(off[1:].long(), slot[live].flatten(), right=True)
    got = torch.zeros(T, E)
    got[t, e] = w[live].flatten()
    want = torch.where(live[:, None], want, 0.0)
    torch.testing.assert_close(got, want.float(), atol=2e-5, rtol=2e-4)


ROUTERS = [(6, 2, 3, 2, 64), (8, 1, 1, 1, 96), (64, 8, 8, 3, 128), (12, 3, 12, 5, 70), (1, 1, 1, 1, 64), (200, 5, 4, 2, 256),
           (512, 20, 64, 7, 64), (16, 16, 1, 1, 33), (65, 3, 5, 5, 512)]


@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("E,top,count,keep,W", ROUTERS)
@pytest.mark.parametrize("T", [1, 19, 300, 1100])
def test_choice_of_experts(dt, E, top, count, keep, W, T):
    x, w = torch.randn(T, W).to(DTYPES[dt]), (torch.randn(E, W) * 3 / W ** 0.5).to(DTYPES[dt])
    ctx = torch.ones(T, dtype=torch.int32)
    ctx[5::7] = 0  # padding rows
    z = x.double() @ w.double().t()
    want = O.route(z, {"experts": E, "top": top, "scale": 1.9, "groups": {"count": count, "keep": keep}}) if E * T < 40000 else None
    spec = MoESpec(E, top, 8, 1.0, count, keep, 1.9)
    spec.validate()
    if want is None:  # (the plain loop is slow: the CPU path, which the plain loop checks at smaller sizes)
        p, idx = eops._choose_cpu(x.float(), w.float(), torch.ones_like(ctx), spec)
        want = torch.zeros(T, E).scatter_(1, idx, p)
    c = eops.choose(x.to(DEV), w.to(DEV), ctx.to(DEV), spec, scratch())
    check_choice(c, want, ctx > 0)
    if dt == "bf16" and W % 32 == 0:
        xp = ops.pack_act(x.to(DEV))
        check_choice(eops.choose(xp, w.to(DEV), ctx.to(DEV), spec, scratch(), packed=True), want, ctx > 0)


def test_a_router_of_no_numbers_stays_in_bounds():
    x, w = torch.full((40, 64), float("nan")), torch.randn(9, 64)
    c = eops.choose(x.to(DEV), w.to(DEV), torch.ones(40, dtype=torch.int32, device=DEV), MoESpec(9, 4, 8, 1.0, 3, 2), scratch())
    assert sorted(c.slot.cpu().flatten().tolist()) == list(range(160)) and int(c.lists[9 + 9]) == 160


def expert_case(E, W, F, dt, skew=0.0, seed=0):
    g = torch.Generator().manual_seed(seed)
    rn = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    w = {"router": rn(E, W) * 3 / W ** 0.5}
    for e in range(E):
        w.update({f"e{e}.gate": 1.5 * rn(F, W) / W ** 0.5, f"e{e}.up": 1.5 * rn(F, W) / W ** 0.5, f"e{e}.down": rn(W, F) / F ** 0.5})
    w = {k: v.to(DTYPES[dt]) for k, v in w.items()}
    if skew:
        w["router"][0] += skew  # (rows of x are positive on average: nearly everyone wants expert 0)
    return w


def run_experts(w, x, ctx, spec, form, dt, packed=False):
    from src.models.weights import _stacked_gate_up

    E, F, W = spec.experts, spec.ff, w["router"].shape[1]
    pairs = [_stacked_gate_up(w[f"e{e}.gate"], w[f"e{e}.up"]) for e in range(E)]
    up, down = torch.stack([p[0] for p in pairs]).to(DEV), torch.stack([w[f"e{e}.down"] for e in range(E)]).to(DEV)
    upp = downp = None
    if form:
        assert eops.expert_mfma_ok(F, W, DTYPES[dt])
        upp, downp = (torch.stack([ops.pack_weight(t) for t in m]) for m in (up, down))
        up = down = None
    e = scratch()
    xd = ops.pack_act(x.to(DEV)) if packed else x.to(DEV)
    c = eops.choose(xd, w["router"].to(DEV), ctx.to(DEV), spec, e, packed=packed)
    old = eops.expert_form
    eops.expert_form = lambda *a: form
    try:
        y = eops.experts(xd, c, up, down, upp, downp, pairs[0][1], e, packed=packed)
    finally:
        eops.expert_form = old
    res = torch.zeros(x.shape[0], W, device=DEV)
    mops.add_norm(None, res, 1.0, None, 1e-5, None, experts=(y, c.slot, c.weights))
    return res


def experts_want(w, x, ctx, spec):
    m = {"router": {"experts": spec.experts, "top": spec.top, "scale": spec.scale,
                    "groups": {"count": spec.groups, "keep": spec.keep}}, "expert": {"limit": spec.limit}}
    y = O.experts({k: v.double() for k, v in w.items()}, "", x.double(), m)
    return torch.where((ctx > 0)[:, None], y, 0.0)


@pytest.mark.parametrize("dt,form,F,W", [("fp32", 0, 24, 70), ("fp32", 0, 64, 128), ("bf16", 0, 20, 72), ("bf16", 0, 64, 96),
                                         ("bf16", 1, 64, 128), ("bf16", 1, 96, 160), ("bf16", 1, 32, 32), ("bf16", 1, 160, 1024),
                                         ("bf16", 2, 64, 128), ("bf16", 2, 96, 160), ("bf16", 2, 224, 96), ("bf16", 3, 64, 128),
                                         ("bf16", 3, 160, 352), ("bf16", 3, 32, 32)])
@pytest.mark.parametrize("T,skew", [(1, 0.0), (17, 0.0), (150, 0.5), (600, 0.5)])
def test_expert_products(dt, form, F, W, T, skew):
    spec = MoESpec(6, 2, F, 1.3, 3, 2, 1.7)
    w = expert_case(6, W, F, dt, skew)
    x = (torch.randn(T, W, generator=torch.Generator().manual_seed(2)) + (0.3 if skew else 0.0)).to(DTYPES[dt])
    ctx = torch.ones(T, dtype=torch.int32)
    ctx[3::11] = 0
    want = experts_want(w, x, ctx, spec)
    close(run_experts(w, x, ctx, spec, form, dt), want, TOL[dt])
    if form == 1 and W % 32 == 0:
        close(run_experts(w, x, ctx, spec, form, dt, packed=True), want, TOL[dt])


# ------------------------------------------------------------------ executor
@pytest.fixture(scope="module", params=sorted(U.MODELS) + ["packed"])
def model(request, tmp_path_factory):
    if request.param == "packed":  # every GEMM has a decode form, attention and the experts their MFMA forms
        cfg = U.config([U.att(8, 2, 64, 64, 32, cap=30.0, mlp=U.moe(8, 2, 64, 1.5, 4, 2, 1.5, (128, 0.9))),
                        U.att(20, 5, 32, 16, 16, cap=30.0, mlp=U.dense(64)),
                        U.att(4, 4, 64, 32, 64, cap=30.0, mlp=U.moe(5, 3, 32, 1.1, 1, 1, 0.7, None)),
                        U.att(3, 1, 32, 128, 8, cap=80.0, mlp=None)], vocab=333, width=256)
    else:
        cfg = U.MODELS[request.param]
    w = U.tensors(cfg, seed=3)
    return cfg, w, U.write(tmp_path_factory.mktemp(request.param), cfg, w), request.param


def check(got, want, dt, scale):
    if dt == "fp32":
        return torch.testing.assert_close(got.float().cpu(), want, atol=1e-3, rtol=1e-3)
    err = (got.float().cpu() - want).pow(2).mean(-1).sqrt() / scale
    # (a close call of a router goes either way: not every position can be close)
    assert err.quantile(0.85) < 0.08 and err.max() < 1.5, err


@pytest.mark.parametrize("dt", sorted(DTYPES))
def test_prompts_decoding_portions_and_batches(model, dt):
    cfg, w, d, _ = model
    n = 230
    toks = {k: U.ids(n, cfg["vocab"], s) for s, k in enumerate("abc")}
    want = {k: O.forward(cfg, w, t).float() for k, t in toks.items()}
    scale = want["a"].std()
    ex = U.executor(d, DEV, dt, max_sessions=4)
    check(ex.forward([("w", n)], toks["a"].to(DEV), logit_rows=range(n)), want["a"], dt, scale)
    ex.sessions.close("w")
    # one token at a time (graph replays), three sessions of different lengths together
    got = {k: [] for k in toks}
    at = {"a": 5, "b": 2, "c": 64}
    ex.forward(list(at.items()), torch.cat([toks[k][:m] for k, m in at.items()]).to(DEV))
    for _ in range(70):
        x = torch.cat([toks[k][at[k]:at[k] + 1] for k in toks]).to(DEV)
        y = ex.forward([(k, 1) for k in toks], x)
        assert ex.last_graphed
        for r, k in enumerate(toks):
            got[k].append(y[r].float().cpu())
            at[k] += 1
    for k, lo in (("a", 5), ("b", 2), ("c", 64)):
        check(torch.stack(got[k]), want[k][lo:lo + 70], dt, scale)
    # portions, short and long, beside decoded tokens
    pieces, wants = [], []
    for step in ({"a": 2, "b": 1}, {"b": 30, "c": 1, "a": 1}, {"a": 17, "b": 3}, {"c": 2, "a": 70, "b": 1},
                 {"b": 64, "a": 2, "c": 65}):
        x = torch.cat([toks[k][at[k]:at[k] + m] for k, m in step.items()]).to(DEV)
        pieces.append(ex.forward(list(step.items()), x, logit_rows=range(x.numel())).float().cpu())
        for k, m in step.items():
            wants.append(want[k][at[k]:at[k] + m])
            at[k] += m
    check(torch.cat(pieces), torch.cat(wants), dt, scale)
    # everything given back and used again, whatever it holds
    for k in toks:
        ex.sessions.close(k)
    for s in ex.cache.rows:
        s.fill_(1e4)
    check(ex.forward([("z", n)], toks["b"].to(DEV), logit_rows=range(n)), want["b"], dt, scale)


def test_graph_replays_equal_the_eager_step(model):
    """Decode graphs with the experts on a stream of their own, replayed with other work between the replays."""
    cfg, w, d, _ = model
    t = [U.ids(60, cfg["vocab"], s) for s in range(3)]
    outs = []
    for graphs in (True, False):
        ex = U.executor(d, DEV, "bf16", use_graphs=graphs)
        ex.forward([(f"s{i}", 9 + i) for i in range(3)], torch.cat([x[:9 + i] for i, x in enumerate(t)]).to(DEV))
        got = []
        for k in range(20):
            got.append(ex.forward([(f"s{i}", 1) for i in range(3)], torch.stack([x[9 + i + k] for i, x in enumerate(t)]).to(DEV)).cpu())
            assert ex.last_graphed == graphs
            if k % 5 == 2:  # another shape and an eager step in between
                ex.forward([("o", 7 + k)], t[0][:7 + k].to(DEV), reset=[True])
                ex.forward([("o", 1)], t[0][:1].to(DEV))
                torch.cuda.synchronize()
        outs.append(torch.stack(got))
    assert torch.equal(outs[0], outs[1])


def test_long_contexts_of_whole_and_cut_prompts(model):
    """1100 tokens: split contexts and denominators, tiled expert products."""
    cfg, w, d, name = model
    if name != "packed":
        pytest.skip("one model is enough")
    n = 1100
    t = U.ids(n, cfg["vocab"], 7)
    want = O.forward(cfg, w, t, torch.float32).float()
    ex = U.executor(d, DEV, "bf16", max_seq_len=1280, max_tokens_per_step=2048)
    check(ex.forward([("w", n)], t.to(DEV), logit_rows=range(n)), want, "bf16", want.std())
    at, got = 0, []
    for m in (700, 2, 63, 64, 1, 200, 3, 33, 1, 33):
        got.append(ex.forward([("c", m)], t[at:at + m].to(DEV), logit_rows=range(m)).cpu())
        at += m
    assert at == n
    check(torch.cat(got), want, "bf16", want.std())


def test_cuts_change_only_rounding(model):
    """The same tokens whole, in pairs and one by one differ by no more than the product's rounding."""
    cfg, w, d, _ = model
    n = 64
    t = U.ids(n, cfg["vocab"], 11)
    ex = U.executor(d, DEV, "fp32")
    res = []
    for name, sizes in (("w", [n]), ("p", [2] * (n // 2)), ("d", [1] * n)):
        at, got = 0, []
        for m in sizes:
            got.append(ex.forward([(name, m)], t[at:at + m].to(DEV), logit_rows=range(m)).float().cpu())
            at += m
        res.append(torch.cat(got))
    for r in res[1:]:
        torch.testing.assert_close(r, res[0], atol=1e-4, rtol=1e-4)


def test_wide_decode_batches(model):
    """65 and more rows take other GEMM forms."""
    cfg, w, d, _ = model
    ex = U.executor(d, DEV, "bf16", max_sessions=80, max_seq_len=64, kv_cache_bytes=512 << 20)
    t = U.ids(80 * 6, cfg["vocab"], 5).view(80, 6)
    ex.forward([(f"s{i}", 5) for i in range(80)], t[:, :5].reshape(-1).to(DEV))
    y = ex.forward([(f"s{i}", 1) for i in range(80)], t[:, 5].to(DEV)).float().cpu()
    want = torch.stack([O.forward(cfg, w, t[i])[-1].float() for i in range(80)])
    check(y, want, "bf16", want.std())


def test_greedy_generation_through_the_scheduler(model):
    from tests.test_kafunex import serve

    cfg, w, d, _ = model
    reqs = [(U.ids(n, cfg["vocab"], n).tolist(), 6 + n % 3) for n in (1, 2, 9, 40, 71)]
    want = [O.greedy(cfg, w, torch.tensor(p), n) for p, n in reqs]
    ex = U.executor(d, DEV, "fp32")
    assert serve(ex, reqs, batch=3, n_slots=2) == want
    assert serve(ex, reqs, batch=5, prefill_chunk=4, max_step_tokens=11) == want
    out = serve(U.executor(d, DEV, "bf16"), reqs, batch=4)  # bf16 may part from it at a near tie
    assert all(len(a) == len(b) for a, b in zip(out, want))
