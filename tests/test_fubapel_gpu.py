"""Fubapel on the GPU: every HIP kernel against the plain oracle (tests/fubapel_oracle.py), then the executor, its
graphs and the scheduler end to end, in bf16 and in 32-bit."""
import pytest
import torch

from src import ops
from src.models.weights import interleave_gate_up
from src.ops import mixers as mops
from tests import fubapel_oracle as O
from tests import fubapel_utils as U

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = {"bf16": torch.bfloat16, "fp32": torch.float32}
TOL = {"bf16": dict(atol=3e-2, rtol=2e-2), "fp32": dict(atol=1e-4, rtol=1e-4)}
FP32 = dict(atol=2e-5, rtol=2e-5)


def close(got, want, tol):
    torch.testing.assert_close(got.float().cpu(), want.float().cpu(), **tol)


# ------------------------------------------------------------------ residual stream and feed-forward
@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("center", [True, False])
@pytest.mark.parametrize("n,W", [(1, 64), (300, 70), (5, 4096), (300, 4096), (3, 33), (2, 6144)])
def test_stream_norms(dt, center, n, W):
    y, res, w = torch.randn(n, W).to(DTYPES[dt]), torch.randn(n, W) + 0.7, torch.randn(W)
    norm = (lambda x: O.layer_norm(x, w.double(), 1e-5)) if center else (lambda x: O.rms(x, 1e-5) * w.double())
    new = lambda k: torch.empty(k, W, dtype=DTYPES[dt], device=DEV)  # noqa: E731
    r, x = res.to(DEV), new(n)
    mops.add_norm(y.to(DEV), r, 0.6, w.to(DEV), 1e-5, x, center)
    want = res.double() + 0.6 * y.double()
    close(r, want, FP32)
    close(x, norm(want), TOL[dt])
    mops.add_norm(None, r, 0.0, w.to(DEV), 1e-5, x, center)
    close(x, norm(want), TOL[dt])
    mops.add_norm(y.to(DEV), r, 0.6, None, 1e-5, None, center)  # (after the last layer: the sum alone)
    close(r, want + 0.6 * y.double(), FP32)
    rows = torch.tensor([n - 1, 0], dtype=torch.int32)
    close(mops.rows_norm(res.to(DEV), rows.to(DEV), w.to(DEV), 1e-5, new(2), center), norm(res.double())[rows.long()],
          TOL[dt])
    table, ids = torch.randn(50, W).to(DTYPES[dt]), torch.randint(0, 50, (n,))
    mops.embed_norm(ids.to(DEV), table.to(DEV), r, w.to(DEV), 1e-5, x, center)
    assert torch.equal(r.cpu(), table[ids].float())
    close(x, norm(table[ids].double()), TOL[dt])


def test_stream_norm_of_slabs_and_packed_output():
    n, W = 21, 512
    part, res, w = torch.randn(5, n, W), torch.randn(n, W), torch.randn(W)
    r, x = res.to(DEV), torch.zeros(ops.packed_numel(n, W), dtype=torch.bfloat16, device=DEV)
    mops.add_norm(part.to(DEV), r, 0.5, w.to(DEV), 1e-5, x, True, packed=True)
    want = res.double() + 0.5 * part.double().sum(0)
    close(r, want, FP32)
    close(ops.unpack_act(x, n, W), O.layer_norm(want, w.double(), 1e-5), TOL["bf16"])


@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("F,block", [(48, 16), (40, 40), (7, 7)])
def test_clamped_glu(dt, F, block):
    g, u = (3 * torch.randn(37, F)).to(DTYPES[dt]), (3 * torch.randn(37, F)).to(DTYPES[dt])
    x = torch.stack([g.view(37, F // block, block), u.view(37, F // block, block)], 2).reshape(37, 2 * F)
    out = mops.clamped_glu(x.to(DEV), torch.empty(37, F, dtype=DTYPES[dt], device=DEV), block, 1.25)
    close(out, O.clamped_glu(g.double(), u.double(), 1.25), TOL[dt])


@pytest.mark.parametrize("kern", ["pk", "sk", "lds22", "lds24", "lds42", "rw"])
@pytest.mark.parametrize("M", [1, 7, 33, 64, 100])
def test_clamped_glu_epilogue(kern, M):
    K, F = 1024, 1024
    x, g, u = torch.randn(M, K).bfloat16(), (torch.randn(F, K) / 16).bfloat16(), (torch.randn(F, K) / 16).bfloat16()
    want = O.clamped_glu(x.double() @ g.double().t(), x.double() @ u.double().t(), 1.25)
    w = interleave_gate_up(g, u).contiguous()
    wp = ops.pack_weight(w.to(DEV))
    ops.set_gemm_sk(kern)
    ops.gemm_workspace(DEV)
    for packed in (False, True):
        if not ops.native_gemm_ok(M, 2 * F, K, 1, packed):
            continue
        out = torch.zeros(ops.packed_numel(M, F), dtype=torch.bfloat16, device=DEV) if packed else \
            torch.zeros(M, F, dtype=torch.bfloat16, device=DEV)
        ops.linear(ops.pack_act(x.to(DEV)), None, wp=wp, a_rows=M, out=out, epilogue=1, out_packed=packed, glu_limit=1.25)
        close(ops.unpack_act(out, M, F) if packed else out, want, TOL["bf16"])


# ------------------------------------------------------------------ linear attention
def lin_case(kind, ntoks, H, D, V, dt, starts, rot=None, seed=0):
    g = torch.Generator().manual_seed(seed)
    T, S = sum(ntoks), len(ntoks)
    rot = D if rot is None else rot
    z = torch.randn(T, mixer_cols(kind, H, D, V), generator=g)
    bias = torch.randn(2, H, generator=g) * 2 + torch.tensor([[-1.0], [3.0]])
    if kind == "mlstm":
        zg = z[:, 2 * H * (D + V):2 * H * (D + V + 1)]
        zg *= 4
        zg[::9, H:] = -40.0   # forget everything
        zg[4::13, :H] = 30.0  # an input that towers over the past
        zg[5::17, :H] = -30.0
    z = z.to(DTYPES[dt])
    decay = [1 - 2.0 ** (-1 - 3 * h) for h in range(H)]
    c = dict(kind=kind, z=z, bias=bias, norm=torch.randn(H * V, generator=g), cap=7.0, eps=1e-5, H=H, D=D, V=V, rot=rot,
             decay=torch.tensor(decay, dtype=torch.float64), state=torch.randn(S + 1, H, D, V, generator=g),
             aux=torch.rand(S + 1, H, D + 1, generator=g), starts=starts, ntoks=ntoks)
    c["q_seq"] = torch.cat([torch.full((n,), i + 1) for i, n in enumerate(ntoks)]).int()
    c["q_ctx"] = torch.cat([torch.arange(s + 1, s + n + 1) for n, s in zip(ntoks, starts)]).int()
    outs, at = [], 0
    c["states"], c["auxs"] = c["state"].double().clone(), c["aux"].double().clone()
    for i, (n, s0) in enumerate(zip(ntoks, starts)):
        q, k, v, gate, rest = z[at:at + n].double().split([H * D, H * D, H * V, H * V, z.shape[1] - 2 * H * (D + V)], 1)
        q, k, v = q.reshape(n, H, D), k.reshape(n, H, D), v.reshape(n, H, V)
        if kind == "mlstm":
            li = O.soft_cap(rest[:, :H] + bias[0].double(), 7.0)
            lf = O.log_sigmoid(O.soft_cap(rest[:, H:2 * H] + bias[1].double(), 7.0))
            st = (c["states"][i + 1], c["auxs"][i + 1][:, :D], c["auxs"][i + 1][:, D]) if s0 else None
            o, (S1, n1, m1) = O.mlstm_scan(q * D ** -0.5, k, v, li, lf, st)
            c["states"][i + 1], c["auxs"][i + 1] = S1, torch.cat([n1, m1[:, None]], 1)
            y = O.rms(o, 1e-5).reshape(n, -1) * c["norm"].double() * O.sigmoid(gate)
        else:
            pos = torch.arange(s0, s0 + n)
            q, k = O.rotate(q, pos, rot, 3000.0), O.rotate(k, pos, rot, 3000.0) * D ** -0.5
            o, c["states"][i + 1] = O.retention_scan(q, k, v, c["decay"], c["states"][i + 1] if s0 else None)
            y = O.rms(o, 1e-5).reshape(n, -1) * gate * O.sigmoid(gate)
        outs.append(y)
        at += n
    c["want"] = torch.cat(outs)
    return c


def mixer_cols(kind, H, D, V):
    from src.models.config import LayerSpec

    return LayerSpec(kind, H, D, V).in_rows


def run_lin(c, dt, plan, packed=False):
    T, HV = c["z"].shape[0], c["H"] * c["V"]
    st, aux = c["state"].to(DEV), c["aux"].to(DEV)
    out = torch.zeros(ops.packed_numel(T, HV) if packed else T * HV, dtype=DTYPES[dt], device=DEV)
    z, q_seq, q_ctx = c["z"].to(DEV), c["q_seq"].to(DEV), c["q_ctx"].to(DEV)
    if c["kind"] == "mlstm":
        mops.mlstm(z, c["bias"].to(DEV), c["cap"], c["norm"].to(DEV), st, aux, q_seq, q_ctx, out, c["eps"], plan=plan,
                   packed=packed)
    else:
        rope = mops.rope_table(3000.0, c["rot"], 800, DEV)
        mops.retention(z, rope, torch.log2(c["decay"]).float().to(DEV), st, q_seq, q_ctx, out, c["eps"], plan=plan,
                       packed=packed)
    return (ops.unpack_act(out, T, HV) if packed else out.view(T, HV)), st, aux


def lin_plan(ntoks, heads, seg_tokens=None, scan=False):
    p = mops.linear_plan(ntoks, heads, seg_tokens=seg_tokens)
    up = lambda a: torch.from_numpy(a).to(DEV)  # noqa: E731
    return {"seqs": up(p["seqs"]), "seg": up(p["seg"]), "multi": up(p["multi"]) if p["slots"] else None,
            "slots": p["slots"], "scan": scan}


LIN_TOL = {"bf16": dict(atol=4e-2, rtol=2e-2), "fp32": dict(atol=3e-4, rtol=3e-4)}
STATE_TOL = dict(atol=3e-4, rtol=3e-4)


def check_lin(c, dt, res):
    out, st, aux = res
    if c["V"] > 1:  # (a head of one value is normed to its sign)
        close(out, c["want"], LIN_TOL[dt])
    close(st[1:], c["states"][1:], STATE_TOL)
    assert torch.equal(st[0].cpu(), c["state"][0])  # nobody's slot
    if c["kind"] == "mlstm":
        close(aux[1:], c["auxs"][1:], STATE_TOL)


KINDS = ["mlstm", "retention"]
LIN_SHAPES = [(2, 16, 16, 16), (3, 40, 32, 8), (2, 20, 33, 20), (1, 2, 1, 2), (2, 64, 128, 32), (2, 128, 128, 128),
              (1, 96, 200, 96), (1, 256, 64, 0), (2, 48, 48, 48), (1, 256, 256, 256), (3, 32, 36, 16)]


@pytest.mark.parametrize("kind", KINDS)
@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("H,D,V,rot", LIN_SHAPES)
@pytest.mark.parametrize("form", ["chunk", "segments", "scan"])
def test_linear_attention_prompts(kind, dt, H, D, V, rot, form):
    ntoks, starts = [33, 1, 2, 150, 16, 97, 32], [0, 5, 0, 9, 1, 0, 64]
    c = lin_case(kind, ntoks, H, D, V, dt, starts, rot)
    check_lin(c, dt, run_lin(c, dt, lin_plan(ntoks, H, 32 if form == "segments" else None, form == "scan")))


@pytest.mark.parametrize("kind", KINDS)
@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("H,D,V,rot", LIN_SHAPES + [(1, 300, 64, 300)])
def test_linear_attention_decode(kind, dt, H, D, V, rot):
    n, starts = 9, [0, 3, 0, 1, 7, 20, 1, 1, 2]
    c = lin_case(kind, [1] * n, H, D, V, dt, starts, rot)
    check_lin(c, dt, run_lin(c, dt, None))
    if dt == "bf16" and (H * V) % 32 == 0:
        close(run_lin(c, dt, None, packed=True)[0], c["want"], LIN_TOL[dt])
    c["q_ctx"] = torch.zeros_like(c["q_ctx"])  # padding rows: nothing is read or written
    _, st, aux = run_lin(c, dt, None)
    assert torch.equal(st.cpu(), c["state"]) and torch.equal(aux.cpu(), c["aux"])


@pytest.mark.parametrize("kind", KINDS)
def test_larger_heads_fall_to_the_scan(kind):
    c = lin_case(kind, [40, 3], 1, 300, 64, "bf16", [0, 2])
    check_lin(c, "bf16", run_lin(c, "bf16", lin_plan([40, 3], 1)))


# ------------------------------------------------------------------ latent attention
def lat_case(ntoks, starts, H, D, R, V, C, dt, page=64, spike=None, sink=None, seed=0):
    """Sequences whose first ``starts`` tokens are cached by an earlier step.  ``spike`` (sequence, query, key): the
    two share a direction no other token has much of."""
    g = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    uk, uv = rnd(H, D, C) / C ** 0.5, rnd(H, V, C) / C ** 0.5
    Q, seqs, qs = 16, [], []
    for i, (n, s) in enumerate(zip(ntoks, starts)):
        z, q = rnd(n + s, Q + C + R), rnd(n + s, H, D + R)
        if spike is not None and spike[0] == i:
            d = torch.sign(rnd(C))
            z[spike[2], Q:Q + C] = 2 * d
            q[spike[1]] = 0
            q[spike[1], :, :D] = (uk @ d) * 12 / (uk @ d).pow(2).sum(-1, keepdim=True) ** 0.5
        seqs.append(z.to(DTYPES[dt]))
        qs.append(q.to(DTYPES[dt]))
    qw, cw = 1 + 0.3 * rnd(Q), 1 + 0.3 * rnd(C)
    if spike is not None:
        cw = torch.ones(C)
    sink = rnd(H) * 2 if sink is None else sink
    uk, uv = uk.to(DTYPES[dt]), uv.to(DTYPES[dt])
    npg = [(z.shape[0] + page - 1) // page for z in seqs]
    perm = torch.randperm(sum(npg) + 3, generator=g)[: sum(npg)]
    cache = torch.full((sum(npg) + 3, 1, page, C + R), 77.0, dtype=DTYPES[dt], device=DEV)
    table = torch.full((len(seqs) + 1, max(npg)), -1, dtype=torch.int32)
    at, slots = 0, []
    for i, z in enumerate(seqs):
        pages = perm[at:at + npg[i]]
        table[i + 1, : npg[i]] = pages.int()
        at += npg[i]
        p = torch.arange(z.shape[0])
        slots.append(pages[p // page] * page + p % page)
    rope = mops.rope_table(700.0, R, 1200, DEV)
    a = dict(seqs=seqs, qs=qs, ntoks=ntoks, starts=starts, uk=uk, uv=uv, sink=sink, cw=cw, qw=qw, H=H, D=D, R=R, V=V, C=C,
             Q=Q, cache=cache, table=table.to(DEV), rope=rope, page=page)

    def prep(lo):
        z = torch.cat([z[s] for z, s in zip(seqs, lo)]).to(DEV)
        sl = torch.cat([x[s] for x, s in zip(slots, lo)]).to(DEV)
        ctx = torch.cat([torch.arange(1, x.shape[0] + 1)[s] for x, s in zip(seqs, lo)]).int().to(DEV)
        cq = torch.zeros(z.shape[0], Q, dtype=DTYPES[dt], device=DEV)
        if z.shape[0]:
            mops.latent_prep(z, qw.to(DEV), cw.to(DEV), cq, cache, sl, ctx, rope, 1e-6)
        return cq

    prep([slice(0, s) for s in starts])
    a["cq"] = prep([slice(s, None) for s in starts])
    a["q"] = torch.cat([q[s:] for q, s in zip(qs, starts)]).reshape(sum(ntoks), -1).to(DEV)
    a["q_seq"] = torch.cat([torch.full((n,), i + 1) for i, n in enumerate(ntoks)]).int().to(DEV)
    a["q_ctx"] = torch.cat([torch.arange(s + 1, s + n + 1) for n, s in zip(ntoks, starts)]).int().to(DEV)
    return a


def lat_oracle(a, scale):
    out, cqs = [], []
    H, D, R, V, C, Q = (a[k] for k in "HDRVCQ")
    for z, q, n in zip(a["seqs"], a["qs"], a["ntoks"]):
        z, q, L = z.double(), q.double(), z.shape[0]
        pos = torch.arange(L)
        c = O.rms(z[:, Q:Q + C], 1e-6) * a["cw"].double()
        kr = O.rotate(z[:, None, Q + C:], pos, R, 700.0)[:, 0]
        kn, v = torch.einsum("lc,hdc->lhd", c, a["uk"].double()), torch.einsum("lc,hvc->lhv", c, a["uv"].double())
        o = O.latent_core(q[..., :D], O.rotate(q[..., D:], pos, R, 700.0), kn, kr, v, a["sink"].double(), scale)
        out.append(o.reshape(L, H * V)[L - n:])
        cqs.append((O.rms(z[:, :Q], 1e-6) * a["qw"].double())[L - n:])
    return torch.cat(out), torch.cat(cqs)


def run_lat(a, scale, form, splits=1, packed=False):
    H, D, R, V, C = (a[k] for k in "HDRVC")
    T = a["q"].shape[0]
    out = torch.zeros(ops.packed_numel(T, H * V) if packed else T * H * V, dtype=a["q"].dtype, device=DEV)
    kw = {}
    if form != "any":
        tb = mops.latent_block(H, D, R, V, C, a["page"])
        assert tb > 0
        kw = dict(u=torch.full((T, H, C + R), 3.0, dtype=torch.bfloat16, device=DEV),
                  oc=torch.full((T, H, C), 3.0, dtype=torch.bfloat16, device=DEV))
        span = int(a["q_ctx"].max())
        ps = 64 * -(-span // (64 * splits))
        kw["parts"] = (ps, -(-span // ps))
        kw["ws"] = torch.full((kw["parts"][1] * T * H * (C + 2),), 3.0, device=DEV)
        if form == "blocks":
            from src.ops.hybrid import talk_blocks

            kw["blocks"] = torch.from_numpy(talk_blocks(a["ntoks"], tb)).to(DEV)
    mops.latent_attention(a["q"], a["uk"].transpose(1, 2).contiguous().to(DEV), a["uv"].to(DEV), a["sink"].to(DEV),
                          a["rope"], a["cache"], a["table"], a["q_seq"], a["q_ctx"], out, scale, packed=packed, **kw)
    return ops.unpack_act(out, T, H * V) if packed else out.view(T, H * V)


LAT_SHAPES = [(4, 64, 16, 64, 128), (1, 8, 8, 4, 32), (8, 64, 32, 64, 128), (3, 40, 24, 20, 96), (16, 128, 64, 128, 512),
              (20, 32, 16, 48, 256), (40, 24, 8, 32, 64), (70, 16, 8, 16, 160), (32, 128, 64, 128, 512), (6, 192, 40, 72, 448)]
LAT_PROMPT = ([70, 2, 1, 130, 33], [0, 30, 63, 64, 100])


@pytest.mark.parametrize("H,D,R,V,C", LAT_SHAPES)
@pytest.mark.parametrize("splits", [1, 2])
def test_latent_prompts(H, D, R, V, C, splits):
    a = lat_case(*LAT_PROMPT, H, D, R, V, C, "bf16")
    want, cq = lat_oracle(a, (D + R) ** -0.5)
    close(a["cq"], cq, TOL["bf16"])
    close(run_lat(a, (D + R) ** -0.5, "blocks", splits), want, TOL["bf16"])


@pytest.mark.parametrize("dt", sorted(DTYPES))
@pytest.mark.parametrize("H,D,R,V,C", [(4, 64, 16, 64, 128), (1, 1, 2, 1, 1), (3, 20, 6, 13, 37), (2, 300, 2, 8, 600)])
def test_latent_any_shape(dt, H, D, R, V, C):
    a = lat_case([20, 1, 2, 300], [0, 30, 63, 64], H, D, R, V, C, dt)
    want, cq = lat_oracle(a, 0.3)
    close(a["cq"], cq, TOL[dt])
    close(run_lat(a, 0.3, "any"), want, TOL[dt])


@pytest.mark.parametrize("H,D,R,V,C", LAT_SHAPES)
@pytest.mark.parametrize("splits", [1, 3])
@pytest.mark.parametrize("page", [64, 128])
def test_latent_decode(H, D, R, V, C, splits, page):
    starts = [0, 30, 49, 50, 63, 64, 200, 299, 300, 511]
    a = lat_case([1] * len(starts), starts, H, D, R, V, C, "bf16", page)
    want, _ = lat_oracle(a, (D + R) ** -0.5)
    close(run_lat(a, (D + R) ** -0.5, "rows", splits), want, TOL["bf16"])
    if (H * V) % 32 == 0:
        close(run_lat(a, (D + R) ** -0.5, "rows", splits, packed=True), want, TOL["bf16"])


def run_wide(a, scale, waves, packed=False):
    """The form that makes every head's own keys and values of the gathered contexts."""
    H, D, R, V, C = (a[k] for k in "HDRVC")
    T, page = a["q"].shape[0], a["page"]
    ctx = [n + s for n, s in zip(a["ntoks"], a["starts"])]
    table = a["table"].cpu().long()
    idx = torch.cat([table[i + 1][torch.arange(n) // page] * page + torch.arange(n) % page for i, n in enumerate(ctx)])
    lat = mops.latent_gather(a["cache"], idx.to(DEV), torch.empty(len(idx), C + R, dtype=torch.bfloat16, device=DEV))
    assert torch.equal(lat, a["cache"].view(-1, C + R)[idx.to(DEV)])
    w = torch.cat([a["uk"], a["uv"]], 1).reshape(H * (D + V), C).to(DEV)
    kv = lat[:, :C] @ w.t()
    blk, off, base, tb = [], 0, 0, 32 * waves
    for n, c in zip(a["ntoks"], ctx):
        blk += [(off + k, min(tb, n - k), base) for k in range(0, n, tb)]
        off, base = off + n, base + c
    out = torch.zeros(ops.packed_numel(T, H * V) if packed else T * H * V, dtype=torch.bfloat16, device=DEV)
    mops.latent_wide(a["q"], kv, lat, a["sink"].to(DEV), a["rope"], a["q_ctx"], out, D, V, scale,
                     torch.tensor(blk, dtype=torch.int32).t().contiguous().to(DEV), waves, packed)
    return ops.unpack_act(out, T, H * V) if packed else out.view(T, H * V)


@pytest.mark.parametrize("H,D,R,V,C", [(4, 64, 16, 64, 128), (1, 8, 16, 8, 32), (3, 40, 32, 24, 96), (8, 128, 64, 128, 512),
                                       (5, 72, 48, 104, 64), (2, 128, 16, 32, 256)])
@pytest.mark.parametrize("waves", [4, 8])
def test_latent_wide(H, D, R, V, C, waves):
    if waves == 8 and D <= 64:
        pytest.skip("the small form has four waves")
    a = lat_case([70, 2, 1, 300, 33, 129], [0, 30, 63, 64, 100, 0], H, D, R, V, C, "bf16")
    want, _ = lat_oracle(a, (D + R) ** -0.5)
    assert mops.latent_wide_ok(D, R, V, C)
    close(run_wide(a, (D + R) ** -0.5, waves), want, TOL["bf16"])
    if (H * V) % 32 == 0:
        close(run_wide(a, (D + R) ** -0.5, waves, packed=True), want, TOL["bf16"])


@pytest.mark.parametrize("form", ["any", "blocks", "rows", "wide"])
@pytest.mark.parametrize("i,j", [(299, 0), (299, 63), (299, 64), (128, 127), (128, 128), (64, 63), (191, 64), (255, 191)])
def test_a_far_key_stands_out(form, i, j):
    """One key among hundreds is what the query asks for: it is found, in a prompt and decoded, wherever its page is;
    and a key after the query is not seen."""
    H, D, R, V, C = 4, 64, 16, 64, 128
    ntoks, starts = ([1], [i]) if form == "rows" else ([i + 1], [0])
    res = []
    for q_at, sign in ((i, 1), (i, -1)):
        a = lat_case(ntoks, starts, H, D, R, V, C, "bf16", spike=(0, q_at, j))
        if sign < 0:
            pg, off = int(a["table"][1, j // 64]), j % 64
            a["cache"][pg, 0, off, :C] *= -1
            a["seqs"][0][j, a["Q"]:a["Q"] + C] *= -1
        got = (run_wide(a, 0.3, 4) if form == "wide" else run_lat(a, 0.3, form))[-1]
        close(got, lat_oracle(a, 0.3)[0][-1], TOL["bf16"])
        res.append(got.float())
    assert (res[0] - res[1]).abs().max() > 0.3


@pytest.mark.parametrize("form", ["any", "blocks", "rows", "wide"])
@pytest.mark.parametrize("sink", [-30.0, 0.0, 4.0, 40.0])
def test_the_sink_counts_once(form, sink):
    """Among the first keys a sink decides how much is left for them; a towering one leaves nothing."""
    H, D, R, V, C = 4, 64, 16, 64, 128
    ntoks, starts = ([1, 1, 1], [0, 1, 130]) if form == "rows" else ([1, 3, 140], [0, 0, 0])
    a = lat_case(ntoks, starts, H, D, R, V, C, "bf16", sink=torch.full((H,), sink))
    for splits in (1, 2) if form in ("blocks", "rows") else (1,):
        got = run_wide(a, 0.2, 4) if form == "wide" else run_lat(a, 0.2, form, splits)
        close(got, lat_oracle(a, 0.2)[0], TOL["bf16"])
    assert (got.abs().max() < 1e-3) == (sink == 40.0)


# ------------------------------------------------------------------ executor
@pytest.fixture(scope="module", params=sorted(U.MODELS) + ["packed"])
def model(request, tmp_path_factory):
    if request.param == "packed":  # every GEMM has a decode form, the recurrences and attention fill their tiles
        cfg = U.config([U.ret(4, 64, 64), U.mla(8, 64, 64, 32, 128, 128, ff=384), U.mem(2, 128, 128),
                        U.mla(5, 32, 64, 16, 256, 160, ff=128), U.ret(2, 128, 128, 64), U.mem(4, 64, 48, ff=256)], vocab=333,
                       width=256, loop={"start": 1, "stop": 3, "times": 2})
    else:
        cfg = U.MODELS[request.param]
    w = U.tensors(cfg, seed=3)
    return cfg, w, U.write(tmp_path_factory.mktemp(request.param), cfg, w), request.param


def check(got, want, dt, name, scale):
    if dt == "fp32":
        return torch.testing.assert_close(got.float().cpu(), want, atol=1e-3, rtol=1e-3)
    err = (got.float().cpu() - want).pow(2).mean(-1).sqrt() / scale
    # (heads of one value are normed to their sign, which rounding can flip)
    assert err.quantile(0.9 if name == "ones" else 1.0) < 0.06, err


@pytest.mark.parametrize("dt", sorted(DTYPES))
def test_prompts_decoding_portions_and_batches(model, dt):
    cfg, w, d, name = model
    n = 230
    toks = {k: U.ids(n, cfg["vocab"], s) for s, k in enumerate("abc")}
    want = {k: O.forward(cfg, w, t).float() for k, t in toks.items()}
    scale = want["a"].std()
    ex = U.executor(d, DEV, dt, max_sessions=4)
    check(ex.forward([("w", n)], toks["a"].to(DEV), logit_rows=range(n)), want["a"], dt, name, scale)
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
        check(torch.stack(got[k]), want[k][lo:lo + 70], dt, name, scale)
    # portions, short and long, beside decoded tokens
    for step in ({"a": 2, "b": 1}, {"b": 30, "c": 1, "a": 1}, {"a": 17, "b": 3}, {"c": 2, "a": 70, "b": 1},
                 {"b": 64, "a": 2, "c": 65}):
        x = torch.cat([toks[k][at[k]:at[k] + m] for k, m in step.items()]).to(DEV)
        y = ex.forward(list(step.items()), x, logit_rows=range(x.numel())).cpu()
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


def test_long_contexts_of_whole_and_cut_prompts(model):
    """1100 tokens: segments of the recurrences, split contexts, both forms of latent attention."""
    cfg, w, d, name = model
    if name != "packed":
        pytest.skip("one model is enough")
    n = 1100
    t = U.ids(n, cfg["vocab"], 7)
    want = O.forward(cfg, w, t, torch.float32).float()
    ex = U.executor(d, DEV, "bf16", max_seq_len=1280, max_tokens_per_step=2048)
    check(ex.forward([("w", n)], t.to(DEV), logit_rows=range(n)), want, "bf16", name, want.std())
    at = 0
    for m in (700, 2, 63, 64, 1, 200, 3, 33, 1, 33):
        y = ex.forward([("c", m)], t[at:at + m].to(DEV), logit_rows=range(m))
        check(y, want[at:at + m], "bf16", name, want.std())
        at += m
    assert at == n


def test_long_contexts_of_the_recurrences_alone():
    """Segments of a session that already has a state."""
    for kind in KINDS:
        ntoks, starts = [700, 3, 513], [40, 0, 0]
        c = lin_case(kind, ntoks, 2, 64, 64, "bf16", starts, 32)
        plan = lin_plan(ntoks, 2, 128)
        assert plan["slots"] > 4
        out, st, _ = run_lin(c, "bf16", plan)
        close(out, c["want"], LIN_TOL["bf16"])
        close(st[1:], c["states"][1:], dict(atol=2e-3, rtol=1e-3))


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
