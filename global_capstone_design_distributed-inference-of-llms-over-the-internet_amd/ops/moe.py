"""Mixtral sparse-MoE MLP: top-k softmax routing and the expert combine.

The reference accepts ``model_type == "mixtral"`` (src/llama_partition.py:81-83) and runs
HF ``MixtralSparseMoeBlock`` on the host; this module gives the same math to this
framework's engine:

* routing (HF semantics): ``softmax(router(h))`` over all E experts in fp32, keep the top-k,
  renormalise the kept weights to sum to 1;
* expert j: ``down_j(silu(gate_j h) * up_j h)``; token output = sum_j w_j * expert_j(h).

MI355X execution strategy (runtime/executor.py ``_moe_mlp``):

* decode steps (T <= 64 rows) run EVERY expert on the whole (tiny) batch through the packed
  weight-streaming GEMMs and combine with a dense [T, E] weight matrix whose unrouted
  entries are zero.  A decode step is HBM-bound: at batch 64 with top-2 of 8 experts every
  expert is routed to by some token (P(unused) = (6/8 * 5/7)^64 ~ 1e-10), so the bytes read
  equal the sparse schedule's, the extra MFMA work is free at M <= 64, and the step has no
  data-dependent shapes - it stays inside the hipGraph;
* prefill (T > 64) groups tokens by expert (one host sync per layer, outside any graph),
  runs each expert's GEMMs on its gathered rows and scatter-adds the weighted result.

The hybrid decoders' experts (``choose`` / ``experts``: group-limited softmax routing, clamped gated experts) run on
kernels of their own (csrc/moe.hip): choice, sorting and grouped products stay on the device at every size, so a step
has no host sync and only experts that were chosen are read.
"""
from __future__ import annotations

from typing import Tuple

import torch
import torch.nn.functional as F

from . import reference as ref
from .reference import GU_BLOCK


def route(logits: torch.Tensor, k: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """Router logits [T, E] -> (weights fp32 [T, k] summing to 1, expert ids [T, k])."""
    p = torch.softmax(logits.float(), dim=-1)
    w, idx = torch.topk(p, k, dim=-1)
    return w / w.sum(-1, keepdim=True), idx


def dense_weights(w: torch.Tensor, idx: torch.Tensor, E: int, out: torch.Tensor = None) -> torch.Tensor:
    """Top-k (w, idx) -> dense combine matrix [T, E] (zeros for unrouted experts)."""
    if out is None:
        out = torch.zeros(w.shape[0], E, dtype=torch.float32, device=w.device)
    else:
        out.zero_()
    return out.scatter_(1, idx, w)


def _split(gu: torch.Tensor):
    F2, H = gu.shape
    v = gu.view(F2 // (2 * GU_BLOCK), 2, GU_BLOCK, H)
    return v[:, 0].reshape(F2 // 2, H), v[:, 1].reshape(F2 // 2, H)


def moe_mlp_torch(h: torch.Tensor, router: torch.Tensor, gate_up: torch.Tensor, down: torch.Tensor,
                  k: int) -> torch.Tensor:
    """Differentiable plain-PyTorch MoE MLP in ``h``'s dtype (oracle + stateless autograd stage).

    h [..., H]; router [E, H]; gate_up [E, 2F, H] (16-row interleaved); down [E, H, F]."""
    shp = h.shape
    x = h.reshape(-1, shp[-1])
    w, idx = route(x @ router.t(), k)
    out = torch.zeros_like(x, dtype=torch.float32)
    for e in range(router.shape[0]):
        tok, slot = (idx == e).nonzero(as_tuple=True)
        if tok.numel() == 0:
            continue
        g, u = _split(gate_up[e])
        xe = x[tok]
        y = (F.silu(xe @ g.t()) * (xe @ u.t())) @ down[e].t()
        out = out.index_add(0, tok, y.float() * w[tok, slot].unsqueeze(1))
    return out.to(h.dtype).reshape(shp)


# ------------------------------------------------------------------ grouped experts (hybrid decoders)
GLU_ALPHA = 1.702


def expert_mfma_ok(ff: int, width: int, dtype) -> bool:
    """Do the MFMA kernels cover experts of this shape?"""
    return dtype == torch.bfloat16 and ff % 32 == 0 and width % 32 == 0


class Choice:
    """What a step's tokens chose: ``weights`` [T, top] fp32, ``slot`` [T, top] row of each choice among the rows sorted by
    expert (-1: none), ``tok`` [T top] token of every row, ``lists`` rows by expert, ``spec`` the ``MoESpec``."""

    def __init__(self, spec, weights, slot, tok, lists, tokens):
        self.spec, self.weights, self.slot, self.tok, self.lists, self.tokens = spec, weights, slot, tok, lists, tokens


def _rows(x, packed, T, W):
    return ref.unpack_act(x, T, W) if packed else x


def _choose_cpu(x, w, ctx, m):
    """Plain form of ``choose``: (weights, expert ids, -1 on padding rows)."""
    z = x.float() @ w.float().t()
    s = torch.softmax(z, -1)
    T, E = z.shape
    g = z.view(T, m.groups, E // m.groups).amax(-1)
    best = torch.argsort(g, dim=-1, descending=True, stable=True)[:, : m.keep]
    allowed = torch.zeros(T, m.groups, dtype=torch.bool, device=z.device).scatter_(1, best, True)
    allowed = allowed.repeat_interleave(E // m.groups, 1)
    idx = torch.argsort(z.masked_fill(~allowed, float("-inf")), dim=-1, descending=True, stable=True)[:, : m.top]
    p = s.gather(1, idx)
    p = p / (p.sum(-1, keepdim=True) + 1e-20) * m.scale
    live = (ctx > 0)[:, None]
    return torch.where(live, p, torch.zeros_like(p)), torch.where(live, idx, torch.full_like(idx, -1))


def choose(x, w, ctx, spec, e, packed=False) -> Choice:
    """Router and choice of a step: ``x`` [T, W] (or packed), ``w`` [experts, W], ``ctx`` [T] (0: a padding row, which
    chooses nothing); ``e(name, shape, dtype)`` gives scratch."""
    E, W = w.shape
    T, k = ctx.numel(), spec.top
    weights = e(f"moe_w{k}", (T, k), torch.float32)
    idx, slot = e(f"moe_i{k}", (T, k), torch.int32), e(f"moe_s{k}", (T, k), torch.int32)
    tok = e(f"moe_t{k}", (T * k,), torch.int32)
    if w.device.type != "cuda":
        p, i = _choose_cpu(_rows(x, packed, T, W), w, ctx, spec)
        weights.copy_(p)
        flat = i.reshape(-1)
        order = torch.argsort(torch.where(flat < 0, torch.full_like(flat, E), flat), stable=True)
        n = int((flat >= 0).sum())
        order = order[:n]
        slot.fill_(-1)
        slot.view(-1)[order] = torch.arange(n, dtype=torch.int32)
        tok[:n] = (order // k).to(torch.int32)
        counts = torch.bincount(flat[flat >= 0], minlength=E)
        return Choice(spec, weights, slot, tok, counts, T)
    lists = e(f"moe_l{E}", (torch.ops.mpamd.moe_lists(E),), torch.int32)
    S = torch.ops.mpamd.moe_router_splits(T, W, E, w.dtype == torch.float32)
    part = e(f"moe_z{E}", (S, T, E), torch.float32)
    torch.ops.mpamd.moe_route(x, w, ctx, part, weights, idx, slot, lists, tok, spec.groups, spec.keep, float(spec.scale),
                              int(packed))
    return Choice(spec, weights, slot, tok, lists, T)


def _glu(z, block, limit):
    R, F2 = z.shape
    v = z.view(R, F2 // (2 * block), 2, block)
    g, u = v[:, :, 0].reshape(R, F2 // 2).clamp(max=limit), v[:, :, 1].reshape(R, F2 // 2).clamp(-limit, limit)
    return g * torch.sigmoid(GLU_ALPHA * g) * (u + 1)


def experts(x, c: Choice, up, down, up_p, down_p, block, e, packed=False):
    """Outputs of the chosen experts, one row per choice in the order of ``c.slot`` (fp32, or the activations' type on
    long steps).  ``up`` [E, 2 ff, W] and ``down`` [E, W, ff], or their packed forms."""
    m, R = c.spec, c.tokens * c.spec.top
    dt = (up if up is not None else up_p).dtype
    W = down.shape[1] if down is not None else 16 * down_p.shape[1]
    act = e(f"moe_a{m.ff}", (R, m.ff), dt)
    if x.device.type != "cuda":
        rows = _rows(x, packed, c.tokens, W).float()
        y, at = e("moe_y", (R, W), torch.float32), 0
        for j, n in enumerate(c.lists.tolist()):
            a = _glu(rows[c.tok[at:at + n].long()] @ up[j].float().t(), block, m.limit)
            act[at:at + n] = a.to(dt)
            y[at:at + n] = act[at:at + n].float() @ down[j].float().t()
            at += n
        return y
    form = 0 if up_p is None else expert_form(R, m.experts, packed)
    y = e("moe_y", (R, W), dt if form > 1 else torch.float32)
    torch.ops.mpamd.moe_gemm(form, x, c.tok, c.lists, up_p if form else up, act, R, c.tokens, 1, block, float(m.limit),
                             int(packed))
    torch.ops.mpamd.moe_gemm(form, act, None, c.lists, down_p if form else down, y, R, c.tokens, 0, 1, 0.0, 0)
    return y


# mean rows per expert from which the tiled products (128 and 256 rows a tile) run instead of the weight-streaming one
TILE_ROWS, BIG_TILE_ROWS = 48, 384


def expert_form(rows: int, experts: int, packed: bool) -> int:
    """Product of ``rows`` choices: 1 few rows per expert, 2 many, 3 very many."""
    return 1 if packed or rows < TILE_ROWS * experts else 2 if rows < BIG_TILE_ROWS * experts else 3
