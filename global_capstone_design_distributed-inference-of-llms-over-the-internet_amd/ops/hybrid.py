"""Ops of the hybrid decoders (post-norm fp32 residual stream, HGRN2, chunked talking-heads attention).

Same dispatch rule as the package: GPU tensors run the HIP kernels (csrc/post_norm.hip, csrc/hgrn2.hip,
csrc/attention_talk.hip), CPU tensors the plain-PyTorch forms of ``reference_hybrid``.  ``packed`` writes an
activation in the packed decode-GEMM layout.
"""
from __future__ import annotations

import torch

from . import reference as ref
from . import reference_hybrid as rh


def _native(t):
    from . import _native as native

    return native(t)


def _put(out, y, packed):
    """Store a CPU result: ``out`` row-major or packed."""
    y = y.to(out.dtype)
    if packed:
        return ref.pack_act(y, out=out)
    out.view(-1)[: y.numel()].copy_(y.reshape(-1))
    return out


def position_frequencies(width: int, device) -> torch.Tensor:
    """fp64 [ceil(width / 2)]: 10000^(-2i / width)."""
    i = torch.arange((width + 1) // 2, dtype=torch.float64)
    return torch.pow(10000.0, -2.0 * i / width).to(device)


def embed_pos(ids, table, positions, inv, res, xb, packed=False):
    """res[t] = table[ids[t]] + sinusoid(positions[t]) (fp32), ``xb`` its activation copy."""
    if not _native(table):
        rh.embed_pos(ids, table, positions, inv, res)
        return _put(xb, res, packed)
    torch.ops.mpamd.embed_pos(ids, table, positions, inv, res, xb, int(packed))
    return xb


def residual_norm(y, res, w, eps, xb, packed=False):
    """res += rms(y) * w, ``xb`` the activation copy.  ``y`` [n, W], or fp32 split-K slabs [S, n, W]."""
    if not _native(res):
        rh.residual_norm(y.sum(0) if y.dim() == 3 else y, res, w, eps)
        return _put(xb, res, packed)
    torch.ops.mpamd.residual_norm(y, res, w, xb, float(eps), int(packed), int(y.dim() == 3))
    return xb


def rows_norm(res, rows, w, eps, out, packed=False):
    """out[i] = rms(res[rows[i]]) * w."""
    if not _native(res):
        return _put(out, rh.rows_norm(res, rows, w, eps), packed)
    torch.ops.mpamd.rows_norm(res, rows, w, out, float(eps), int(packed))
    return out


def relu2(x, out, packed=False):
    """out = max(x, 0)^2."""
    if not _native(x):
        return _put(out, rh.relu2(x), packed)
    torch.ops.mpamd.relu2(x, out, int(packed))
    return out


def hgrn2(z, bias, lower, norm, state, q_seq, q_ctx, out, eps, plan=None, packed=False):
    """HGRN2 over a ragged step.  ``z`` [T, H (2 D + V)], ``state`` [rows, H, D, V] fp32 updated in place for
    row q_seq[t]; a token of context 1 starts from a zero state, a row of context 0 is padding.
    ``plan``: None = every row is one token of its own sequence (decode), else the step's device plan
    (``HybridStage.plan``)."""
    if not _native(z):
        return _put(out, rh.hgrn2(z, bias, lower, norm, state, q_seq, q_ctx, eps), packed)
    torch.ops.mpamd.hgrn2_scan(z, bias, lower, norm, state, q_seq, q_ctx, out, float(eps),
                               None if plan is None else plan["seg"], int(packed))
    return out


def talk_prep(z, wqk, qn, cache, rk, slots, eps):
    """Query / key norms of projected rows [q | k | gate]: ``qn`` gets the scaled queries, the raw key rows go to
    ``cache`` and their reciprocal root mean squares to ``rk`` at ``slots`` (-1: skip)."""
    if not _native(z):
        return rh.talk_prep(z, wqk, qn, cache, rk, slots, eps)
    torch.ops.mpamd.talk_prep(z, wqk, qn, cache, rk, slots, float(eps))


def talk_attention(z, qn, talk, cache, rk, table, q_seq, q_ctx, out, chunk, scale, packed=False):
    """Chunked talking-heads attention with the output gate of ``z``."""
    if not _native(z):
        return _put(out, rh.talk_attention(z, qn, talk, cache, rk, table, q_seq, q_ctx, chunk, scale), packed)
    torch.ops.mpamd.talk_attention(z, qn, talk, cache, rk, table, q_seq, q_ctx, out, int(chunk), float(scale),
                                   int(packed))
    return out
