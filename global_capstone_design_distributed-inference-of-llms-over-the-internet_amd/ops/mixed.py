"""Ops of decoders with head-mixing attention and parallel sublayers (csrc/attention_mixed.hip).

Same dispatch rule as the package: GPU tensors run the HIP kernels, CPU tensors the plain-PyTorch forms of
``reference_mixed``.  Attention and the feed-forward's activation write one buffer [T, K] side by side, the input of the
layer's output projection; ``packed`` writes it in the packed decode-GEMM layout.
"""
from __future__ import annotations

import torch

from . import reference_mixed as rx
from .hybrid import _native, _put

FF_KINDS = {None: 0, "gelu": 1, "clamped_glu": 2, "gated_glu": 3}


def ffn_act(z, out, kind, F, block=1, limit=0.0, packed=False):
    """Activation of a feed-forward's projected rows: ``gelu`` of [up], the clamped gated form of [gate and up in blocks],
    or (``gated_glu``) that times the sigmoid of the column after them."""
    if not _native(z):
        return _put(out, rx.ffn_act(z, kind, F, block, limit), packed)
    torch.ops.mpamd.ffn_act(z, out, FF_KINDS[kind], int(F), int(block), float(limit), int(packed))
    return out


def mixed_prep(z, q_gain, k_gain, qn, cache, slots, q_ctx, rope, vrope, out, K, eps, ff=None, packed=False):
    """Norms and rotations of projected rows [q | k | v | gate]: ``qn`` gets the queries, keys and turned values go to the
    cache at ``slots`` (-1: skip).  ``ff`` (kind, F, block, column, limit): the feed-forward activation of the row's later
    columns, which goes to columns [H V, H V + F) of ``out`` [T, K]."""
    if not _native(z):
        rx.mixed_prep(z, q_gain, k_gain, qn, cache, slots, q_ctx, rope, vrope, eps)
        if ff is not None:
            kind, F, block, col, limit = ff
            H = qn.shape[1] // q_gain.numel()
            rx.put_columns(out, rx.ffn_act(z[:, col:], kind, F, block, limit), H * vrope.shape[1], K, packed)
        return
    kind, F, block, col, limit = ff if ff is not None else (None, 0, 1, 0, 0.0)
    torch.ops.mpamd.mixed_prep(z, q_gain, k_gain, qn, cache, slots, q_ctx, rope, vrope, out, int(K), FF_KINDS[kind],
                               int(F), int(block), int(col), float(limit), float(eps), int(packed))


def mixed_attention(z, qn, talk, cache, table, q_seq, q_ctx, vrope, out, K, scale, cap, packed=False):
    """Causal attention over the cache, into columns [0, H V) of ``out`` [T, K]; the head gates come from ``z``."""
    if not _native(z):
        y = rx.mixed_attention(z, qn, talk, cache, table, q_seq, q_ctx, vrope, scale, cap)
        return rx.put_columns(out, y, 0, K, packed)
    torch.ops.mpamd.mixed_attention(z, qn, talk, cache, table, q_seq, q_ctx, vrope, out, int(K), float(scale), float(cap),
                                    int(packed))
    return out
