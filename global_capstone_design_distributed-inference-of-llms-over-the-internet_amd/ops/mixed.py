"""Ops of decoders with head-mixing attention and parallel sublayers (csrc/attention_mixed.hip).

Same dispatch rule as the package: GPU tensors run the HIP kernels, CPU tensors the plain-PyTorch forms of
``reference_mixed``.  Attention and the feed-forward's activation write one buffer [T, K] side by side, the input of the
layer's output projection; ``packed`` writes it in the packed decode-GEMM layout.
"""
from __future__ import annotations

import numpy as np
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


KEYS = 32  # keys of a tile: splits of a context are multiples of it
XCDS = 8


def mfma_ok(H, G, D, V, page, cap):
    """(tokens of a query block of the MFMA form for prompts, 0: not covered; does the decode form cover the shape)."""
    r = int(torch.ops.mpamd.mixed_mfma_ok(int(H), int(G), int(D), int(V), int(page), float(cap)))
    return (r >> 8 if r & 1 else 0), bool(r & 2)


def sum_splits(blocks: int, span: int, n_cu: int = 256):
    """(keys per split, splits) of a prompt's denominators: as many as even out the triangle of a causal mask."""
    span = max(1, int(span))
    n = max(1, min(-(-4 * n_cu // max(1, int(blocks))), span // 256, 16))
    ps = KEYS * -(-span // (KEYS * n))
    return ps, -(-span // ps)


def mixed_blocks(ntoks, starts, tokens: int):
    """Query blocks of a ragged step: int32 [2, n] (first flat token, tokens; 0: a filler).  Workgroup i runs on XCD
    i % 8, and every XCD has an L2 of its own: a sequence's blocks stay on one XCD unless it is more than an XCD's share
    of the keys to read.  Blocks with long contexts come first."""
    seqs, off = [], 0
    for n, s in zip(np.asarray(ntoks).tolist(), np.asarray(starts).tolist()):
        b = [(s + min(k + tokens, n), off + k, min(tokens, n - k)) for k in range(0, n, tokens)]
        if b:
            seqs.append((sum(x[0] for x in b), b))
        off += n
    seqs.sort(key=lambda x: -x[0])
    total = sum(w for w, _ in seqs)
    bins, load = [[] for _ in range(XCDS)], [0] * XCDS
    for w, b in seqs:
        if w * XCDS > total * 1.05:
            for x in b:
                i = load.index(min(load))
                bins[i].append(x)
                load[i] += x[0]
        else:
            i = load.index(min(load))
            bins[i] += b
            load[i] += w
    depth = max((len(b) for b in bins), default=0)
    out = np.zeros((2, depth, XCDS), dtype=np.int32)
    for i, b in enumerate(bins):
        b.sort(key=lambda x: -x[0])
        for k, (_, t, n) in enumerate(b):
            out[:, k, i] = t, n
    return np.ascontiguousarray(out.reshape(2, -1))


def mixed_parts(groups: int, span: int, n_cu: int = 256, least: int = 2 * KEYS):
    """(keys per split, splits) of ``groups`` workgroups whose queries see at most ``span`` keys: about one workgroup per
    CU, no split under ``least`` keys."""
    span = max(1, int(span))
    n = max(1, min(n_cu // max(1, int(groups)), span // least))
    ps = KEYS * -(-span // (KEYS * n))
    return ps, -(-span // ps)


def mixed_attention(z, qn, talk, cache, table, q_seq, q_ctx, vrope, out, K, scale, cap, packed=False, form=0, blocks=None,
                    parts=(0, 1), sums=None, part=None, sum_parts=(0, 1)):
    """Causal attention over the cache, into columns [0, H V) of ``out`` [T, K]; the head gates come from ``z``.
    On the GPU ``form`` 1 (prompts: ``blocks`` [2, n] first token and tokens of every query block) and 2 (decode: every
    row one token) run on MFMA, with the context in ``parts`` (keys per split, splits) and fp32 scratch ``sums``
    [splits T H] and ``part`` [splits T H V] (prompts of several splits) or [splits T G H V]; a prompt's denominators
    have splits of their own (``sum_parts``, ``sums``).  0 takes any shape."""
    if not _native(z):
        y = rx.mixed_attention(z, qn, talk, cache, table, q_seq, q_ctx, vrope, scale, cap)
        return rx.put_columns(out, y, 0, K, packed)
    torch.ops.mpamd.mixed_attention(z, qn, talk, cache, table, q_seq, q_ctx, vrope, out, int(K), float(scale), float(cap),
                                    int(packed), int(form), blocks, int(parts[0]), int(parts[1]), sums, part, int(sum_parts[0]),
                                    int(sum_parts[1]))
    return out
