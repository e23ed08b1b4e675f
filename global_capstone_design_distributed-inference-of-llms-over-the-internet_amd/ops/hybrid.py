"""Ops of the hybrid decoders (post-norm fp32 residual stream, HGRN2, chunked talking-heads attention).

Same dispatch rule as the package: GPU tensors run the HIP kernels (csrc/post_norm.hip, csrc/hgrn2.hip,
csrc/attention_talk.hip), CPU tensors the plain-PyTorch forms of ``reference_hybrid``.  ``packed`` writes an
activation in the packed decode-GEMM layout.
"""
from __future__ import annotations

import numpy as np
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
    _, H, D, V = state.shape
    if plan is None:
        torch.ops.mpamd.hgrn2_scan(z, bias, lower, norm, state, q_seq, q_ctx, out, float(eps), None, int(packed))
    elif D <= CHUNK_MAX and V <= CHUNK_MAX and not plan.get("scan"):
        slots = plan["slots"]
        ws = torch.empty(slots * H * D * (V + 1), dtype=torch.float32, device=z.device) if slots else None
        torch.ops.mpamd.hgrn2_chunk(z, bias, lower, norm, state, q_seq, q_ctx, out, float(eps), plan["seg"],
                                    plan["multi"], slots, ws, int(packed))
    else:
        torch.ops.mpamd.hgrn2_scan(z, bias, lower, norm, state, q_seq, q_ctx, out, float(eps), plan["seqs"],
                                   int(packed))
    return out


# largest head sizes of the chunk form (csrc/hgrn2.hip hgrn2_chunk_kernel)
CHUNK_MAX = 256


def hgrn2_plan(ntoks, heads: int, n_cu: int = 256, seg_tokens: int = None):
    """Segments of a ragged step for the chunk form: int32 ``seqs`` [2, n] (first flat token, tokens of every
    sequence that brings any), ``seg`` [4, nseg], ``multi`` [4, nm] and the number of workspace slots
    (csrc/hgrn2.hip).  Sequences are cut so that about two workgroups per CU exist, at whole 16-token blocks."""
    n = np.asarray(ntoks, dtype=np.int64)
    off = np.concatenate([[0], np.cumsum(n)[:-1]])
    keep = n > 0
    off, n = off[keep], n[keep]
    if seg_tokens is None:
        want = max(1, -(-2 * n_cu // max(heads, 1)))  # segments over the whole step
        seg_tokens = max(128, 16 * (-(-int(n.sum()) // want) // 16))
    seg, multi, slots = [], [], 0
    for o, c in zip(off.tolist(), n.tolist()):
        k = max(1, -(-c // seg_tokens)) if c > seg_tokens * 3 // 2 else 1
        per = 16 * -(-c // (16 * k))
        k = -(-c // per)
        if k == 1:
            seg.append((o, c, -1, -1))
            continue
        multi.append((slots, k, o, 0))
        for i in range(k):
            seg.append((o + i * per, min(per, c - i * per), slots + i, slots + i + 1 if i < k - 1 else -1))
        slots += k
    mk = lambda v, r: np.ascontiguousarray(np.asarray(v, dtype=np.int32).reshape(-1, r).T)  # noqa: E731
    return {"seqs": np.stack([off, n]).astype(np.int32), "seg": mk(seg, 4), "multi": mk(multi, 4), "slots": slots}


def talk_prep(z, wqk, qn, cache, rk, slots, eps):
    """Query / key norms of projected rows [q | k | gate]: ``qn`` gets the scaled queries, the raw key rows go to
    ``cache`` and their reciprocal root mean squares to ``rk`` at ``slots`` (-1: skip)."""
    if not _native(z):
        return rh.talk_prep(z, wqk, qn, cache, rk, slots, eps)
    torch.ops.mpamd.talk_prep(z, wqk, qn, cache, rk, slots, float(eps))


# MFMA form of the attention: 0 = by shape, 1 = mixing folded into the queries, 2 = scores exchanged through LDS
TALK_FORM = 0


def talk_block(H: int, G: int, D: int) -> int:
    """Tokens of a prompt's query block on the MFMA forms (0: shape not covered)."""
    return int(torch.ops.mpamd.talk_block(int(H), int(G), int(D), TALK_FORM))


def talk_slopes(H: int) -> torch.Tensor:
    """fp32 [H]: the heads' distance slopes, 2^(-8 (h + 1) / H)."""
    return torch.exp2(-8.0 * torch.arange(1, H + 1, dtype=torch.float64) / H).float()


def talk_sigma(talk: torch.Tensor) -> torch.Tensor:
    """fp32 [H]: the slopes after the heads' mixing."""
    return (talk.double() @ talk_slopes(talk.shape[0]).to(talk.device).double()).float()


def talk_blocks(ntoks, tokens: int):
    """Query blocks of a ragged step: int32 [2, nblk] (first flat token, tokens)."""
    out, off = [], 0
    for n in ntoks:
        for k in range(0, int(n), tokens):
            out.append((off + k, min(tokens, int(n) - k)))
        off += int(n)
    return np.ascontiguousarray(np.asarray(out, dtype=np.int32).reshape(-1, 2).T)


def talk_parts(rows: int, H: int, G: int, D: int, span: int, n_cu: int = 256):
    """(keys per split, splits) of a decode step whose queries see at most ``span`` keys: one workgroup per CU
    (what fits one), no split under 64 keys.  (The first split starts on a 32-key boundary at or before the first key.)"""
    span = int(span) + 31
    want = max(1, n_cu // max(1, rows))
    n = max(1, min(want, span // 64))
    ps = 32 * -(-span // (32 * n))
    return ps, -(-span // ps)


def talk_attention(z, qn, talk, cache, rk, table, q_seq, q_ctx, out, chunk, scale, packed=False, sigma=None,
                   blocks=None, parts=None, ws=None):
    """Chunked talking-heads attention with the output gate of ``z``.  On the GPU the MFMA form runs when
    ``blocks`` (prompt steps: ``talk_blocks`` on the device) or ``parts`` (decode: ``talk_parts``, ``ws`` fp32
    scratch) is given, with ``sigma`` = talk @ slopes (``talk_sigma``), else the form for any shape and element type."""
    if not _native(z):
        return _put(out, rh.talk_attention(z, qn, talk, cache, rk, table, q_seq, q_ctx, chunk, scale), packed)
    if blocks is not None or parts is not None:
        ps, np_ = parts if blocks is None else (0, 1)
        torch.ops.mpamd.talk_mfma(z, qn, talk, sigma, cache, rk, table, q_seq, q_ctx, out, int(chunk), float(scale), blocks,
                                  int(ps), int(np_), ws, int(packed), TALK_FORM)
        return out
    torch.ops.mpamd.talk_attention(z, qn, talk, cache, rk, table, q_seq, q_ctx, out, int(chunk), float(scale),
                                   int(packed))
    return out
