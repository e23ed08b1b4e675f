"""Forward step of the hybrid decoders inside a StageExecutor (``ModelConfig.layers``).

The residual stream is fp32 and lives in one buffer; a sublayer reads its activation copy ``xb`` and its
RMS-normed, layer-scaled output is added to it:

    z = xb W_in^T          one fused input projection per mixer
    y = mixer(z) W_o^T     hgrn2: recurrence + head norm; attention: norms + cache write, attention + gate
    res += rms(y) n1 ; xb = res
    y = relu2(xb W_up^T) W_down^T
    res += rms(y) n2 ; xb = res

Activations feeding a decode-sized GEMM stay in the packed MFMA-fragment layout where the shape has a native
GEMM (``ops.native_gemm_ok``); other shapes, prompts and fp32 run the library GEMM on row-major activations.
Keys of attention layers live in the executor's paged cache, recurrent states in its ``RecurrentState``.
"""
from __future__ import annotations

import math
from typing import Optional

import torch

from .. import ops
from ..ops import hybrid as hops


class HybridStage:
    """Layer loop of one stage; ``ex`` owns the weights, the cache, the states and the plans."""

    def __init__(self, ex):
        self.ex = ex
        cfg = ex.cfg
        self.W, self.eps = cfg.hidden_size, cfg.rms_norm_eps
        self.inv = hops.position_frequencies(self.W, ex.device)
        # per-layer cache / state index: attention layers count in the paged cache, recurrent ones in the states
        self.index, na, nr = [], 0, 0
        for lay in ex.w.layers:
            if lay.spec.recurrent:
                self.index.append(nr)
                nr += 1
            else:
                self.index.append(na)
                na += 1
        # query-block tokens of each attention shape's MFMA form (0: the any-shape form)
        self.talk_block = {}
        for lay in ex.w.layers:
            sp = lay.spec
            if not sp.recurrent and ex.device.type == "cuda":
                ok = ex.dtype == torch.bfloat16 and ex.cache.page_size >= 32
                self.talk_block[(sp.heads, sp.kv_heads, sp.dim)] = \
                    hops.talk_block(sp.heads, sp.kv_heads, sp.dim) if ok else 0
        self.rec_heads = min([lay.spec.heads for lay in ex.w.layers if lay.spec.recurrent], default=0)
        self.max_chunk = max([lay.spec.chunk for lay in ex.w.layers if not lay.spec.recurrent], default=1)

    def autotune(self) -> None:
        """Decode-GEMM kernel choices for this stage's shapes (none while tuning is off)."""
        if ops.autotune_mode() == "off":
            return
        shapes = {(getattr(lay, n).shape[0], getattr(lay, n).shape[1], 4 if n == "w_up" else 0)
                  for lay in self.ex.w.layers for n in lay.GEMMS if getattr(lay, n + "_p") is not None}
        if self.ex.w.lm_head_p is not None:
            shapes.add((self.ex.w.lm_head.shape[0], self.W, 0))
        # (small products are launch-bound whatever kernel runs them)
        ops.autotune_gemm([s for s in sorted(shapes) if s[0] * s[1] >= 1 << 22], self.ex.device)

    # ------------------------------------------------------------------ GEMMs
    def _packed(self, T: int, w, wp) -> bool:
        """Does the GEMM over ``w`` take a packed T-row activation?"""
        return (wp is not None and self.ex.device.type == "cuda" and ops.gemm_policy() != "hipblaslt" and
                ops.native_gemm_ok(T, w.shape[0], w.shape[1], 0))

    def _act(self, e, name: str, T: int, K: int, packed: bool):
        if packed:
            return e(f"{name}_p{K}", (ops.packed_numel(T, K),))
        return e(f"{name}_{K}", (T, K))

    def _mm(self, x, w, wp, T: int, packed: bool, out):
        if packed:
            return ops.linear(x, None, wp=wp, a_rows=T, out=out)
        return ops.linear(x, w, out=out)

    def _add(self, y_in, w, wp, packed: bool, T: int, res, n, xb, xb_packed: bool, e):
        """res += rms(y_in w^T) n, xb = res.  A packed projection with a split-K form hands its fp32 slabs
        straight to the norm kernel (no reduce launch, no rounding of y)."""
        if packed and ops.rwk_split(T, w.shape[0], w.shape[1]) > 0:
            y = ops.linear_partials(y_in, T, wp=wp, out=e("y", (T, self.W)))
        else:
            y = self._mm(y_in, w, wp, T, packed, e("y", (T, self.W)))
        hops.residual_norm(y, res, n, self.eps, xb, packed=xb_packed)

    # ------------------------------------------------------------------ the step
    def forward(self, x, positions, slots, q_seq, q_ctx, last_rows, T, bufs: Optional[dict] = None, plan=None,
                span: int = 0, prompt=None):
        """``plan``: the ragged step's ``plan`` (None: a decode step, every row one token); ``span``: most keys a
        query sees.  Returns the fp32
        residual rows [T, W] (non-last stage) or the logits of ``last_rows``."""
        ex, W, eps = self.ex, self.W, self.eps
        dev, dt = ex.device, ex.dtype
        layers = ex.w.layers
        cache: dict = {} if bufs is None else bufs

        def e(name, shape, dtype=dt):
            t = cache.get(name)
            if t is None or tuple(t.shape) != tuple(shape) or t.dtype != dtype:
                t = cache[name] = torch.empty(shape, dtype=dtype, device=dev)
            return t

        def entry(i):  # (packed?, buffer) of the activation that layer i's input projection reads
            pk = i < len(layers) and self._packed(T, layers[i].w_in, layers[i].w_in_p)
            return pk, self._act(e, "xb", T, W, pk)

        res = torch.empty(T, W, dtype=torch.float32, device=dev)
        pk, xb = entry(0)
        if ex.is_first:
            hops.embed_pos(x, ex.w.embed, positions, self.inv, res, xb, packed=pk)
        else:
            res.copy_(x)
            self._copy_in(res, xb, pk, T)
        table = ex.sessions.table_dev
        for i, lay in enumerate(layers):
            sp = lay.spec
            if prompt is not None:  # deep prompt: the block input += prompt[i]
                res.index_add_(0, prompt[0], prompt[1][i].float())
                self._copy_in(res, xb, pk, T)
            z = self._mm(xb, lay.w_in, lay.w_in_p, T, pk, e(f"z{sp.in_rows}", (T, sp.in_rows)))
            pko = self._packed(T, lay.w_o, lay.w_o_p)
            o = self._act(e, "o", T, sp.out_cols, pko)
            if sp.recurrent:
                hops.hgrn2(z, lay.f_bias, lay.f_lower, lay.o_norm, ex.state.layer(self.index[i]), q_seq, q_ctx, o, eps,
                           plan=plan, packed=pko)
            else:
                kv, rk = ex.cache.layer(self.index[i])
                qn = e(f"qn{sp.out_cols}", (T, sp.out_cols))
                hops.talk_prep(z, lay.w_qk, qn, kv, rk, slots, eps)
                tb = self.talk_block.get((sp.heads, sp.kv_heads, sp.dim), 0)
                blocks = parts = ws = None
                if tb and plan is not None:
                    blocks = plan["blocks"][tb]
                elif tb:
                    parts = hops.talk_parts(T, sp.heads, sp.kv_heads, sp.dim, min(span, sp.chunk), ex._n_cu)
                    if parts[1] > 1:
                        ws = e("talk_ws", (parts[1] * T * sp.heads * (sp.dim + 2),), torch.float32)
                hops.talk_attention(z, qn, lay.talk, kv, rk, table, q_seq, q_ctx, o, sp.chunk, sp.scale, packed=pko,
                                    sigma=lay.sigma, blocks=blocks, parts=parts, ws=ws)
            if sp.ff:
                pku = self._packed(T, lay.w_up, lay.w_up_p)
                xu = self._act(e, "xb", T, W, pku)
                self._add(o, lay.w_o, lay.w_o_p, pko, T, res, lay.n1, xu, pku, e)
                pkd = self._packed(T, lay.w_down, lay.w_down_p)
                a = self._act(e, "act", T, sp.ff, pkd)
                if pku and ops.native_gemm_ok(T, sp.ff, W, 4):  # the squared relu in the GEMM's epilogue
                    ops.linear(xu, None, wp=lay.w_up_p, a_rows=T, out=a, epilogue=4, out_packed=pkd)
                else:
                    u = self._mm(xu, lay.w_up, lay.w_up_p, T, pku, e(f"u{sp.ff}", (T, sp.ff)))
                    hops.relu2(u, a, packed=pkd)
                pk, xb = entry(i + 1)
                self._add(a, lay.w_down, lay.w_down_p, pkd, T, res, lay.n2, xb, pk, e)
            else:
                pk, xb = entry(i + 1)
                self._add(o, lay.w_o, lay.w_o_p, pko, T, res, lay.n1, xb, pk, e)
        if not ex.is_last:
            return res
        S, V = last_rows.numel(), ex.cfg.vocab_size
        head = ex.w.lm_head
        if S == 0:
            return torch.empty(0, V, dtype=dt, device=dev)
        pkh = self._packed(S, head, ex.w.lm_head_p)
        fn = hops.rows_norm(res, last_rows, ex.w.final_norm, eps, self._act(e, "fn", S, W, pkh), packed=pkh)
        logits = self._mm(fn, head, ex.w.lm_head_p, S, pkh, torch.empty(S, head.shape[0], dtype=dt, device=dev))
        return logits[:, :V]

    def _copy_in(self, res, xb, packed: bool, T: int) -> None:
        y = res.to(self.ex.dtype)
        if packed:
            ops.pack_act(y, out=xb)
        else:
            xb.copy_(y)

    # ------------------------------------------------------------------ plans
    def plan(self, ntoks) -> dict:
        """Device description of a ragged step (not one token per session)."""
        if self.ex.device.type != "cuda":
            return {}
        up = lambda a: torch.from_numpy(a).to(self.ex.device, non_blocking=True)  # noqa: E731
        p = {"blocks": {tb: up(hops.talk_blocks(ntoks, tb)) for tb in set(self.talk_block.values()) if tb}}
        if self.rec_heads:
            h = hops.hgrn2_plan(ntoks, self.rec_heads, self.ex._n_cu)
            p.update(seqs=up(h["seqs"]), seg=up(h["seg"]), multi=up(h["multi"]) if h["slots"] else None,
                     slots=h["slots"])
        return p

    def span(self, max_ctx: int) -> int:
        """Most keys a decode query of context <= max_ctx can see."""
        return max(1, min(int(max_ctx), self.max_chunk))
