"""Trace replay: ``bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N``.

Feeds given token ids through a model step by step and writes the logits asked for; nothing is sampled.  It is a
thin driver of the serving stack: ``load_stage_model`` builds the stage, every step is ONE ragged
``StageExecutor.forward`` (prompt portions beside single decoded tokens, hipGraph replay when every entry is one
token), sessions hold cache pages and state slots and give them back when a request ends.

Steps come from standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["b"]}

``want`` lists the places among the entry's tokens whose logits are written, in order, to ``OUT/<step>.f32``
(little-endian fp32 rows of the vocabulary).  ``done <step>`` follows every step.  The cache pool holds N tokens (in
whole pages) and four sessions.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

LIVE_REQUESTS = 4
DTYPES = {"bfloat16": "bf16", "float32": "fp32"}


def build_parser() -> argparse.ArgumentParser:
    p = argparse.ArgumentParser(prog="trace_run", description="replay token ids through a model, write logits")
    p.add_argument("--model", required=True, help="folder with config.json and safetensors weights")
    p.add_argument("--dtype", default="bfloat16", choices=sorted(DTYPES))
    p.add_argument("--out", required=True, help="folder for <step>.f32")
    p.add_argument("--max-tokens", type=int, required=True, help="tokens that live requests hold at most")
    p.add_argument("--device", default=None, help="cuda:N / cpu (default: the GPU if there is one)")
    return p


class TraceRunner:
    def __init__(self, model: str, dtype: str, max_tokens: int, device=None):
        import torch

        from .llama_partition import load_stage_model
        from .models.config import resolve_model
        from .runtime.executor import StageExecutor
        from .runtime.kv_cache import pages_needed

        torch.set_float32_matmul_precision("highest")
        device = torch.device(device or ("cuda:0" if torch.cuda.is_available() else "cpu"))
        page = 64
        pages = max(1, pages_needed(max_tokens, page))
        cfg = resolve_model(model)
        if DTYPES[dtype] == "fp32" and device.type == "cuda" and not cfg.hybrid:
            raise NotImplementedError(f"{cfg.model_type} has no 32-bit kernels on the GPU")
        full = load_stage_model(model, device, "full", dtype=DTYPES[dtype])
        self.ex = StageExecutor(full.cfg, full.weights, device, dtype=full.dtype, page_size=page, num_pages=pages,
                                max_sessions=LIVE_REQUESTS, max_seq_len=pages * page, warmup=False,
                                max_tokens_per_step=max(pages * page, 64))
        self.torch, self.device = torch, device

    def step(self, entries, end):
        """Logits [wanted, vocab] fp32 (CPU) of one step, or None when nothing is wanted."""
        torch = self.torch
        entries = [e for e in entries if e["tokens"]]
        out = None
        if entries:
            want, off, ids = [], 0, []
            for e in entries:
                want += [off + int(k) for k in e.get("want", [])]
                off += len(e["tokens"])
                ids += e["tokens"]
            x = torch.tensor(ids, dtype=torch.long, device=self.device)
            with torch.no_grad():
                y = self.ex.forward([(str(e["id"]), len(e["tokens"])) for e in entries], x, logit_rows=want)
                if want:
                    out = y.float().cpu()
        for sid in end:
            self.ex.sessions.close(str(sid))
        if self.device.type == "cuda":
            torch.cuda.synchronize(self.device)
        return out


def main(argv=None) -> int:
    args = build_parser().parse_args(argv)
    # one kernel choice on every machine: the committed table, no timing at start-up
    os.environ.setdefault("MPAMD_GEMM_AUTOTUNE", "0")
    try:
        run = TraceRunner(args.model, args.dtype, args.max_tokens, args.device)
    except NotImplementedError as e:
        print(f"trace_run: {e}", file=sys.stderr)
        return 3
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        y = run.step(s.get("entries", []), s.get("end", []))
        if y is not None:
            path = os.path.join(args.out, f"{s['step']}.f32")
            y.numpy().astype("<f4").tofile(path)
        print(f"done {s['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
