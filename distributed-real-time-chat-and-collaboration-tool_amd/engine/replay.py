"""Trace replay: feed given token ids through a checkpoint's model on the serving engine, step by
step, and write the logits that are asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N < steps

Every line of standard input is one step, run as one batch (``LLMEngine.feed``):

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["a"]}

A request is admitted at its first entry and released when a step names it in "end".  A step in
which something is wanted writes OUT/<step>.f32 - little-endian fp32 rows [wanted, vocab] in the
order of the entries and their "want" - and every step prints "done <step>".
"""
from __future__ import annotations

import argparse
import json
import os
import sys

SLOTS = 4  # live requests at any time


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__,
                                 formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder of the logits files")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="tokens the live requests hold together at most, each rounded up to 64")
    args = ap.parse_args(argv)

    import torch

    if not torch.cuda.is_available():
        print("trace_run needs a GPU", file=sys.stderr)
        return 2
    from .. import _build
    from ..ops._ext import hipk
    from .block_allocator import native_missing

    if native_missing():
        _build.build_native()
    hipk()  # builds the kernel library if it is not there

    from ..models import load_model
    from ..ops import KV_BLOCK
    from .engine import LLMEngine
    from .request import Request

    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    n = -(-args.max_tokens // 64) * 64
    model = load_model(args.model, "cuda:0", dtype=getattr(torch, args.dtype), max_position=n)
    eng = LLMEngine(model, max_batch=SLOTS, max_model_len=n,
                    num_blocks=n // KV_BLOCK + 1)  # + the padding block
    live: dict[str, Request] = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = []
        for e in step["entries"]:
            r = live.get(e["id"])
            if r is None:
                r = live[e["id"]] = Request([], request_id=e["id"])
            entries.append((r, e["tokens"], e["want"]))
        rows = eng.feed(entries) if entries else []
        if any(e["want"] for e in step["entries"]):
            out = torch.cat([t.float() for t in rows]).cpu().contiguous()
            path = os.path.join(args.out, f"{step['step']}.f32")
            with open(path, "wb") as f:
                f.write(out.numpy().astype("<f4").tobytes())
        eng.check_health()
        for i in step.get("end", []):
            eng.release(live.pop(i))
        print(f"done {step['step']}", flush=True)
    eng.shutdown()
    return 0


if __name__ == "__main__":
    sys.exit(main())
