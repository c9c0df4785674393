"""Replay a trace of token ids through a model and write logits.

    trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 3], "want": [1]}],
     "end": []}

Each step is one batch of the serving engine.  The wanted logits go to
<out>/<step>.f32 (little-endian float32, [wanted, vocab]); ``done <step>``
is printed after every step.  Requests named in ``end`` give back their
pages and slots.
"""

import argparse
import json
import os
import sys

MAX_LIVE = 4
DTYPES = ("bfloat16", "float32")


def main(argv=None):
    p = argparse.ArgumentParser(prog="trace_run")
    p.add_argument("--model", required=True)
    p.add_argument("--dtype", choices=DTYPES, default="bfloat16")
    p.add_argument("--out", required=True)
    p.add_argument("--max-tokens", type=int, required=True)
    a = p.parse_args(argv)

    from ..ops.serving import ensure_built

    ensure_built()

    import numpy as np
    import torch

    from ..inference.engine import InferenceEngine, StepEntry
    from ..inference.parallel_context import single_process_groups
    from ..models.registry import load_pretrained

    torch.backends.cuda.matmul.allow_tf32 = False
    torch.cuda.set_device(0)
    single_process_groups()
    model = load_pretrained(a.model, getattr(torch, a.dtype), "cuda")
    engine = InferenceEngine(model, max_tokens=a.max_tokens,
                             max_seqs=MAX_LIVE)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = engine.step([StepEntry(e["id"], e["tokens"],
                                        e.get("want", []))
                              for e in s["entries"]])
        if logits is not None:
            logits.cpu().numpy().astype(np.dtype("<f4")).tofile(
                os.path.join(a.out, f"{s['step']}.f32"))
        for rid in s.get("end", []):
            engine.finish(rid)
        print(f"done {s['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
