"""Generate from a model folder (config.json + *.safetensors).

    python -m neuronx_distributed_amd.scripts.generate --model DIR \\
        --prompt 5,17,3 --prompt 9,9 --max-new-tokens 16

Prompts are token ids; one JSON line per prompt is printed.  The model class
is chosen by config.json.  On a GPU, models of the serving engine run all
prompts in one continuous batch; otherwise prompts are generated one by one.
"""

import argparse
import json
import sys


def main(argv=None):
    p = argparse.ArgumentParser(prog="nxd_generate")
    p.add_argument("--model", required=True)
    p.add_argument("--prompt", action="append", required=True,
                   help="comma-separated token ids (repeat for more prompts)")
    p.add_argument("--max-new-tokens", type=int, default=32)
    p.add_argument("--dtype", choices=("bfloat16", "float32"),
                   default="bfloat16")
    p.add_argument("--eos", type=int, default=-1)
    p.add_argument("--top-k", type=int, default=0, help="0 = greedy")
    p.add_argument("--temperature", type=float, default=1.0)
    p.add_argument("--max-seqs", type=int, default=None)
    p.add_argument("--max-step-tokens", type=int, default=2048)
    a = p.parse_args(argv)
    prompts = [[int(t) for t in s.split(",") if t.strip()] for s in a.prompt]

    import torch

    from ..inference.generation import generate
    from ..inference.parallel_context import single_process_groups
    from ..inference.scheduler import generate_ragged
    from ..models.registry import load_pretrained
    from ..utils.sampling import Sampler

    device = "cuda" if torch.cuda.is_available() else "cpu"
    single_process_groups()
    model = load_pretrained(a.model, getattr(torch, a.dtype), device)
    sampler = Sampler(do_sample=a.top_k > 0, top_k=a.top_k or 50,
                      temperature=a.temperature)
    if device == "cuda" and hasattr(model, "forward_ragged"):
        outs = generate_ragged(model, prompts, a.max_new_tokens, sampler,
                               a.eos, a.max_seqs, a.max_step_tokens)
    else:
        outs = [generate(model, torch.tensor([q], device=device),
                         a.max_new_tokens, sampler,
                         a.eos)[0, len(q):].tolist() for q in prompts]
    for q, o in zip(prompts, outs):
        print(json.dumps({"prompt": q, "output": o}), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
