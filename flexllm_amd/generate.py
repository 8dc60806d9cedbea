"""Command line: token ids in, token ids out.

    python -m flexllm_amd.generate --model DIR --prompt 1,2,3 --steps 32 [--top-k 5 --seed 0]

DIR is any folder that registry.load_model serves.  Prints the generated ids on one line."""
import argparse
import sys

import numpy as np


def main(argv=None):
    ap = argparse.ArgumentParser(prog="flexllm_amd.generate")
    ap.add_argument("--model", required=True, help="model folder")
    ap.add_argument("--prompt", required=True, help="token ids with commas between them")
    ap.add_argument("--steps", type=int, default=16)
    ap.add_argument("--dtype", default=None, help="bfloat16 or float32 where the model has both")
    ap.add_argument("--max-pos", type=int, default=4096, help="longest sequence")
    ap.add_argument("--top-k", type=int, default=0, help="0: greedy")
    ap.add_argument("--seed", type=int, default=0, help="of the sampler's uniform numbers")
    ap.add_argument("--w4a4", action="store_true", help="reference-format parameters: the W4A4 configuration")
    a = ap.parse_args(argv)
    from .registry import load_model
    prompt = [int(t) for t in a.prompt.replace(",", " ").split()]
    model = load_model(a.model, dtype=a.dtype, max_pos=a.max_pos, w4a4=a.w4a4)
    rands = np.random.default_rng(a.seed).random(max(a.steps, 1), np.float32) if a.top_k else None
    print(",".join(str(t) for t in model.generate(prompt, a.steps, top_k=a.top_k, rands=rands)))
    return 0


if __name__ == "__main__":
    sys.exit(main())
