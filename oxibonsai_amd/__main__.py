"""Command line: what a checkpoint holds, and generation from token ids.

    python -m oxibonsai_amd info PATH
    python -m oxibonsai_amd generate PATH --tokens 5,17,3 [--steps N] [--dtype ...] [--temperature T --top-k K --top-p P --seed S]

PATH is a GGUF file or a folder with config.json and model.safetensors.  (Text is tokenised elsewhere.)"""
from __future__ import annotations

import argparse
import json
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="python -m oxibonsai_amd", description=__doc__.split("\n")[0])
    sub = ap.add_subparsers(dest="command", required=True)
    info = sub.add_parser("info", help="architecture and sizes of a checkpoint (no GPU needed)")
    info.add_argument("path")
    gen = sub.add_parser("generate", help="continue a sequence of token ids; prints the new ids")
    gen.add_argument("path")
    gen.add_argument("--tokens", required=True, help="prompt token ids, separated by commas")
    gen.add_argument("--steps", type=int, default=32, help="tokens to generate")
    gen.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    gen.add_argument("--max-seq", type=int, default=0, help="context positions (default: prompt and steps)")
    gen.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    gen.add_argument("--top-k", type=int, default=40)
    gen.add_argument("--top-p", type=float, default=0.9)
    gen.add_argument("--seed", type=int, default=1)
    a = ap.parse_args(argv)
    from .model import HipModel, checkpoint_info
    if a.command == "info":
        print(json.dumps(checkpoint_info(a.path)))
        return 0
    from .backend import NativeHipBackend
    ids = [int(t) for t in a.tokens.split(",")]
    if a.steps < 1:
        ap.error("--steps must be positive")
    model, embedding, _ = HipModel.from_checkpoint(NativeHipBackend(0), a.path, a.dtype, max_seq=a.max_seq or len(ids) + a.steps)
    try:
        # the last prompt token is the first one of the loop, so that the sampler draws every new token
        if len(ids) > 1:
            model.forward_tokens(embedding, ids[:-1], 0, want=[])
        start = len(ids) - 1
        if a.temperature > 0:
            out, _ = model.generate_sampled(embedding, ids[-1], start, a.steps, a.temperature, a.top_k, a.top_p, a.seed)
        else:
            out = model.generate(embedding, ids[-1], start, a.steps)
        print(" ".join(str(int(t)) for t in out[:, 0]))
    finally:
        embedding.close()
        model.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
