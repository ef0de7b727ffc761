"""Replay of a token trace through a model: given token ids in, logits out, step by step, nothing sampled.

Every step is read as one JSON line {"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]} and runs as one portion
of its request, continuing from the cache (HipModel.forward_tokens: a prefill, or for a single token the decode step that
generation replays).  The logits of the wanted tokens go to <out>/<step>.f32, little-endian float32 [wanted, vocab]."""
from __future__ import annotations

import argparse
import json
import os
import sys

PAGE = 64   # positions per cache page


def replay(model, embedding, lines, out_dir: str, report) -> None:
    """Requests come one after the other and take the model's sequence slot in turn; their pages go back at their end."""
    import numpy as np
    live: dict[str, int] = {}   # request -> tokens so far
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = []
        for entry in step["entries"]:
            rid = entry["id"]
            if rid not in live and len(live) >= model.batch:
                raise RuntimeError(f"request {rid} starts while {sorted(live)} holds the only sequence slot")
            pos = live.setdefault(rid, 0)
            if entry["tokens"]:
                logits = model.forward_tokens(embedding, entry["tokens"], pos, want=entry.get("want", []))
                live[rid] = pos + len(entry["tokens"])
                if len(logits):
                    rows.append(logits)
        if rows:
            with open(os.path.join(out_dir, f"{step['step']}.f32"), "wb") as f:
                f.write(np.concatenate(rows).astype("<f4").tobytes())
        for rid in step.get("end", []):
            if live.pop(rid, None) is not None:
                model.kv_release(0)
        report(f"done {step['step']}")


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors (or a GGUF file)")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens live requests hold at any time")
    a = ap.parse_args(argv)
    import oxibonsai_amd as ox
    from .model import KV_F16, HipModel
    pages = (max(a.max_tokens, 1) + PAGE - 1) // PAGE
    model, embedding, _ = HipModel.from_checkpoint(ox.NativeHipBackend(0), a.model, a.dtype, max_seq=pages * PAGE)
    model.set_attention(KV_F16, page_size=PAGE, n_pages=pages)
    replay(model, embedding, sys.stdin, a.out, lambda text: print(text, flush=True))
    embedding.close()
    model.close()
    return 0
