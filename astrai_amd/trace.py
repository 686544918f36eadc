"""Replay a recorded schedule of token portions through a model and write the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Standard input holds one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

Each entry's tokens follow what its request has been given so far; ``want`` are the places among them
whose logits are written, all of a step to ``<out>/<step>.f32`` (little-endian float32 rows, in the
order of the entries and of ``want``). ``done <step>`` on standard output ends a step; the requests
in ``end`` then give back what they hold. Nothing is sampled: the model's forward, the one
``greedy_generate`` steps, runs on the cache of each request.
"""

from __future__ import annotations

import argparse
import json
import os
import sys

import torch

from astrai_amd.model import RequestCaches, load_checkpoint

_DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


def replay(model, caches: RequestCaches, step: dict, out_dir: str) -> None:
    """Run one step and write its logits."""
    device = next(model.parameters()).device
    rows = []
    for entry in step["entries"]:
        ids = torch.tensor([entry["tokens"]], dtype=torch.long, device=device)
        if ids.size(1) == 0:
            continue
        cache = caches.of(entry["id"])
        want = torch.tensor(entry["want"], dtype=torch.long, device=device)
        logits = model(ids, cache, logits_at=want)["logits"]
        cache.advance(ids.size(1))
        rows.append(logits[0])
    # (the copy to the host also waits for the step)
    host = [r.float().cpu().numpy() for r in rows]
    if any(len(r) for r in host):
        path = os.path.join(out_dir, f"{step['step']}.f32")
        with open(path, "wb") as f:
            for r in host:
                f.write(r.astype("<f4").tobytes())
    for request in step["end"]:
        caches.end(request)


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=sorted(_DTYPES), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    args = ap.parse_args(argv)
    torch.backends.cuda.matmul.allow_tf32 = False
    with torch.no_grad():
        model = load_checkpoint(args.model, "cuda", _DTYPES[args.dtype])
        caches = RequestCaches(lambda: model.new_cache(1, max(args.max_tokens, 1)))
        for line in sys.stdin:
            if not line.strip():
                continue
            step = json.loads(line)
            replay(model, caches, step, args.out)
            print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
