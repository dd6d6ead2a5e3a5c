"""``trace_run``: drive a model with tokens chosen by the caller instead of sampled ones, and write the logits it gives.

The input has a line of JSON per step, for instance::

    {"step": 3, "entries": [{"id": "req7", "tokens": [40, 8, 2], "want": [2]}], "end": ["req5"]}

The entries form one batch: each appends its tokens to its request (a new id starts one).  ``want`` lists places among the
entry's own tokens; their logits go to ``OUT/<step>.f32`` as little-endian fp32 rows, entry after entry.  ``end`` finishes
requests, whose blocks and state slots become free.  ``done <step>`` follows on standard output.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

LIVE_REQUESTS = 4      # state slots of a replay


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a trace of token ids and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="most tokens live requests hold at any time, each request rounded up to a multiple of 64")
    ap.add_argument("--enforce-eager", action="store_true", help="no graph replay of decode steps")
    a = ap.parse_args(argv)

    import torch

    from .engine import LLMEngine

    torch.backends.cuda.matmul.allow_tf32 = False
    block = 16
    tokens = max(a.max_tokens, 1)
    eng = LLMEngine(a.model, dtype=a.dtype, max_num_seqs=LIVE_REQUESTS, max_model_len=tokens, max_num_batched_tokens=tokens,
                    block_size=block, num_blocks=-(-tokens // block), enforce_eager=a.enforce_eager)
    os.makedirs(a.out, exist_ok=True)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        portions = {e["id"]: e["tokens"] for e in s["entries"]}
        wanted = {e["id"]: e.get("want") or [] for e in s["entries"]}
        logits = eng.run_portions(portions, wanted, s.get("end") or [])
        if logits is not None:
            path = os.path.join(a.out, f"{s['step']}.f32")
            with open(path + ".part", "wb") as f:
                f.write(logits.cpu().numpy().astype("<f4").tobytes())
            os.replace(path + ".part", path)
        print(f"done {s['step']}", flush=True)
    torch.cuda.synchronize()
    return 0
