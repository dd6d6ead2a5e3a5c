"""Command line: ``python -m vllm_omni_amd generate|trace ...``"""
from __future__ import annotations

import argparse
import json
import sys


def _generate(argv) -> int:
    ap = argparse.ArgumentParser(prog="vllm_omni_amd generate", description="generate from token-id prompts")
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--prompt", action="append", required=True, help="comma-separated token ids; may be repeated")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--max-tokens", type=int, default=16)
    ap.add_argument("--temperature", type=float, default=0.0)
    ap.add_argument("--top-k", type=int, default=0)
    ap.add_argument("--top-p", type=float, default=1.0)
    ap.add_argument("--seed", type=int, default=None)
    ap.add_argument("--eos", type=int, default=None, help="token id that ends a request")
    ap.add_argument("--max-model-len", type=int, default=4096)
    ap.add_argument("--max-num-seqs", type=int, default=64)
    ap.add_argument("--max-num-batched-tokens", type=int, default=8192)
    ap.add_argument("--block-size", type=int, default=16)
    ap.add_argument("--enforce-eager", action="store_true")
    a = ap.parse_args(argv)

    from .engine import LLMEngine
    from .sched_output import SamplingParams

    eng = LLMEngine(a.model, dtype=a.dtype, max_num_seqs=a.max_num_seqs, max_model_len=a.max_model_len,
                    max_num_batched_tokens=a.max_num_batched_tokens, block_size=a.block_size, enforce_eager=a.enforce_eager)
    prompts = [[int(t) for t in p.split(",") if t.strip()] for p in a.prompt]
    params = SamplingParams(temperature=a.temperature, top_k=a.top_k, top_p=a.top_p, max_tokens=a.max_tokens, seed=a.seed)
    for p, toks in zip(prompts, eng.generate(prompts, params, a.eos)):
        print(json.dumps({"prompt": p, "tokens": toks}), flush=True)
    return 0


def main(argv=None) -> int:
    argv = sys.argv[1:] if argv is None else argv
    if argv and argv[0] == "generate":
        return _generate(argv[1:])
    if argv and argv[0] == "trace":
        from .trace import main as trace

        return trace(argv[1:])
    print("usage: python -m vllm_omni_amd {generate,trace} --help", file=sys.stderr)
    return 2


if __name__ == "__main__":
    sys.exit(main())
