"""Prefill and decode throughput of the Lifuzen stack beside the Pupopel and talker stacks of equal size (random weights).

    python bench.py --lifuzen [--lifuzen-size 2k,4k] [--lifuzen-mode decode,prefill] [--steps K --warmup W]

One JSON line per (model, size, mode).  Equal size: the same width, layer runs, attention heads of the same dimension, (active)
feed-forward width, vocabulary, batch and context; a state-space layer's state is as large as a delta layer's.  Lifuzen: six layers,
the middle two looped twice (eight runs); half of the runs are state-space layers, half attention; every feed-forward is routed
(64 experts, 8 chosen).
"""
import json

import torch

from bench_dogulorn import DIM, LAYERS, SIZES, VOCAB, decode, dogulorn_config, prefill, talker_config
from bench_pupopel import pupopel_config


def lifuzen_config(s):
    from vllm_omni_amd.registry import config_from_hf

    h = s["heads"]
    ssm = {"type": "mamba2", "mixer": {"heads": 2 * h, "groups": 8, "state": 128, "vdim": 64, "conv": 4, "norm_groups": 8}}
    attn = {"type": "attention", "mixer": {"heads": h, "kv_heads": h // 4, "dim": DIM, "vdim": DIM, "conv": 4, "scale": DIM ** -0.5,
                                           "rot": {"base": 500000.0, "dims": DIM // 2}}}
    moe = {"kind": "moe", "router": {"experts": 64, "top": 8}, "expert": {"ff": s["ff"] // 8}}
    cfg = config_from_hf({"architecture": "Lifuzen", "vocab": VOCAB, "width": s["width"], "norm": {"eps": 1e-6}, "residual_mult": 0.5,
                          "logit_softcap": 25.0, "layers": [dict(m, mlp=moe) for m in (ssm, attn) * 3],
                          "loop": {"start": 2, "stop": 4, "times": 2}})
    assert len(cfg.runs) == LAYERS
    return cfg


CONFIGS = {"lifuzen": lifuzen_config, "pupopel": pupopel_config, "dogulorn": dogulorn_config, "talker": talker_config}


def run(a):
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    for size in a.lifuzen_size.split(","):
        for mode in a.lifuzen_mode.split(","):
            cases = ([(int(b), a.lifuzen_ctx) for b in a.lifuzen_batches.split(",")] if mode == "decode" else
                     [[int(n) for n in c.split(",")] for c in a.lifuzen_prompts.split(";")])
            for case in cases:
                for name in a.lifuzen_models.split(","):
                    cfg = CONFIGS[name](SIZES[size])
                    with torch.inference_mode():
                        if mode == "decode":
                            res = decode(name, cfg, dev, case[0], case[1], a.steps, a.warmup)
                            extra = {"batch": case[0], "ctx": case[1]}
                        else:
                            res = prefill(name, cfg, dev, case, max(2, a.steps // 6), 2)
                            extra = {"prompts": case}
                    print(json.dumps({"metric": f"{mode} tokens/s", "unit": "tokens/s", "model": name, "size": size, "layer_runs": LAYERS,
                                      "dtype": "bf16", "data": "synthetic", **extra, **res}), flush=True)
                    torch.cuda.empty_cache()
