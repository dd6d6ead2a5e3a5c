"""Prefill and decode throughput of the Bodopel stack beside the talker and Pupopel stacks of equal size (random weights).

    python bench.py --bodopel [--bodopel-size 2k,4k] [--bodopel-mode decode,prefill] [--steps K --warmup W]

One JSON line per (model, size, mode).  Equal size: the same width, layer runs, heads of the same dimension, feed-forward width,
vocabulary, batch and context.  Bodopel: six layers, the middle two looped twice (eight runs), a window of 4096 tokens.
"""
import json

import torch

from bench_dogulorn import DIM, LAYERS, SIZES, VOCAB, decode, prefill, talker_config
from bench_pupopel import pupopel_config


def bodopel_config(s):
    from vllm_omni_amd.registry import config_from_hf

    layer = {"type": "attention", "mixer": {"heads": s["heads"], "kv_heads": s["heads"] // 4, "dim": DIM, "vdim": DIM, "scale": DIM ** -0.5,
                                            "softcap": 50.0, "mask": {"size": 4096}}, "mlp": {"kind": "dense", "ff": s["ff"]}}
    cfg = config_from_hf({"architecture": "Bodopel", "vocab": VOCAB, "width": s["width"], "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
                          "canon": {"taps": 4}, "max_positions": 16384, "layers": [layer] * 6, "loop": {"start": 2, "stop": 4, "times": 2}})
    assert len(cfg.runs) == LAYERS
    return cfg


CONFIGS = {"bodopel": bodopel_config, "pupopel": pupopel_config, "talker": talker_config}


def run(a):
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    for size in a.bodopel_size.split(","):
        for mode in a.bodopel_mode.split(","):
            cases = ([(int(b), a.bodopel_ctx) for b in a.bodopel_batches.split(",")] if mode == "decode" else
                     [[int(n) for n in c.split(",")] for c in a.bodopel_prompts.split(";")])
            for case in cases:
                for name in a.bodopel_models.split(","):
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
