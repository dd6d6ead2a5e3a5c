"""Prefill and decode throughput of the Pupopel stack beside the Dogulorn and talker stacks of equal size (random weights).

    python bench.py --pupopel [--pupopel-size 2k,4k] [--pupopel-mode decode,prefill] [--steps K --warmup W]

One JSON line per (model, size, mode).  Equal size: the same width, layer runs, heads of the same dimension, (active)
feed-forward width, vocabulary, batch and context.  Pupopel: six layers, the middle two looped twice (eight runs); half of the
runs are channel-wise delta layers, half attention (full, with bias and sink) beside decayed linear attention; half of the
feed-forwards are routed (64 experts, 6 chosen, a shared one).
"""
import json

import torch

from bench_dogulorn import DIM, LAYERS, SIZES, VOCAB, decode, dogulorn_config, prefill, talker_config


def pupopel_config(s):
    from vllm_omni_amd.registry import config_from_hf

    h, ff = s["heads"], s["ff"]
    delta = {"type": "channel_delta", "mixer": {"heads": h, "kv_heads": s["kvh"], "dim": DIM, "vdim": DIM, "conv": 4}}
    par = {"type": "parallel", "mixer": {
        "left": {"heads": h, "kv_heads": h // 4, "dim": DIM, "vdim": DIM, "scale": DIM ** -0.5, "q_temp": {"coef": 0.1, "every": 8192}},
        "right": {"heads": h // 2, "dim": DIM, "vdim": DIM, "decay": [1 - 2.0 ** -(3 + 5 * i / h) for i in range(h // 2)]},
        "left_scale": 0.8, "right_scale": 0.5}}
    dense = {"kind": "dense", "ff": ff}
    moe = {"kind": "moe", "router": {"experts": 64, "top": 6}, "expert": {"ff": ff // 8}, "shared": {"ff": ff // 4}}
    layers = [dict(m, mlp=f) for m, f in ((delta, dense), (par, dense), (delta, moe), (par, moe), (delta, dense), (par, dense))]
    cfg = config_from_hf({"architecture": "Pupopel", "vocab": VOCAB, "width": s["width"], "norm": {"eps": 1e-6}, "layers": layers,
                          "loop": {"start": 2, "stop": 4, "times": 2}})
    assert len(cfg.runs) == LAYERS
    return cfg


CONFIGS = {"pupopel": pupopel_config, "dogulorn": dogulorn_config, "talker": talker_config}


def run(a):
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    for size in a.pupopel_size.split(","):
        for mode in a.pupopel_mode.split(","):
            cases = ([(int(b), a.pupopel_ctx) for b in a.pupopel_batches.split(",")] if mode == "decode" else
                     [[int(n) for n in c.split(",")] for c in a.pupopel_prompts.split(";")])
            for case in cases:
                for name in a.pupopel_models.split(","):
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
