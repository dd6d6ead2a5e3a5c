"""Prefill and decode throughput of the Dogulorn stack beside the talker stack of equal size (random weights).

    python bench.py --dogulorn [--dogulorn-size 2k,4k] [--dogulorn-mode decode,prefill] [--steps K --warmup W]

One JSON line per (model, size, mode).  Equal size: the same width, depth, heads of the same dimension, feed-forward width,
vocabulary, batch and context; the talker attends to the whole context, Dogulorn's attention layers to their window.
"""
import json
import time

import torch

SIZES = {   # width, ff, heads, delta q/k heads, q_rank, kv_rank, window, side
    "2k": dict(width=2048, ff=6144, heads=16, kvh=8, q_rank=768, kv_rank=256, window=1024, side=128),
    "4k": dict(width=4096, ff=12288, heads=32, kvh=16, q_rank=1536, kv_rank=512, window=1024, side=256),
}
LAYERS, VOCAB, DIM = 8, 15360, 128


def dogulorn_config(s):
    from vllm_omni_amd.registry import config_from_hf

    attn = {"heads": s["heads"], "dim": DIM, "vdim": DIM, "q_rank": s["q_rank"], "kv_rank": s["kv_rank"], "scale": DIM ** -0.5,
            "mask": {"size": s["window"]}}
    layers = []
    for i in range(LAYERS):
        if i % 4 < 2:
            layer = {"type": "delta", "mixer": {"heads": s["heads"], "kv_heads": s["kvh"], "dim": DIM, "vdim": DIM, "conv": 4}}
        else:
            layer = {"type": "latent_attention", "mixer": dict(attn, **({"kv_from": i - 1} if i % 4 == 3 else {}))}
        layers.append(dict(layer, mlp={"kind": "dense", "ff": s["ff"], "limit": 7.0}))
    return config_from_hf({"architecture": "Dogulorn", "vocab": VOCAB, "width": s["width"], "norm": {"eps": 1e-6},
                           "embedding": {"scale": 1.0, "bigram": {"buckets": 65536, "mul_prev": 31, "mul_cur": 7}},
                           "token_side": {"dim": s["side"]}, "layers": layers})


def talker_config(s):
    from vllm_omni_amd.talker import TalkerConfig

    return TalkerConfig(name="talker-sized", hidden_size=s["width"], embedding_size=s["width"], num_hidden_layers=LAYERS,
                        num_attention_heads=s["heads"], num_key_value_heads=s["heads"] // 4, head_dim=DIM,
                        intermediate_size=s["ff"], vocab_size=VOCAB, input_projection=False, attention_bias=False,
                        tts_codec_start_token_id=None, tts_codec_end_token_id=None)


def make_runner(cfg, dev, batch, ctx, tokens, eager=False):
    from vllm_omni_amd.model_runner import GPUARModelRunner

    r = GPUARModelRunner(cfg, dev, torch.bfloat16, max_num_reqs=batch, max_model_len=ctx + 16, max_num_batched_tokens=max(tokens, batch),
                         block_size=16, seed=0, engine_output_type="text", copy_outputs=False, enforce_eager=eager)
    r.load_model()
    return r


def fill(runner):
    g = torch.Generator(device=runner.device).manual_seed(1)
    for kv in runner.kv_caches:
        for t in ([kv] if isinstance(kv, torch.Tensor) else kv):
            t.normal_(0.0, 1.0, generator=g)


def decode(name, cfg, dev, batch, ctx, steps, warmup):
    import bench

    r = make_runner(cfg, dev, batch, ctx, batch)
    sched = bench.SyntheticScheduler(batch, ctx, 16, VOCAB, 0)
    r.initialize_kv_cache(sched.num_blocks)
    fill(r)

    def run(k):
        pend = None
        for _ in range(k):
            r.execute_model(sched.schedule())
            out = r.sample_tokens(async_output=True)
            if pend is not None:
                pend.get_output()
            pend = out
        if pend is not None:
            pend.get_output()

    run(warmup)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    run(steps)
    torch.cuda.synchronize()
    ms = (time.perf_counter() - t0) / steps * 1e3
    return {"ms_per_step": round(ms, 3), "value": round(batch / ms * 1e3, 1), "weight_gb": round(r.model.weight_bytes() / 1e9, 3)}


def prefill(name, cfg, dev, lens, steps, warmup):
    from vllm_omni_amd.kv_cache import KVCacheManager
    from vllm_omni_amd.sched_output import NewRequestData, Request, SamplingParams, SchedulerOutput

    total = sum(lens)
    r = make_runner(cfg, dev, len(lens), max(lens), total, eager=True)
    nb = sum(-(-n // 16) for n in lens) + 1
    r.initialize_kv_cache(nb)
    g = torch.Generator().manual_seed(0)
    prompts = [torch.randint(0, VOCAB, (n,), generator=g).tolist() for n in lens]
    prev = set()

    def once(tag):
        nonlocal prev
        mgr = KVCacheManager(nb, 16)
        new = []
        for i, p in enumerate(prompts):
            q = Request(f"{tag}-{i}", p, SamplingParams())
            assert mgr.allocate_slots(q, len(p)) is not None
            new.append(NewRequestData(q.request_id, p, q.sampling_params, mgr.get_block_ids(q.request_id), 0))
        r.execute_model(SchedulerOutput(scheduled_new_reqs=new, num_scheduled_tokens={x.req_id: len(p) for x, p in zip(new, prompts)},
                                        total_num_scheduled_tokens=total, finished_req_ids=prev))
        r.sample_tokens()
        prev = {x.req_id for x in new}

    for i in range(warmup):
        once(f"w{i}")
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for i in range(steps):
        once(f"s{i}")
    torch.cuda.synchronize()
    ms = (time.perf_counter() - t0) / steps * 1e3
    return {"ms_per_step": round(ms, 3), "value": round(total / ms * 1e3, 1)}


def run(a):
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    for size in a.dogulorn_size.split(","):
        s = SIZES[size]
        for mode in a.dogulorn_mode.split(","):
            for name in a.dogulorn_models.split(","):
                cfg = (dogulorn_config if name == "dogulorn" else talker_config)(s)
                cases = ([(int(b), a.dogulorn_ctx) for b in a.dogulorn_batches.split(",")] if mode == "decode" else
                         [[int(n) for n in c.split(",")] for c in a.dogulorn_prompts.split(";")])
                for case in cases:
                    with torch.inference_mode():
                        if mode == "decode":
                            res = decode(name, cfg, dev, case[0], case[1], a.steps, a.warmup)
                            extra = {"batch": case[0], "ctx": case[1]}
                        else:
                            res = prefill(name, cfg, dev, case, max(2, a.steps // 6), 2)
                            extra = {"prompts": case}
                    print(json.dumps({"metric": f"{mode} tokens/s", "unit": "tokens/s", "model": name, "size": size, "layers": LAYERS,
                                      "dtype": "bf16", "data": "synthetic", **extra, **res}), flush=True)
                    torch.cuda.empty_cache()
