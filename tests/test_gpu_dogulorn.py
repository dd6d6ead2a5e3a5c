"""Dogulorn behind the engine: logits against the plain forward for whole prompts, portions, decoding, mixed batches and
re-used pages and slots; graph replay against eager; greedy generation through the scheduler."""
import json

import pytest
import torch

import dogulorn_models as dm
from oracle import ref_dogulorn as ref

pytestmark = pytest.mark.gpu


def engine(cfg, weights, dtype, tokens=1024, seqs=4, **kw):
    from vllm_omni_amd.engine import LLMEngine
    from vllm_omni_amd.registry import config_from_hf

    kw = {"num_blocks": -(-tokens // 16), "max_model_len": tokens, "max_num_batched_tokens": tokens, **kw}
    return LLMEngine(config_from_hf(cfg), dtype=dtype, max_num_seqs=seqs, weights=weights, **kw)


def check(got, want, limit, what=None):
    e = dm.row_error(got, want)
    assert (e <= limit).all(), (what, int((e / limit).argmax()), float((e / limit).max()))


_REF = {}


def expected(name, tokens, dtype=torch.float32):
    """weights, logits and streams of the plain forward, and per logits row and per stream row the limit of ``dtype``: what
    rounding alone does to that row, with room (kept between tests)"""
    cfg = dm.CONFIGS[name]
    w = _REF.setdefault((name, "w"), dm.random_weights(cfg, seed=7))
    key = (name, tuple(tokens))
    if key not in _REF:
        lg, st = ref.forward(cfg, w, tokens)
        with dm.Bf16Products():
            lg2, st2 = ref.forward(cfg, w, tokens)
        _REF[key] = lg, st, 0.04 + 3 * dm.row_error(lg2, lg), [0.04 + 3 * dm.row_error(b, a) for a, b in zip(st, st2)]
    lg, st, lim, lims = _REF[key]
    if dtype == torch.float32:
        lim, lims = torch.full_like(lim, 3e-5), [torch.full_like(x, 3e-5) for x in lims]
    return w, lg, st, lim, lims


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", list(dm.CONFIGS))
def test_every_layer_of_a_prompt(dev, name, dtype):
    cfg = dm.CONFIGS[name]
    toks = dm.random_tokens(cfg, 150, 1)
    w, logits, streams, lim, lims = expected(name, toks, dtype)
    e = engine(cfg, w, dtype)
    e.model.residual_tap = []
    got = e.run_portions({"a": toks}, {"a": list(range(150))}, ["a"])
    for i, (x, s) in enumerate(zip(e.model.residual_tap, streams)):
        assert x.dtype == torch.float32
        check(x, s, lims[i], f"layer {i}")
    check(got, logits, lim)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", list(dm.CONFIGS))
def test_portions_and_decoding(dev, name, dtype):
    """one engine, one request after the other (pages and slots are used again): token by token from the first token on,
    portions of changing size, most of the prompt and then single tokens"""
    cfg = dm.CONFIGS[name]
    toks = dm.random_tokens(cfg, 150, 1)
    w, logits, _, lim, _ = expected(name, toks, dtype)
    e = engine(cfg, w, dtype, tokens=160, seqs=1)
    plans = {"tokens": [1] * 40, "pairs": [2] * 30 + [1, 2, 3], "uneven": [7, 64, 1, 1, 33, 2, 5, 37], "tail": [100] + [1] * 50,
             "blocks": [16, 48, 17, 15, 54]}
    for kind, sizes in plans.items():
        at = 0
        for k in sizes:
            end = at + k
            got = e.run_portions({kind: toks[at:end]}, {kind: list(range(k))}, [kind] if end == sum(sizes) else [])
            check(got, logits[at:end], lim[at:end], (kind, at))
            at = end
        assert e.scheduler.kv_cache_manager.block_pool.get_num_free_blocks() == 10


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_mixed_batches_pages_and_slots_used_again(dev, dtype):
    name = "mixed"
    cfg = dm.CONFIGS[name]
    seqs = {f"r{i}": dm.random_tokens(cfg, n, 20 + i) for i, n in enumerate([90, 33, 1, 64, 17, 120, 2, 48])}
    w = expected(name, seqs["r0"])[0]
    want = {r: expected(name, t, dtype) for r, t in seqs.items()}
    e = engine(cfg, w, dtype, tokens=400)
    g = torch.Generator().manual_seed(3)
    at, waiting, live = dict.fromkeys(seqs, 0), list(seqs), []
    for _ in range(400):
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
        if not live:
            break
        step, places, done = {}, {}, []
        for r in live:
            if len(live) > 1 and torch.rand(1, generator=g).item() < 0.2:      # left out of this step
                continue
            k = [1, 1, 2, 5, 31][int(torch.randint(5, (1,), generator=g))]
            k = min(k, len(seqs[r]) - at[r])
            step[r], places[r] = seqs[r][at[r]:at[r] + k], list(range(k))
        if not step:
            continue
        for r in step:
            if at[r] + len(step[r]) == len(seqs[r]):
                done.append(r)
        got = e.run_portions(step, places, done)
        lo = 0
        for r, t in step.items():
            check(got[lo:lo + len(t)], want[r][1][at[r]:at[r] + len(t)], want[r][3][at[r]:at[r] + len(t)], (r, at[r]))
            lo += len(t)
            at[r] += len(t)
        live = [r for r in live if r not in done]
    assert not waiting and not live
    e.step()
    assert e.runner.state_cache.num_free == 4 and not e.runner.requests


def test_far_tokens_show_through_the_recurrence(dev):
    """one early token changed: everything after it must move as the plain forward says (state carried over pages, chunks
    and decoding)"""
    cfg = dm.CONFIGS["mixed"]
    a = dm.random_tokens(cfg, 300, 5)
    b = list(a)
    b[3] = (b[3] + 1) % cfg["vocab"]
    w = dm.random_weights(cfg, seed=7)
    for k in w:
        if k.endswith("A_log"):
            w[k] = w[k] - 5.0          # a state that hardly decays
    e = engine(cfg, w, torch.float32, tokens=640)
    for r, t in (("a", a), ("b", b)):
        e.run_portions({r: t[:200]})
    got = torch.cat([e.run_portions({"a": a[i:i + 1], "b": b[i:i + 1]}, {"a": [0], "b": [0]}) for i in range(200, 300)])
    want_a, want_b = (ref.forward(cfg, w, t)[0][200:] for t in (a, b))
    assert dm.row_error(want_b, want_a).median() > 1e-3          # the change is there after 300 tokens, far above rounding
    check(got[0::2], want_a, 5e-5)
    check(got[1::2], want_b, 5e-5)


def greedy_reference(cfg, w, prompt, n, got):
    """the plain forward on prompt + got: greedy token wherever the top two are apart"""
    lg = ref.forward(cfg, w, list(prompt) + got[:-1], torch.float64)[0][len(prompt) - 1:]
    top = lg.topk(2, -1)
    sure = (top.values[:, 0] - top.values[:, 1]) > 0.15 * lg.std()
    assert sure.sum() >= 0.3 * n
    for i in range(n):
        if sure[i]:
            assert got[i] == int(top.indices[i, 0]), i


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_greedy_generation_through_the_scheduler(dev, dtype):
    from vllm_omni_amd.sched_output import SamplingParams

    cfg = dm.CONFIGS["wide"]
    w = dm.random_weights(cfg, seed=7)
    prompts = [dm.random_tokens(cfg, n, 60 + i) for i, n in enumerate([1, 40, 97, 5, 64, 3])]
    e = engine(cfg, w, dtype, tokens=256, max_num_batched_tokens=48, num_blocks=64)     # chunked prefill beside decoding
    out = e.generate(prompts, SamplingParams(max_tokens=24, ignore_eos=True))
    for p, o in zip(prompts, out):
        assert len(o) == 24
        greedy_reference(cfg, w, p, 24, o)
    assert e.runner.state_cache.num_free == 4
    again = e.generate(prompts[:3], SamplingParams(max_tokens=24, ignore_eos=True))
    for p, o in zip(prompts, again):
        greedy_reference(cfg, w, p, 24, o)


def test_preempted_requests_recompute_their_state(dev):
    """a pool too small for all: the newest request loses its blocks and its state slot, and starts over from its tokens"""
    from vllm_omni_amd.sched_output import SamplingParams

    cfg = dm.CONFIGS["mixed"]
    w = dm.random_weights(cfg, seed=7)
    prompts = [dm.random_tokens(cfg, 30, 80 + i) for i in range(4)]
    params = SamplingParams(max_tokens=40, ignore_eos=True)
    roomy = engine(cfg, w, torch.float32, tokens=512).generate(prompts, params)
    e = engine(cfg, w, torch.float32, tokens=128, num_blocks=12)
    preempted = []
    orig = e.scheduler._preempt
    e.scheduler._preempt = lambda r: (preempted.append(r.request_id), orig(r))[1]
    tight = e.generate(prompts, params)
    assert preempted and e.runner.state_cache.num_free == 4
    for p, a, b in zip(prompts, roomy, tight):
        greedy_reference(cfg, w, p, 40, a)
        greedy_reference(cfg, w, p, 40, b)


def test_sampled_generation_is_reproducible(dev):
    from vllm_omni_amd.sched_output import SamplingParams

    cfg = dm.CONFIGS["mixed"]
    w = dm.random_weights(cfg, seed=7)
    prompts = [dm.random_tokens(cfg, 9, 3), dm.random_tokens(cfg, 20, 4)]
    p = SamplingParams(temperature=0.8, top_k=20, top_p=0.9, seed=5, max_tokens=16, ignore_eos=True)
    e = engine(cfg, w, torch.float32, tokens=256)
    a, b = e.generate(prompts, p), e.generate(prompts, p)
    assert a == b and all(0 <= t < cfg["vocab"] for o in a for t in o)


@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_graph_replay_equals_eager(dev, name):
    """decode steps replayed from graphs, with other eager work between replays, against an engine that never captures"""
    cfg = dm.CONFIGS[name]
    w = dm.random_weights(cfg, seed=7)
    toks = {f"r{i}": dm.random_tokens(cfg, 60, 40 + i) for i in range(3)}
    g, x = engine(cfg, w, torch.bfloat16), engine(cfg, w, torch.bfloat16, enforce_eager=True)
    for e in (g, x):
        e.run_portions({r: t[:30 + 5 * i] for i, (r, t) in enumerate(toks.items())})
    at = {r: 30 + 5 * i for i, r in enumerate(toks)}
    for step in range(15):
        names = list(toks) if step % 4 else list(toks)[:2]
        part = {r: [toks[r][at[r]]] for r in names}
        a, b = (e.run_portions(part, {r: [0] for r in names}) for e in (g, x))
        assert torch.equal(a, b), step
        for r in names:
            at[r] += 1
        torch.cuda.synchronize()
        torch.randn(64, 64, device=dev).sum()
    assert g.runner._graphs and not x.runner._graphs


def test_checkpoint_folder_to_trace_and_command_line(dev, tmp_path, capsys, monkeypatch):
    """config.json + safetensors -> trace replay and the generate command"""
    import io

    from safetensors.torch import save_file

    from vllm_omni_amd import trace
    from vllm_omni_amd.__main__ import main as cli

    cfg = dm.CONFIGS["odd"]
    w = dm.random_weights(cfg, seed=7)
    (tmp_path / "m").mkdir()
    (tmp_path / "m" / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "m" / "model.safetensors"))
    toks = dm.random_tokens(cfg, 70, 2)
    lg = ref.forward(cfg, w, toks, torch.float64)[0]
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:40], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": toks[40:41], "want": [0]}, {"id": "b", "tokens": toks[:9], "want": [8, 2]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": toks[41:], "want": [28]}], "end": ["a"]}]
    with dm.Bf16Products():
        rounded = ref.forward(cfg, w, toks)[0]
    lim16 = 0.04 + 3 * dm.row_error(rounded, lg)
    for dtype, lim in (("float32", torch.full_like(lim16, 3e-5)), ("bfloat16", lim16)):
        out = tmp_path / dtype
        monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
        assert trace.main(["--model", str(tmp_path / "m"), "--dtype", dtype, "--out", str(out), "--max-tokens", "192"]) == 0
        assert [x for x in capsys.readouterr().out.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
        assert not (out / "0.f32").exists()
        got = [torch.frombuffer(bytearray((out / f"{i}.f32").read_bytes()), dtype=torch.float32).view(-1, cfg["vocab"]) for i in (1, 2)]
        for g, rows in zip(got, ([40, 8, 2], [69])):
            e = (g.double() - lg[rows]).pow(2).mean(-1).sqrt() / lg.std()
            assert (e <= lim[rows]).all()
    assert cli(["generate", "--model", str(tmp_path / "m"), "--prompt", ",".join(map(str, toks[:12])), "--max-tokens", "5",
                "--dtype", "float32", "--max-model-len", "128", "--max-num-seqs", "2"]) == 0
    line = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert line["prompt"] == toks[:12] and len(line["tokens"]) == 5
    greedy_reference(cfg, w, toks[:12], 5, line["tokens"])
