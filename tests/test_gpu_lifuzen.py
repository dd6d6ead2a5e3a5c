"""Lifuzen behind the engine: logits against the plain forward for whole prompts, portions, decoding, mixed batches and
re-used pages and slots; graph replay against eager; greedy generation through the scheduler."""
import io
import json

import pytest
import torch

import lifuzen_models as lm
from oracle import ref_lifuzen as ref
from test_gpu_dogulorn import engine as _engine

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]


def engine(name, weights, dtype, tokens=512, seqs=4, **kw):
    return _engine(lm.CONFIGS[name] if isinstance(name, str) else name, weights, dtype, tokens, seqs, **kw)


_REF = {}


def weights(cfg, dtype, seed=7):
    """bf16 runs: routers without close calls; the 32-bit runs keep those that choose token by token"""
    w = lm.random_weights(cfg, seed)
    return lm.steady(w) if dtype == torch.bfloat16 else w


def plain(cfg, w, tokens, dtype):
    """logits, streams, and per row the limit of ``dtype``: what rounding alone does to that row, with room"""
    lg, st = ref.forward(cfg, w, tokens)
    if dtype == torch.float32:
        return lg, st, torch.full((len(tokens),), 5e-5), [torch.full((len(tokens),), 5e-5)] * len(st)
    with lm.Bf16Products():
        lg2, st2 = ref.forward(cfg, w, tokens)
    return lg, st, 0.04 + 3 * lm.row_error(lg2, lg), [0.04 + 3 * lm.row_error(b, a) for a, b in zip(st, st2)]


def expected(name, tokens, dtype=torch.float32):
    if (name, dtype) not in _REF:
        _REF[name, dtype] = weights(lm.CONFIGS[name], dtype)
    w = _REF[name, dtype]
    key = (name, dtype, tuple(tokens))
    if key not in _REF:
        _REF[key] = plain(lm.CONFIGS[name], w, tokens, dtype)
    return (w, *_REF[key])


def check(got, want, limit, what=None):
    e = lm.row_error(got, want)
    assert (e <= limit).all(), (what, int((e / limit).argmax()), float((e / limit).max()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(lm.CONFIGS))
def test_every_layer_run_of_a_prompt(dev, name, dtype):
    toks = lm.random_tokens(lm.CONFIGS[name], 150, 1)
    w, logits, streams, lim, lims = expected(name, toks, dtype)
    e = engine(name, w, dtype)
    e.model.residual_tap = []
    got = e.run_portions({"a": toks}, {"a": list(range(150))}, ["a"])
    assert len(e.model.residual_tap) == len(streams)
    for i, (x, s) in enumerate(zip(e.model.residual_tap, streams)):
        assert x.dtype == torch.float32
        check(x, s, lims[i], f"run {i}")
    check(got, logits, lim)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(lm.CONFIGS))
def test_portions_and_decoding(dev, name, dtype):
    """one engine, one request after the other (pages and slots are used again): token by token from the first token on,
    portions of changing size, most of the prompt and then single tokens"""
    toks = lm.random_tokens(lm.CONFIGS[name], 150, 1)
    w, logits, _, lim, _ = expected(name, toks, dtype)
    e = engine(name, w, dtype, tokens=160, seqs=1)
    plans = {"tokens": [1] * 40, "pairs": [2] * 30 + [1, 2, 3], "uneven": [7, 64, 1, 1, 33, 2, 5, 37], "tail": [100] + [1] * 50,
             "blocks": [16, 48, 17, 15, 54]}
    for kind, sizes in plans.items():
        at, rows = 0, []
        for k in sizes:
            end = at + k
            rows.append(e.run_portions({kind: toks[at:end]}, {kind: list(range(k))}, [kind] if end == sum(sizes) else []))
            at = end
        check(torch.cat(rows), logits[:at], lim[:at], kind)
        assert e.scheduler.kv_cache_manager.block_pool.get_num_free_blocks() == 10


@pytest.mark.parametrize("wait", [True, False])
@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_batches_pages_and_slots_used_again(dev, dtype, wait):
    """``wait`` False: nothing is read between the steps, so the host runs ahead of the device while requests come and go"""
    name = "mixed"
    cfg = lm.CONFIGS[name]
    seqs = {f"r{i}": lm.random_tokens(cfg, n, 20 + i) for i, n in enumerate([90, 33, 1, 64, 17, 120, 2, 48, 1, 75])}
    want = {r: expected(name, t, dtype) for r, t in seqs.items()}
    e = engine(name, want["r0"][0], dtype, tokens=400)
    g = torch.Generator().manual_seed(3)
    at, waiting, live, rows = dict.fromkeys(seqs, 0), list(seqs), [], {r: [] for r in seqs}
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
        if wait:
            got = got.cpu()
        lo = 0
        for r, t in step.items():
            rows[r].append(got[lo:lo + len(t)].clone())
            lo += len(t)
            at[r] += len(t)
        live = [r for r in live if r not in done]
    assert not waiting and not live
    for r in seqs:
        check(torch.cat(rows[r]), want[r][1], want[r][3], r)
    e.step()
    assert e.runner.state_cache.num_free == 4 and not e.runner.requests


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_first_tokens_and_one_far_back(dev, dtype):
    """one early token changed: the rows behind it move as the plain forward says, the rows in front of it not at all, in prompts
    and in decoding, at page and chunk borders"""
    cfg = lm.model([(lm.attn(6, 2, 48, 24, 4, 0.5), lm.moe(5, 2, 40)), (lm.mamba(4, 2, 40, 32, 4, 1), None)], (0, 2, 2))
    w = weights(cfg, dtype, 9)
    a = lm.random_tokens(cfg, 130, 5)
    e = engine(cfg, w, dtype, tokens=1024)

    def run(t, rid):
        got = [e.run_portions({rid: t[:70]}, {rid: list(range(70))})]
        return torch.cat(got + [e.run_portions({rid: t[i:i + 1]}, {rid: [0]}, [rid] if i == 129 else []) for i in range(70, 130)]).cpu()

    base = run(a, "base")
    for spot in (0, 1, 2, 3, 15, 16, 31, 63, 64, 80):
        b = list(a)
        b[spot] = (b[spot] + 1) % cfg["vocab"]
        lg, _, lim, _ = plain(cfg, w, b, dtype)
        got = run(b, f"s{spot}")
        check(got, lg, lim, spot)
        moved = lm.row_error(got, base.double())
        assert moved[spot] > 1e-3 and moved[spot + 1:spot + 8].min() > 1e-6, spot
        assert spot == 0 or moved[:spot].max() < (1e-6 if dtype == torch.float32 else 0.02), spot


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_key_that_stands_out_far_back(dev, dtype):
    """queries that find the earlier token of their own kind among hundreds, across pages and portions: the same projection for
    queries and keys, no rotation to speak of, and a large scale"""
    cfg = lm.model([(lm.attn(4, 2, 64, 4, 1, 1.0, 1e9), lm.moe(4, 2, 64)), (lm.attn(4, 4, 64, 2, 1, 0.7, 1e9), None)], (0, 2, 1))
    w = weights(cfg, dtype, 11)
    for i, g in ((0, 2), (1, 1)):
        for n in ("q", "k"):
            w[f"l{i}.mix.{n}.conv"] = torch.ones_like(w[f"l{i}.mix.{n}.conv"])
        k = w[f"l{i}.mix.k"].view(-1, 64, cfg["width"])
        k[:, :4] = 0            # what is rotated
        w[f"l{i}.mix.q"] = k.repeat_interleave(g, 0).reshape(-1, cfg["width"]).contiguous()
    n = 420
    toks = lm.random_tokens(cfg, n, 3)
    odd = cfg["vocab"] - 1
    toks = [0 if t == odd else t for t in toks]
    for i in (12, 200, 411):
        toks[i] = odd
    lg, _, lim, _ = plain(cfg, w, toks, dtype)
    e = engine(cfg, w, dtype, tokens=512)
    got = [e.run_portions({"a": toks[:130]}, {"a": list(range(130))}), e.run_portions({"a": toks[130:257]}, {"a": list(range(127))}),
           e.run_portions({"a": toks[257:400]}, {"a": list(range(143))})]
    got += [e.run_portions({"a": toks[i:i + 1]}, {"a": [0]}) for i in range(400, n)]
    check(torch.cat(got), lg, lim)


def greedy_reference(cfg, w, prompt, n, got):
    """the plain forward on prompt + got: greedy token wherever the top two are apart"""
    lg = ref.forward(cfg, w, list(prompt) + got[:-1], torch.float64)[0][len(prompt) - 1:]
    top = lg.topk(2, -1)
    sure = (top.values[:, 0] - top.values[:, 1]) > 0.1 * lg.std()
    assert sure.sum() >= 0.1 * n
    for i in range(n):
        if sure[i]:
            assert got[i] == int(top.indices[i, 0]), i


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_scheduler(dev, dtype):
    from vllm_omni_amd.sched_output import SamplingParams

    cfg = dict(lm.CONFIGS["mixed"], logit_softcap=40.0)        # far from the cap's flat ends: the top two are apart
    w = weights(cfg, dtype)
    prompts = [lm.random_tokens(cfg, n, 60 + i) for i, n in enumerate([1, 40, 97, 5, 64, 3])]
    e = engine(cfg, w, dtype, tokens=256, max_num_batched_tokens=48, num_blocks=64)     # chunked prefill beside decoding
    out = e.generate(prompts, SamplingParams(max_tokens=24, ignore_eos=True))
    for p, o in zip(prompts, out):
        assert len(o) == 24
        greedy_reference(cfg, w, p, 24, o)
    assert e.runner.state_cache.num_free == 4
    for p, o in zip(prompts, e.generate(prompts[:3], SamplingParams(max_tokens=24, ignore_eos=True))):
        greedy_reference(cfg, w, p, 24, o)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dev, dtype):
    from vllm_omni_amd.sched_output import SamplingParams

    cfg = dict(lm.CONFIGS["odd"], logit_softcap=40.0)
    w = weights(cfg, dtype)
    prompt = lm.random_tokens(cfg, 11, 1)
    out = engine(cfg, w, dtype, tokens=384).generate([prompt], SamplingParams(max_tokens=300, ignore_eos=True))[0]
    assert len(out) == 300
    greedy_reference(cfg, w, prompt, 300, out)


def test_preempted_requests_recompute_their_state(dev):
    """a pool too small for all: the newest request loses its blocks and its state slot, and starts over from its tokens"""
    from vllm_omni_amd.sched_output import SamplingParams

    cfg = dict(lm.CONFIGS["mixed"], logit_softcap=40.0)
    w = weights(cfg, torch.float32)
    prompts = [lm.random_tokens(cfg, 30, 80 + i) for i in range(4)]
    params = SamplingParams(max_tokens=40, ignore_eos=True)
    e = engine(cfg, w, torch.float32, tokens=128, num_blocks=12)
    preempted = []
    orig = e.scheduler._preempt
    e.scheduler._preempt = lambda r: (preempted.append(r.request_id), orig(r))[1]
    tight = e.generate(prompts, params)
    assert preempted and e.runner.state_cache.num_free == 4
    for p, b in zip(prompts, tight):
        greedy_reference(cfg, w, p, 40, b)


@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_graph_replay_equals_eager(dev, name):
    """decode steps replayed from graphs, with other eager work between replays, against an engine that never captures"""
    cfg = lm.CONFIGS[name]
    w = weights(cfg, torch.bfloat16)
    toks = {f"r{i}": lm.random_tokens(cfg, 60, 40 + i) for i in range(3)}
    g, x = engine(name, w, torch.bfloat16), engine(name, w, torch.bfloat16, enforce_eager=True)
    for e in (g, x):
        e.run_portions({r: t[:30 + 5 * i] for i, (r, t) in enumerate(toks.items())})
    at = {r: 30 + 5 * i for i, r in enumerate(toks)}
    for step in range(15):
        names = list(toks) if step % 4 else list(toks)[:2]
        part = {r: [toks[r][at[r]]] for r in names}
        a, b = (e.run_portions(part, {r: [0] for r in names}) for e in (g, x))
        # (the graph's launches are sized for the longest context, the eager step's for this one: other parts)
        assert lm.row_error(a, b.double().cpu()).max() < 0.02, step
        for r in names:
            at[r] += 1
        torch.cuda.synchronize()
        torch.randn(64, 64, device=dev).sum()
    assert g.runner._graphs and not x.runner._graphs


def test_sampling_sees_capped_logits(dev):
    """a temperature run goes through the sampler on the capped logits; a seed repeats it"""
    from vllm_omni_amd.sched_output import SamplingParams

    cfg = lm.CONFIGS["mixed"]
    w = weights(cfg, torch.bfloat16)
    prompt = lm.random_tokens(cfg, 20, 4)
    e = engine("mixed", w, torch.bfloat16, tokens=128)
    p = SamplingParams(max_tokens=12, temperature=0.8, top_k=20, seed=5, ignore_eos=True)
    a, b = e.generate([prompt], p), e.generate([prompt], p)
    assert a == b and len(a[0]) == 12 and all(0 <= t < cfg["vocab"] for t in a[0])


def test_checkpoint_folder_to_trace_and_command_line(dev, tmp_path, capsys, monkeypatch):
    """config.json + safetensors -> trace replay and the generate command"""
    from safetensors.torch import save_file

    from vllm_omni_amd import trace
    from vllm_omni_amd.__main__ import main as cli

    cfg = lm.CONFIGS["odd"]
    toks = lm.random_tokens(cfg, 70, 2)
    w, lg, _, lim16, _ = expected("odd", toks, torch.bfloat16)
    (tmp_path / "m").mkdir()
    (tmp_path / "m" / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "m" / "model.safetensors"))
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:40], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": toks[40:41], "want": [0]}, {"id": "b", "tokens": toks[:9], "want": [8, 2]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": toks[41:], "want": [28]}], "end": ["a"]}]
    for dtype, lim in (("float32", torch.full_like(lim16, 5e-5)), ("bfloat16", lim16)):
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
