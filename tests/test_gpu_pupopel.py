"""Pupopel behind the engine: logits against the plain forward for whole prompts, portions, decoding, mixed batches and
re-used pages and slots; graph replay against eager; greedy generation through the scheduler."""
import io
import json

import pytest
import torch

import pupopel_models as pm
from oracle import ref_pupopel as ref
from test_gpu_dogulorn import engine as _engine

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]


def with_ranks(cfg, ranks):
    """the configuration with the low-rank sizes that a checkpoint's tensors would give"""
    layers = [dict(x, mixer=dict(x["mixer"], **({"decay_rank": r[0], "gate_rank": r[1]} if r else {}))) for x, r in zip(cfg["layers"], ranks)]
    return dict(cfg, layers=layers)


def engine(name, weights, dtype, tokens=1024, seqs=4, **kw):
    return _engine(with_ranks(*pm.CONFIGS[name]), weights, dtype, tokens, seqs, **kw)


def steady(w):
    """the same weights with routers that leave no close calls (every token takes the experts of largest bias): rounding cannot
    turn a choice.  The 32-bit runs keep the routers that choose token by token."""
    out = dict(w)
    for k, v in w.items():
        if k.endswith("mlp.router"):
            out[k] = v * 0.05
        elif k.endswith("mlp.router.b"):
            out[k] = torch.randperm(v.numel(), generator=torch.Generator().manual_seed(v.numel())).to(v.dtype) * 1.5
    return out


_REF = {}


def weights(name, dtype):
    if (name, dtype) not in _REF:
        w = pm.random_weights(*pm.CONFIGS[name], seed=7)
        _REF[name, dtype] = steady(w) if dtype == torch.bfloat16 else w
    return _REF[name, dtype]


def expected(name, tokens, dtype=torch.float32):
    """weights, logits and streams of the plain forward, and per logits row and per stream row the limit of ``dtype``: what
    rounding alone does to that row, with room (kept between tests)"""
    cfg, w = pm.CONFIGS[name][0], weights(name, dtype)
    key = (name, dtype, tuple(tokens))
    if key not in _REF:
        lg, st = ref.forward(cfg, w, tokens)
        if dtype == torch.float32:
            lim, lims = torch.full((len(tokens),), 5e-5), [torch.full((len(tokens),), 5e-5)] * len(st)
        else:
            with pm.Bf16Products():
                lg2, st2 = ref.forward(cfg, w, tokens)
            lim, lims = 0.04 + 3 * pm.row_error(lg2, lg), [0.04 + 3 * pm.row_error(b, a) for a, b in zip(st, st2)]
        _REF[key] = lg, st, lim, lims
    lg, st, lim, lims = _REF[key]
    return w, lg, st, lim, lims


def check(got, want, limit, what=None):
    e = pm.row_error(got, want)
    assert (e <= limit).all(), (what, int((e / limit).argmax()), float((e / limit).max()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(pm.CONFIGS))
def test_every_layer_run_of_a_prompt(dev, name, dtype):
    toks = pm.random_tokens(pm.CONFIGS[name][0], 150, 1)
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
@pytest.mark.parametrize("name", list(pm.CONFIGS))
def test_portions_and_decoding(dev, name, dtype):
    """one engine, one request after the other (pages and slots are used again): token by token from the first token on,
    portions of changing size, most of the prompt and then single tokens"""
    toks = pm.random_tokens(pm.CONFIGS[name][0], 150, 1)
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


@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_batches_pages_and_slots_used_again(dev, dtype):
    name = "mixed"
    cfg = pm.CONFIGS[name][0]
    seqs = {f"r{i}": pm.random_tokens(cfg, n, 20 + i) for i, n in enumerate([90, 33, 1, 64, 17, 120, 2, 48])}
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
def test_far_tokens_show_at_page_borders_and_in_decoding(dev, dtype):
    """one early token changed (the first, the last of a page, the first of the next, the last of a chunk): everything after it
    must move as the plain forward says, in prompts and in decoding"""
    cfg, ranks = pm.CONFIGS["mixed"]
    sharp = lambda x: dict(x, mixer=dict(x["mixer"], left=dict(x["mixer"]["left"], scale=0.5)))   # noqa: E731
    cfg = dict(cfg, layers=[sharp(x) if x["type"] == "parallel" else x for x in cfg["layers"]])
    w = {k: v - 5.0 if k.endswith("A_log") else v for k, v in weights("mixed", dtype).items()}      # a state that hardly decays
    a = pm.random_tokens(cfg, 230, 5)
    e = _engine(with_ranks(cfg, ranks), w, dtype, tokens=1280)
    want_a = ref.forward(cfg, w, a)[0]
    for spot in (None, 0, 15, 16, 63):
        b = list(a)
        if spot is not None:
            b[spot] = (b[spot] + 1) % cfg["vocab"]
        want = ref.forward(cfg, w, b)[0]
        assert spot is None or pm.row_error(want[150:], want_a[150:]).median() > 1e-3          # the change is there, far above rounding
        lim = torch.full((80,), 2e-4)
        if dtype == torch.bfloat16:
            with pm.Bf16Products():
                lim = 0.04 + 3 * pm.row_error(ref.forward(cfg, w, b)[0][150:], want[150:])
        got = [e.run_portions({"b": b[:180]}, {"b": list(range(150, 180))})]
        got += [e.run_portions({"b": b[i:i + 1]}, {"b": [0]}, ["b"] if i == 229 else []) for i in range(180, 230)]
        check(torch.cat(got), want[150:], lim, spot)


def greedy_reference(cfg, w, prompt, n, got):
    """the plain forward on prompt + got: greedy token wherever the top two are apart"""
    lg = ref.forward(cfg, w, list(prompt) + got[:-1], torch.float64)[0][len(prompt) - 1:]
    top = lg.topk(2, -1)
    sure = (top.values[:, 0] - top.values[:, 1]) > 0.25 * lg.std()
    assert sure.sum() >= 0.2 * n
    for i in range(n):
        if sure[i]:
            assert got[i] == int(top.indices[i, 0]), i


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_scheduler(dev, dtype):
    from vllm_omni_amd.sched_output import SamplingParams

    cfg, ranks = pm.CONFIGS["wide"]
    w = weights("wide", dtype)
    prompts = [pm.random_tokens(cfg, n, 60 + i) for i, n in enumerate([1, 40, 97, 5, 64, 3])]
    e = engine("wide", w, dtype, tokens=256, max_num_batched_tokens=48, num_blocks=64)     # chunked prefill beside decoding
    out = e.generate(prompts, SamplingParams(max_tokens=24, ignore_eos=True))
    for p, o in zip(prompts, out):
        assert len(o) == 24
        greedy_reference(cfg, w, p, 24, o)
    assert e.runner.state_cache.num_free == 4
    for p, o in zip(prompts, e.generate(prompts[:3], SamplingParams(max_tokens=24, ignore_eos=True))):
        greedy_reference(cfg, w, p, 24, o)


def test_preempted_requests_recompute_their_state(dev):
    """a pool too small for all: the newest request loses its blocks and its state slot, and starts over from its tokens"""
    from vllm_omni_amd.sched_output import SamplingParams

    cfg, ranks = pm.CONFIGS["mixed"]
    w = pm.random_weights(cfg, ranks, seed=7)
    prompts = [pm.random_tokens(cfg, 30, 80 + i) for i in range(4)]
    params = SamplingParams(max_tokens=40, ignore_eos=True)
    roomy = engine("mixed", w, torch.float32, tokens=512).generate(prompts, params)
    e = engine("mixed", w, torch.float32, tokens=128, num_blocks=12)
    preempted = []
    orig = e.scheduler._preempt
    e.scheduler._preempt = lambda r: (preempted.append(r.request_id), orig(r))[1]
    tight = e.generate(prompts, params)
    assert preempted and e.runner.state_cache.num_free == 4
    for p, a, b in zip(prompts, roomy, tight):
        greedy_reference(cfg, w, p, 40, a)
        greedy_reference(cfg, w, p, 40, b)


@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_graph_replay_equals_eager(dev, name):
    """decode steps replayed from graphs, with other eager work between replays, against an engine that never captures"""
    cfg, ranks = pm.CONFIGS[name]
    w = pm.random_weights(cfg, ranks, seed=7)
    toks = {f"r{i}": pm.random_tokens(cfg, 60, 40 + i) for i in range(3)}
    g, x = engine(name, w, torch.bfloat16), engine(name, w, torch.bfloat16, enforce_eager=True)
    for e in (g, x):
        e.run_portions({r: t[:30 + 5 * i] for i, (r, t) in enumerate(toks.items())})
    at = {r: 30 + 5 * i for i, r in enumerate(toks)}
    for step in range(15):
        names = list(toks) if step % 4 else list(toks)[:2]
        part = {r: [toks[r][at[r]]] for r in names}
        a, b = (e.run_portions(part, {r: [0] for r in names}) for e in (g, x))
        # (the graph's launches are sized for the longest context, the eager step's for this one: other partitions)
        assert pm.row_error(a, b.double().cpu()).max() < 0.02, step
        for r in names:
            at[r] += 1
        torch.cuda.synchronize()
        torch.randn(64, 64, device=dev).sum()
    assert g.runner._graphs and not x.runner._graphs


def test_checkpoint_folder_to_trace_and_command_line(dev, tmp_path, capsys, monkeypatch):
    """config.json + safetensors (which alone has the low ranks) -> trace replay and the generate command"""
    from safetensors.torch import save_file

    from vllm_omni_amd import trace
    from vllm_omni_amd.__main__ import main as cli

    cfg, ranks = pm.CONFIGS["odd"]
    toks = pm.random_tokens(cfg, 70, 2)
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
    greedy_reference(cfg, w, toks[:12], 5, line["tokens"])
