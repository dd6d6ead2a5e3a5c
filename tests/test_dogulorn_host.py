"""CPU: configuration, registry, state slots, given-portion scheduling and argument checks of the Dogulorn path, and the
plain restatement against independent formulations of the same mechanisms."""
import copy
import ctypes
import json

import pytest
import torch

import dogulorn_models as dm
from oracle import ref_dogulorn as ref


# ------------------------------------------------------------------------------------------------ configuration
def test_registry_reads_the_architecture(tmp_path):
    from vllm_omni_amd import registry
    from vllm_omni_amd.dogulorn import DogulornConfig, DogulornForCausalLM
    from vllm_omni_amd.talker import Qwen2_5OmniTalkerForConditionalGeneration, TalkerConfig

    (tmp_path / "config.json").write_text(json.dumps(dm.CONFIGS["mixed"]))
    cfg = registry.config_from_dir(str(tmp_path))
    assert isinstance(cfg, DogulornConfig) and registry.model_class_for(cfg) is DogulornForCausalLM
    assert registry.config_from_hf(cfg) is cfg
    assert registry.model_class_for(TalkerConfig()) is Qwen2_5OmniTalkerForConditionalGeneration
    hf = dict(hidden_size=64, num_attention_heads=2, num_hidden_layers=1, vocab_size=32, intermediate_size=64)
    assert isinstance(registry.config_from_hf(hf), TalkerConfig)
    with pytest.raises(ValueError, match="unknown architecture"):
        registry.config_from_hf({"architecture": "Nothing"})
    with pytest.raises(TypeError):
        registry.model_class_for(object())


def test_every_size_and_constant_comes_from_the_configuration():
    from vllm_omni_amd.registry import config_from_hf

    d = dm.CONFIGS["mixed"]
    c = config_from_hf(d)
    assert (c.vocab_size, c.hidden_size, c.num_hidden_layers, c.token_side_dim) == (131, 96, 7, 16)
    assert (c.rms_norm_eps, c.embedding_scale, c.bigram_buckets, c.bigram_mul_prev, c.bigram_mul_cur) == (1e-5, 2.5, 97, 31, 5)
    for got, want in zip(c.layers, d["layers"]):
        m = want["mixer"]
        assert (got.ff, got.limit) == ((want["mlp"]["ff"], want["mlp"]["limit"]) if want["mlp"] else (0, 0.0))
        if want["type"] == "delta":
            assert vars(got.mixer) == m
        else:
            assert vars(got.mixer) == {**{k: v for k, v in m.items() if k != "mask"}, "window": m["mask"]["size"], "kv_from": m.get("kv_from")}


@pytest.mark.parametrize("change,match", [
    (lambda d: d["layers"][2]["mixer"].update(kv_from=0), "kv_from"),          # a recurrent layer has no latent
    (lambda d: d["layers"][2]["mixer"].update(kv_from=4), "kv_from"),          # a later layer
    (lambda d: d["layers"][5]["mixer"].update(kv_from=2), "kv_from"),          # a layer without a cache of its own
    (lambda d: d["layers"][2]["mixer"].update(kv_rank=24), "kv_from"),         # another rank
    (lambda d: d["layers"][1]["mixer"]["mask"].update(size=0), "window"),
    (lambda d: d["layers"][0].update(type="other"), "mixer type"),
    (lambda d: d["layers"][0]["mlp"].update(kind="sparse"), "feed-forward kind"),
])
def test_configurations_that_do_not_exist_are_refused(change, match):
    from vllm_omni_amd.registry import config_from_hf

    d = copy.deepcopy(dm.CONFIGS["mixed"])
    change(d)
    with pytest.raises(ValueError, match=match):
        config_from_hf(d)


def test_weights_map_one_to_one_and_caches_follow_the_layers():
    from vllm_omni_amd.dogulorn import DogulornForCausalLM
    from vllm_omni_amd.registry import config_from_hf

    for name, d in dm.CONFIGS.items():
        m = DogulornForCausalLM(config_from_hf(d), torch.float32, torch.device("cpu"))
        w = dm.random_weights(d, 1)
        params = dict(m.named_weights())
        assert {k: tuple(v.shape) for k, v in params.items()} == {k: tuple(v.shape) for k, v in w.items()}
        assert m.load_weights(w) == set(w)
        for k, v in w.items():       # fused parameters hold every piece at its place
            assert torch.equal(params[k], v.float()), k
        with pytest.raises(KeyError):
            m.load_weights({"l0.mix.nothing": torch.zeros(1)})
        with pytest.raises(ValueError, match="shape"):
            m.load_weights({"head": torch.zeros(1, 1)})
        own = [i for i, x in enumerate(d["layers"]) if x["type"] != "delta" and "kv_from" not in x["mixer"]]
        specs = m.kv_cache_specs(16)
        assert list(specs) == own and all(s.page_bytes == 16 * s.rank * 4 for s in specs.values())
        caches = {i: torch.zeros(2, 16, s.rank) for i, s in specs.items()}
        m.bind_kv_caches(caches)
        for i, x in enumerate(d["layers"]):
            if x["type"] != "delta":
                assert m.layers[i].mixer.cache is caches[x["mixer"].get("kv_from", i)]
        assert len(m.state_specs()) == 1 + 2 * sum(x["type"] == "delta" for x in d["layers"])
        assert m.prefill_windows() == sorted({x["mixer"]["mask"]["size"] for x in d["layers"] if x["type"] != "delta"})


def test_padded_projection_rows_stay_zero():
    from vllm_omni_amd.mixers import ReplicatedLinear

    lin = ReplicatedLinear(8, {"a": 3, "b": 6}, torch.float32, torch.device("cpu"), pad=True)
    assert lin.weight.shape == (16, 8) and not lin.weight[9:].any() and lin.weight[:9].any()
    assert [(n, tuple(t.shape)) for n, t in lin.named("x.")] == [("x.a", (3, 8)), ("x.b", (6, 8))]


# ------------------------------------------------------------------------------------------------ state, scheduling
def test_state_slots():
    from vllm_omni_amd.state_cache import StateCache, StateSpec

    c = StateCache(2, torch.device("cpu"))
    t = c.allocate([StateSpec((3, 2), torch.float32), StateSpec((), torch.int64)])
    assert t[0].shape == (3, 3, 2) and t[1].shape == (3,) and StateSpec((3, 2), torch.float32).slot_bytes == 24
    a, b = c.acquire(), c.acquire()
    assert {a, b} == {0, 1} and c.scratch_slot == 2
    with pytest.raises(RuntimeError, match="state slots"):
        c.acquire()
    c.release(a)
    with pytest.raises(ValueError):
        c.release(a)
    with pytest.raises(ValueError):
        c.release(2)
    assert c.acquire() == a


def scheduler(num_blocks=9, seqs=2, tokens=64, length=64):
    from vllm_omni_amd.scheduler import StandaloneARScheduler

    class Cfg:
        scheduler_config = {"max_num_seqs": seqs, "max_num_batched_tokens": tokens}
        cache_config = {"block_size": 16}
        model_config = {"max_model_len": length}

    return StandaloneARScheduler(Cfg, num_blocks=num_blocks)


def test_given_portions_are_scheduled_exactly():
    from vllm_omni_amd.sched_output import RequestStatus

    s = scheduler()
    so = s.schedule_portions({"a": [1, 2, 3]})
    assert so.num_scheduled_tokens == {"a": 3} and so.scheduled_new_reqs[0].prompt_token_ids == [1, 2, 3]
    so = s.schedule_portions({"a": [4], "b": list(range(20))})
    assert so.scheduled_cached_reqs.req_ids == ["a"] and so.scheduled_cached_reqs.new_token_ids == [[4]]
    assert so.scheduled_cached_reqs.num_computed_tokens == [3] and len(so.scheduled_new_reqs[0].block_ids[0]) == 2
    so = s.schedule_portions({"b": list(range(13))})             # a sits the step out, b grows into its third block
    assert so.num_scheduled_tokens == {"b": 13} and len(so.scheduled_cached_reqs.new_block_ids[0][0]) == 1
    assert s.requests["a"].num_computed_tokens == 4 and s.requests["b"].num_computed_tokens == 33
    free = s.kv_cache_manager.block_pool.get_num_free_blocks()
    for bad in ({"c": [1]}, {"a": []}, {"a": [0] * 65}):          # a third live request, no tokens, too many tokens
        with pytest.raises((RuntimeError, ValueError)):
            s.schedule_portions(bad)
    assert s.kv_cache_manager.block_pool.get_num_free_blocks() == free and s.requests["a"].num_computed_tokens == 4
    s.finish_requests(["a"], RequestStatus.FINISHED_STOPPED)
    so = s.schedule_portions({"c": [7]})
    assert so.finished_req_ids == {"a"} and set(s.requests) == {"b", "c"}
    with pytest.raises(RuntimeError, match="KV blocks"):
        scheduler(num_blocks=3).schedule_portions({"x": [0] * 33})


def test_preempted_requests_are_named_to_the_runner():
    from vllm_omni_amd.sched_output import Request, SamplingParams

    s = scheduler(num_blocks=4, seqs=2)
    for r in ("a", "b"):
        s.add_request(Request(r, list(range(16)), SamplingParams(max_tokens=30, ignore_eos=True)))
    assert s.schedule().preempted_req_ids == set()
    for r in ("a", "b"):
        s.requests[r].output_token_ids.append(1)
    so = s.schedule()                                     # three blocks: a takes the last one, b goes
    assert so.preempted_req_ids == {"b"} and so.num_scheduled_tokens == {"a": 1}


def test_runner_frees_and_takes_state_slots_and_learns_portions():
    """host side of the runner on the CPU: the forward pass is replaced, everything before it is the product"""
    from vllm_omni_amd.model_runner import GPUARModelRunner
    from vllm_omni_amd.registry import config_from_hf
    from vllm_omni_amd.sched_output import RequestStatus

    r = GPUARModelRunner(config_from_hf(dm.CONFIGS["mixed"]), torch.device("cpu"), torch.float32, max_num_reqs=2, max_model_len=64,
                         max_num_batched_tokens=64, block_size=16, engine_output_type="text", enforce_eager=True)
    r.load_model()
    r.initialize_kv_cache(9)
    seen = []

    def forward(n, total, md):
        pure = md.num_decodes == n == total
        seen.append({"ids": (r.last_token_ids.gpu[:n] if pure else r.input_ids.gpu[:total]).tolist(), "slots": md.state_rows.tolist(),
                     "prev": None if md.prev_ids is None else md.prev_ids.tolist(), "leave": md.prev_slots.tolist(),
                     "ctx": {w: (b.tolist(), k) for w, (b, k) in md.prefill_ctx.items()}, "decodes": md.num_decodes})
        h = torch.zeros(total, 96)
        return h, torch.zeros(n, 131), torch.zeros(n, dtype=torch.int64)

    r._forward = forward
    s = scheduler()

    def step(p):
        r.execute_model(s.schedule_portions(p))
        r.discard_step()
        return seen[-1]

    a = step({"a": [5, 6, 7]})
    assert a["ids"] == [5, 6, 7] and a["prev"] == [-1, 5, 6] and a["leave"] == [-1, -1, 0] and a["slots"] == [0]
    assert a["ctx"][5] == ([0, 64], 64)
    b = step({"a": [8], "b": list(range(20, 60))})          # a decodes beside b's prompt
    assert b["decodes"] == 1 and b["ids"] == [8] + list(range(20, 60)) and b["prev"][:3] == [-1, -1, 20]
    assert b["leave"] == [0] + [-1] * 39 + [1] and b["slots"] == [0, 1]
    c = step({"b": [60, 61]})                               # a is left out; b goes on behind position 39
    assert c["ids"] == [60, 61] and c["prev"] == [59, 60] and c["slots"] == [1] and c["ctx"][21] == ([0, 64], 64)
    assert c["ctx"][5] == ([0, 64], 64) and c["ctx"][70] == ([0, 64], 64)
    d = step({"a": [9], "b": [62]})
    assert d["decodes"] == 2 and sorted(zip(d["slots"], d["ids"])) == [(0, 9), (1, 62)] and d["prev"] is None and d["leave"] == d["slots"]
    s.finish_requests(["a"], RequestStatus.FINISHED_STOPPED)
    e = step({"c": [1]})
    assert e["slots"] == [0] and r.state_cache.num_free == 0
    with pytest.raises(RuntimeError, match="State error"):
        r.discard_step()


def test_prefix_caching_is_refused_behind_recurrent_layers():
    from vllm_omni_amd.model_runner import GPUARModelRunner
    from vllm_omni_amd.registry import config_from_hf

    r = GPUARModelRunner(config_from_hf(dm.CONFIGS["mixed"]), torch.device("cpu"), torch.float32, max_num_reqs=2, max_model_len=64,
                         max_num_batched_tokens=64, block_size=16, engine_output_type="text", enable_prefix_caching=True)
    r.load_model()
    with pytest.raises(ValueError, match="recurrent"):
        r.initialize_kv_cache(9)


# ------------------------------------------------------------------------------------------------ C ABI
def test_argument_validation_without_gpu():
    from vllm_omni_amd import _C

    lib = _C.lib
    buf = (ctypes.c_char * 4096)()
    p = (ctypes.addressof(buf) + 15) & ~15
    bad = _C.MI_ERR_INVALID_ARG
    assert lib.mi_residual_norm(None, p, 0, p, p, p, 1e-6, 2, 8, 8, 8, 8, 1, None) == bad
    assert lib.mi_residual_norm(p, p, 0, p, p, p, 1e-6, 2, 8, 8, 8, 8, _C.MI_DTYPE_F16, None) == _C.MI_ERR_UNSUPPORTED
    assert lib.mi_residual_norm(p, p, 0, p, p, p, 1e-6, 0, 8, 8, 8, 8, 1, None) == _C.MI_OK
    assert lib.mi_latent_decode(p, p, p, p, p, 1, 4, 516, 16, 8, 64, 1.0, 8256, 516, 4, None, 0, None) == _C.MI_ERR_UNSUPPORTED
    assert lib.mi_latent_decode(p, p, p, p, p, 1, 4, 64, 12, 8, 64, 1.0, 768, 64, 4, None, 0, None) == _C.MI_ERR_UNSUPPORTED
    need = lib.mi_latent_decode_workspace_bytes(1, 4, 64, 4096, 4096)
    assert need > 0 and lib.mi_latent_decode_workspace_bytes(512, 4, 64, 4096, 4096) == 0
    assert lib.mi_latent_decode(p, p, p, p, p, 1, 4, 64, 16, 4096, 4096, 1.0, 1024, 64, 4, p, need - 1, None) == _C.MI_ERR_WORKSPACE
    assert lib.mi_latent_prefill(p, p, p, p, p, p, p, 1, 8, 2, 12, 16, 8, 1.0, 32, 24, 24, 64, None) == _C.MI_ERR_UNSUPPORTED
    # heads that do not divide, a projection row too short, a workspace too small
    def delta(**kw):
        n = [f for f, t in _C.GatedDeltaArgs._fields_ if t is ctypes.c_void_p]
        a = _C.GatedDeltaArgs(**{**dict.fromkeys(n, p), **dict(qkv_stride=400, gate_stride=400, beta_stride=400, decay_stride=400,
                              out_stride=400, num_reqs=1, heads=4, kv_heads=2, dim=16, vdim=16, taps=4, eps=1e-6), **kw})
        return ctypes.byref(a)

    assert lib.mi_gated_delta_step(delta(kv_heads=3), 1, 1, None) == bad
    assert lib.mi_gated_delta_step(delta(qkv_stride=100), 1, 1, None) == bad
    assert lib.mi_gated_delta_step(delta(channel_decay=1, decay_stride=32), 1, 1, None) == bad
    assert lib.mi_gated_delta_chunked_workspace_bytes(64, 1, 4, 300, 64, 0) == 0
    assert lib.mi_gated_delta_chunked_workspace_bytes(64, 1, 4, 136, 64, 1) == 0
    ws = lib.mi_gated_delta_chunked_workspace_bytes(64, 1, 4, 64, 64, 0)
    assert lib.mi_gated_delta_chunked(delta(dim=64, vdim=64, qkv_stride=600), 0, 64, 64, p, ws - 1, 1, None) == _C.MI_ERR_WORKSPACE
    assert lib.mi_linear_clamped_glu(p, p, p, 1, 16, 64, 64, 16, 0.0, 1.0, 1, None) == bad


# ------------------------------------------------------------------------------------------------ the restatement itself
def test_window_attention_against_a_masked_softmax():
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(30, 2, 8, generator=g, dtype=torch.float64) for _ in range(3))
    for size in (1, 4, 30, 99):
        i = torch.arange(30)
        d = i[:, None] - i[None]
        s = torch.einsum("ihd,jhd->hij", q, k) * 0.3
        s = s.masked_fill(~((d >= 0) & (d < size)), float("-inf"))
        want = torch.einsum("hij,jhd->ihd", s.softmax(-1), v)
        torch.testing.assert_close(ref.window_attention(q, k, v, 0.3, size), want)


def test_delta_rule_against_the_chunk_formulation():
    """U from one triangular system over the whole sequence"""
    g = torch.Generator().manual_seed(1)
    T, D, V = 17, 6, 5
    q, k, v = (torch.randn(T, 1, n, generator=g, dtype=torch.float64) for n in (D, D, V))
    k = ref.unit(k)
    beta, decay = torch.rand(T, 1, generator=g, dtype=torch.float64), torch.rand(T, 1, generator=g, dtype=torch.float64)
    o, s = ref.delta_rule(q, k, v, beta, decay)
    G = decay[:, 0].log().cumsum(0)
    e = torch.exp(G[:, None] - G[None]).tril()
    A = (beta * (k[:, 0] @ k[:, 0].T) * e).tril(-1)
    U = torch.linalg.solve(torch.eye(T, dtype=torch.float64) + A, beta * v[:, 0])
    torch.testing.assert_close(o[:, 0], ((q[:, 0] @ k[:, 0].T) * e) @ U)
    torch.testing.assert_close(s[0], (k[:, 0] * torch.exp(G[-1] - G)[:, None]).T @ U)


def test_convolution_and_embedding_at_the_first_tokens():
    x = torch.arange(8, dtype=torch.float64).view(4, 2) + 1
    w = torch.tensor([[1.0, 10.0, 100.0], [0.5, 0.0, 2.0]], dtype=torch.float64)
    want = torch.stack([torch.tensor([100 * x[t, 0] + 10 * (x[t - 1, 0] if t else 0) + (x[t - 2, 0] if t > 1 else 0),
                                      2 * x[t, 1] + 0.5 * (x[t - 2, 1] if t > 1 else 0)]) for t in range(4)])
    torch.testing.assert_close(ref.causal_conv(x, w), want)
    table, pairs = torch.randn(9, 3).double(), torch.randn(6, 3).double()
    got = ref.embed([8, 2, 2], table, pairs, 3.0, 4, 7)
    for i, row in enumerate((5, (8 * 4 + 2 * 7) % 5, (2 * 4 + 2 * 7) % 5)):
        torch.testing.assert_close(got[i], table[[8, 2, 2][i]] * 3 + pairs[row])
