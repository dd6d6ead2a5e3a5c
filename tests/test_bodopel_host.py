"""CPU: configuration, weights map, layer runs, argument checks of the Bodopel path, and the restatement itself."""
import copy
import ctypes
import json
import math

import pytest
import torch

import bodopel_models as bm
from oracle import ref_bodopel as ref


def build(cfg, dtype=torch.float32):
    from vllm_omni_amd.bodopel import BodopelConfig, BodopelForCausalLM

    c = BodopelConfig.from_dict(cfg)
    return c, BodopelForCausalLM(c, dtype, "cpu"), bm.random_weights(cfg)


def test_registry_picks_the_model(tmp_path):
    from vllm_omni_amd.bodopel import BodopelConfig, BodopelForCausalLM
    from vllm_omni_amd.registry import config_from_dir, config_from_hf, model_class_for

    cfg = bm.CONFIGS["mixed"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    c = config_from_dir(str(tmp_path))
    assert isinstance(c, BodopelConfig) and model_class_for(c) is BodopelForCausalLM
    assert config_from_hf(c) is c and config_from_hf(cfg) == c and BodopelConfig.from_json(str(tmp_path)) == c


def test_every_size_and_constant_comes_from_the_configuration():
    c, _, _ = build(bm.CONFIGS["mixed"])
    a = c.layers[1].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.softcap, a.scale) == (6, 3, 64, 24, 37, 4.0, 64 ** -0.5)
    assert c.layers[2].mixer.scale == 0.3 and c.layers[0].ff == 120 and c.layers[1].ff == 0
    assert (c.vocab_size, c.hidden_size, c.rms_norm_eps, c.embedding_scale, c.taps, c.max_positions) == (131, 96, 1e-5, 3.0, 4, 512)
    assert (c.loop.start, c.loop.stop, c.loop.times) == (1, 3, 3)


@pytest.mark.parametrize("name", list(bm.CONFIGS))
def test_layer_runs_and_their_memory(name):
    """every pass of a looped layer has a cache and rings of its own; a pass's vector comes ahead of its first layer only"""
    cfg = bm.CONFIGS[name]
    c, m, _ = build(cfg)
    assert c.runs == ref.layer_runs(cfg) == m.runs
    assert [t for _, t in c.runs if t is not None] == list(range(c.loop.times))
    specs = m.kv_cache_specs(16)
    assert list(specs) == list(range(len(c.runs)))
    taps = cfg["canon"]["taps"]
    want = sum(2 if cfg["layers"][i]["mlp"] else 1 for i, _ in c.runs) if taps > 1 else 0
    states = [torch.zeros(3, *s.shape, dtype=s.dtype) for s in m.state_specs()]
    assert len(states) == want and all(t.shape == (3, taps - 1, cfg["width"]) for t in states)
    assert m.is_recurrent == (taps > 1)
    m.bind_states(states)
    rings = [r.ring for run in m.rings for r in run]
    assert [r.data_ptr() for r in rings if r is not None] == [t.data_ptr() for t in states]
    assert m.prefill_windows() == sorted({x["mixer"]["mask"]["size"] for x in cfg["layers"]})


def test_loop_mask_and_cap_are_optional():
    cfg = copy.deepcopy(bm.CONFIGS["odd"])
    cfg["loop"] = None
    cfg["layers"][0]["mixer"].pop("mask")
    cfg["layers"][1]["mixer"]["softcap"] = None
    c, m, _ = build(cfg)
    assert c.runs == [(0, None), (1, None)] and c.layers[0].mixer.window is None and c.layers[1].mixer.softcap == 0.0
    assert "loop.step" not in dict(m.named_weights()) and m.prefill_windows()[-1] == 2**31 - 1


@pytest.mark.parametrize("change,match", [
    (lambda d: d["layers"][0].update(type="mamba"), "unknown mixer type"),
    (lambda d: d["layers"][0]["mlp"].update(kind="sparse"), "unknown feed-forward kind"),
    (lambda d: d["loop"].update(stop=9), "does not fit"),
    (lambda d: d["loop"].update(times=0), "does not fit"),
    (lambda d: d["canon"].update(taps=0), "tap"),
    (lambda d: d.update(max_positions=0), "position table"),
    (lambda d: d.update(layers=[]), "at least one layer"),
])
def test_configurations_that_do_not_exist_are_refused(change, match):
    from vllm_omni_amd.bodopel import BodopelConfig

    d = copy.deepcopy(bm.CONFIGS["mixed"])
    change(d)
    with pytest.raises(ValueError, match=match):
        BodopelConfig.from_dict(d)


@pytest.mark.parametrize("change,match", [
    (lambda m: m.update(heads=7), "multiple"),
    (lambda m: m.update(mask={"size": 0}), "window"),
    (lambda m: m.update(softcap=-1.0), "soft cap"),
])
def test_sizes_that_do_not_fit_are_refused(change, match):
    from vllm_omni_amd.bodopel import BodopelConfig, BodopelForCausalLM

    d = copy.deepcopy(bm.CONFIGS["mixed"])
    change(d["layers"][1]["mixer"])
    with pytest.raises(ValueError, match=match):
        BodopelForCausalLM(BodopelConfig.from_dict(d), torch.float32, "cpu")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", list(bm.CONFIGS))
def test_weights_map_one_to_one(name, dtype):
    """every checkpoint tensor has a place of its own in the fused product; scores' and weights' constants stay 32-bit"""
    cfg = bm.CONFIGS[name]
    _, m, w = build(cfg, dtype)
    assert m.load_weights(w) == set(w)
    params = dict(m.named_weights())
    assert set(params) == set(w)
    for n, t in w.items():
        keep = torch.float32 if n.rsplit(".", 1)[-1] in ("r1", "r2", "talk") else dtype
        assert params[n].dtype == keep and torch.equal(params[n].float(), t.to(keep).float()), n
    for i, layer in enumerate(m.layers):
        lin = layer.mixer.proj
        assert int(lin.weight.count_nonzero()) == sum(int(w[f"l{i}.mix.{x}"].count_nonzero()) for x in "qkvg")
        assert int(lin.bias.count_nonzero()) == sum(int(w[f"l{i}.mix.{x}.b"].count_nonzero()) for x in "qkv")
    with pytest.raises(KeyError):
        m.load_weights({"l0.mix.g.b": torch.zeros(1)})
    with pytest.raises(ValueError):
        m.load_weights({"embed": torch.zeros(3, 3)})


def test_models_outside_the_envelope_say_so():
    from vllm_omni_amd.bodopel import BodopelForCausalLM
    from vllm_omni_amd.model_runner import GPUARModelRunner

    c, m, _ = build(bm.CONFIGS["odd"])
    with pytest.raises(ValueError, match="bfloat16 or float32"):
        BodopelForCausalLM(c, torch.float16, "cpu")
    with pytest.raises(ValueError):
        m.quantize_int8()
    r = GPUARModelRunner(c, "cpu", torch.float32, max_num_reqs=2, max_model_len=c.max_positions + 1, max_num_batched_tokens=16,
                         block_size=16, engine_output_type="text")
    with pytest.raises(ValueError, match="position table"):
        r.load_model()


def test_prefix_caching_is_refused_with_state():
    from vllm_omni_amd.model_runner import GPUARModelRunner

    c, _, _ = build(bm.CONFIGS["odd"])
    r = GPUARModelRunner(c, "cpu", torch.float32, max_num_reqs=2, max_model_len=64, max_num_batched_tokens=16, block_size=16,
                         engine_output_type="text", enable_prefix_caching=True)
    r.load_model()
    with pytest.raises(ValueError, match="prefix caching"):
        r.initialize_kv_cache(8)


def test_argument_validation_without_gpu():
    from vllm_omni_amd import _C

    lib = _C.lib
    buf = (ctypes.c_char * 4096)()
    p = (ctypes.addressof(buf) + 15) & ~15
    bad, no, ws = _C.MI_ERR_INVALID_ARG, _C.MI_ERR_UNSUPPORTED, _C.MI_ERR_WORKSPACE
    add = lambda **k: lib.mi_residual_add_norm_conv(p, k.get("y", p), 0, None, p, 1.0, p, p, k.get("ring", p), p, p, k.get("taps", 2),   # noqa: E731
                                                    1e-6, 2, 8, 8, 8, k.get("hs", 8), k.get("dt", 1), None)
    assert add(y=None) == bad and add(hs=7) == bad and add(taps=0) == bad and add(ring=None) == bad and add(dt=_C.MI_DTYPE_F16) == no
    assert lib.mi_embed_pos_norm(p, p, p, 1.0, p, None, 4, None, p, 1.0, p, None, None, None, 0, 1e-6, 2, 8, 10, 8, 8, 1, None) == bad
    conv = lambda out, taps: lib.mi_input_conv(out, p, p, p, p, p, p, 0, 1, 4, taps, 8, 8, 8, 1, None)   # noqa: E731
    assert conv(p, 2) == bad and conv(p + 64, 0) == bad and conv(p + 64, 40) == no
    assert lib.mi_relu_squared(p, p, 0, 2, 8, 8, 7, 1, None) == bad
    assert lib.mi_linear_relu_squared(p, p, p, 2, 16, 100, 104, 16, None, 0, 1, None) == no
    assert lib.mi_row_norm_cache(p, 100, p, p, p, 64, p, p, p, 2, 4, 2, 16, 16, 12, 16, 512, 32, 16, 1e-6, 1, None) == bad
    ta = {n: p for n, t in _C.TalkingAttnArgs._fields_ if t is ctypes.c_void_p}
    ta.update(q_stride=256, out_stride=256, gate_stride=256, cache_block_stride=2048, cache_token_stride=128, cache_head_stride=64,
              table_stride=4, heads=4, kv_heads=2, head_dim=64, vdim=64, block_size=16, window=8, scale=1.0, softcap=5.0)
    a = lambda **kw: ctypes.byref(_C.TalkingAttnArgs(**{**ta, **kw}))   # noqa: E731
    for kw in (dict(heads=5), dict(r1=None), dict(talk=None), dict(window=0), dict(vdim=65), dict(out_stride=255), dict(gate_stride=9)):
        assert lib.mi_talking_attn_rows(a(**kw), 0, 2, 1, 1, None) == bad, kw
        assert lib.mi_talking_decode(a(**kw), 1, 8, p, 1 << 30, None) == bad, kw
        assert lib.mi_talking_prefill(a(**kw), p, 64, 1, 2, 2, p, 1 << 30, None) == bad, kw
    assert lib.mi_talking_attn_rows(a(heads=500, kv_heads=1, q_stride=1 << 20, out_stride=1 << 20, gate_stride=1 << 20), 0, 2, 1, 1, None) == no
    for kw in (dict(head_dim=96), dict(block_size=8), dict(softcap=5000.0), dict(heads=66, q_stride=9999, out_stride=9999, gate_stride=9999)):
        q = dict(q_stride=512) if "head_dim" in kw else {}
        assert lib.mi_talking_decode(a(**{**q, **kw}), 1, 8, p, 1 << 30, None) == no, kw
        assert lib.mi_talking_prefill(a(**{**q, **kw}), p, 64, 1, 2, 2, p, 1 << 30, None) == no, kw
    assert lib.mi_talking_prefill(a(), p, 63, 1, 2, 2, p, 1 << 30, None) == bad
    need = lib.mi_talking_decode_workspace_bytes(1, 4, 2, 64, 8, 100)
    assert need > 0 and lib.mi_talking_decode(a(), 1, 100, p, need - 1, None) == ws
    need = lib.mi_talking_prefill_workspace_bytes(2, 4, 2, 64, 64)
    assert need > 0 and lib.mi_talking_prefill(a(), p, 64, 1, 2, 2, p, need - 1, None) == ws
    assert lib.mi_talking_attn_supported(32, 8, 128, 96, 16, 50.0) == 1 and lib.mi_talking_attn_supported(40, 8, 128, 96, 16, 50.0) == 0


def test_engine_runs_no_longer_than_the_position_table():
    from vllm_omni_amd.bodopel import BodopelConfig
    from vllm_omni_amd.engine import LLMEngine

    seen = {}

    class Stop(Exception):
        pass

    def worker(wc):
        seen["len"] = wc.max_model_len
        raise Stop

    import vllm_omni_amd.engine as engine

    orig, engine.GPUARWorker = engine.GPUARWorker, worker
    try:
        for asked, got in ((100, 100), (5000, 512)):
            with pytest.raises(Stop):
                LLMEngine(BodopelConfig.from_dict(bm.CONFIGS["mixed"]), max_model_len=asked)
            assert seen["len"] == got
    finally:
        engine.GPUARWorker = orig


# ------------------------------------------------------------------------------------------------ the restatement itself
def test_heads_that_do_not_talk_are_a_softmax():
    g = torch.Generator().manual_seed(1)
    q, k, v = torch.randn(9, 2, 4, generator=g), torch.randn(9, 1, 4, generator=g), torch.randn(9, 1, 3, generator=g)
    r1, r2 = torch.tensor([0.5, 0.1]), torch.tensor([1.0, 3.0])
    got = ref.talking_attention(q, k, v, 0.7, 2.0, r1, r2, 4, torch.eye(2))
    for h in range(2):
        d = (torch.arange(9)[:, None] - torch.arange(9)[None]).float()
        s = 2.0 * torch.tanh(q[:, h] @ k[:, 0].T * 0.7 / 2.0) - r1[h] * torch.log(1 + r2[h] * d.clamp(min=0))
        s = s.masked_fill((d < 0) | (d > 3), -math.inf)
        assert torch.allclose(got[:, h], torch.softmax(s, -1) @ v[:, 0], atol=1e-6)


def test_mixed_heads_read_their_own_values():
    """head h's output is sum_g T[h, g] (g's weights on h's values)"""
    g = torch.Generator().manual_seed(2)
    p, v = torch.rand(4, 5, 5, generator=g), torch.randn(5, 2, 3, generator=g)
    t = torch.randn(4, 4, generator=g)
    got = ref.apply_weights(ref.mix_heads(p, t), v)
    for h in range(4):
        want = sum(t[h, x] * (p[x] @ v[:, h // 2]) for x in range(4))
        assert torch.allclose(got[:, h], want, atol=1e-5)


def test_filter_starts_from_zeros_and_keeps_its_row():
    y = ref.with_conv(torch.ones(4, 1), torch.tensor([[1000.0, 100.0, 10.0]]))
    assert y[:, 0].tolist() == [11.0, 111.0, 1111.0, 1111.0]


def test_a_pass_adds_its_vector_once():
    """a model of layers that add nothing: the stream is the embedding and the passes' vectors"""
    cfg = bm.model([bm.layer(2, 1, 8, 8, 4, 0), bm.layer(2, 1, 8, 8, 4, 8)], (0, 2, 3), vocab=11, width=16)
    w = {k: torch.zeros_like(v) if k.endswith((".o", ".down")) else v for k, v in bm.random_weights(cfg).items()}
    _, st = ref.forward(cfg, w, [1, 2, 3])
    x = 3.0 * w["embed"][[1, 2, 3]].double() + w["pos"][:3].double()
    steps = w["loop.step"].double().cumsum(0)
    for r, s in enumerate(st):
        assert torch.allclose(s, x + steps[r // 2])
