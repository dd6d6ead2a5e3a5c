"""CPU: configuration, weights map, layer runs, argument checks of the Pupopel path, and the restatement itself."""
import copy
import ctypes
import json
import math

import pytest
import torch

import pupopel_models as pm
from oracle import ref_pupopel as ref


def build(name, dtype=torch.float32):
    from vllm_omni_amd.pupopel import PupopelConfig, PupopelForCausalLM

    cfg, ranks = pm.CONFIGS[name]
    w = pm.random_weights(cfg, ranks)
    c = PupopelConfig.from_dict(cfg, {k: tuple(v.shape) for k, v in w.items()})
    return c, PupopelForCausalLM(c, dtype, "cpu"), w


def test_registry_takes_ranks_from_the_checkpoint(tmp_path):
    from safetensors.torch import save_file

    from vllm_omni_amd.pupopel import PupopelConfig, PupopelForCausalLM
    from vllm_omni_amd.registry import config_from_dir, config_from_hf, model_class_for

    cfg, ranks = pm.CONFIGS["mixed"]
    w = pm.random_weights(cfg, ranks)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    c = config_from_dir(str(tmp_path))
    assert isinstance(c, PupopelConfig) and model_class_for(c) is PupopelForCausalLM
    assert [(x.mixer.decay_rank, x.mixer.gate_rank) for x in c.layers if hasattr(x.mixer, "decay_rank")] == [r for r in ranks if r]
    assert config_from_hf(c) is c
    assert config_from_hf(cfg).layers[0].mixer.decay_rank == cfg["layers"][0]["mixer"]["dim"]      # nothing known: the head size


def test_every_size_and_constant_comes_from_the_configuration():
    c, _, _ = build("mixed")
    a = c.layers[1].mixer
    assert (a.left.heads, a.left.kv_heads, a.left.dim, a.left.vdim, a.left.temp_coef, a.left.temp_every) == (6, 2, 48, 40, 0.4, 7)
    assert a.left.scale == 48 ** -0.5 and a.left.slopes == ref.head_slopes(6)
    assert (a.right.heads, a.right.dim, a.right.vdim, a.right.decay) == (3, 24, 32, [0.5, 0.9, 0.999])
    assert (a.left_scale, a.right_scale) == (0.7, 1.3)
    d = c.layers[0].mixer
    assert (d.heads, d.kv_heads, d.dim, d.vdim, d.conv, d.decay_rank, d.gate_rank) == (4, 2, 24, 40, 3, 16, 12)
    assert c.layers[0].mlp == 72 and c.layers[2].mlp is None
    m = c.layers[4].mlp
    assert (m.experts, m.top, m.ff, m.shared_ff) == (9, 3, 24, 32)
    assert (c.vocab_size, c.hidden_size, c.rms_norm_eps) == (131, 96, 1e-5)


@pytest.mark.parametrize("name", list(pm.CONFIGS))
def test_layer_runs_and_their_memory(name):
    c, m, _ = build(name)
    assert c.runs == ref.layer_runs(pm.CONFIGS[name][0]) == m.runs
    assert sum(s for _, s in c.runs) == c.loop.times
    attn = [r for r, (i, _) in enumerate(c.runs) if pm.CONFIGS[name][0]["layers"][i]["type"] == "parallel"]
    specs = m.kv_cache_specs(16)
    assert list(specs) == attn
    states = [torch.zeros(3, *s.shape, dtype=s.dtype) for s in m.state_specs()]
    m.bind_states(states)
    assert [t.data_ptr() for mem in m.memory for t in mem.states] == [t.data_ptr() for t in states]     # every run its own, once


def test_loop_is_optional():
    from vllm_omni_amd.pupopel import PupopelConfig, PupopelForCausalLM

    cfg = copy.deepcopy(pm.CONFIGS["odd"][0])
    cfg["loop"] = None
    c = PupopelConfig.from_dict(cfg)
    assert c.runs == [(0, False), (1, False), (2, False)]
    assert "loop.in" not in dict(PupopelForCausalLM(c, torch.float32, "cpu").named_weights())


@pytest.mark.parametrize("change,match", [
    (lambda d: d["layers"][0].update(type="mamba"), "unknown mixer type"),
    (lambda d: d["layers"][0]["mlp"].update(kind="sparse"), "unknown feed-forward kind"),
    (lambda d: d["loop"].update(stop=9), "does not fit"),
    (lambda d: d["loop"].update(times=0), "does not fit"),
    (lambda d: d["layers"][1]["mixer"]["left"]["q_temp"].update(every=0), "q_temp.every"),
])
def test_configurations_that_do_not_exist_are_refused(change, match):
    from vllm_omni_amd.pupopel import PupopelConfig

    d = copy.deepcopy(pm.CONFIGS["mixed"][0])
    change(d)
    with pytest.raises(ValueError, match=match):
        PupopelConfig.from_dict(d)


@pytest.mark.parametrize("change,match", [
    (lambda m: m["left"].update(heads=5), "multiple"),
    (lambda m: m["left"].update(scale=0.0), "positive"),
    (lambda m: m["right"].update(decay=[0.5]), "decay per head"),
])
def test_sizes_that_do_not_fit_are_refused(change, match):
    from vllm_omni_amd.pupopel import PupopelConfig, PupopelForCausalLM

    d = copy.deepcopy(pm.CONFIGS["mixed"][0])
    change(d["layers"][1]["mixer"])
    with pytest.raises(ValueError, match=match):
        PupopelForCausalLM(PupopelConfig.from_dict(d), torch.float32, "cpu")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", list(pm.CONFIGS))
def test_weights_map_one_to_one(name, dtype):
    """every checkpoint tensor has a place of its own in the fused products, and what is not written stays zero"""
    _, m, w = build(name, dtype)
    assert m.load_weights(w) == set(w)
    params = dict(m.named_weights())
    assert set(params) == set(w)
    for n, t in w.items():
        assert torch.equal(params[n].reshape(t.shape).float(), t.to(dtype).float()), n
    for layer in m.layers:
        for lin, names in ((layer.proj.inp, layer.proj.ins), (layer.proj.out, layer.proj.outs)):
            live = sum(int(t.count_nonzero()) for n, t in layer.proj.named_weights()
                       if (n in {x for b in layer.proj.ins for x in b.parts}) == (lin is layer.proj.inp))
            assert int(lin.weight.count_nonzero()) == live
    with pytest.raises(KeyError):
        m.load_weights({"l0.mix.nothing": torch.zeros(1)})
    with pytest.raises(ValueError):
        m.load_weights({"embed": torch.zeros(3, 3)})


def test_fused_products_equal_the_separate_ones():
    """the input product's views and the output product over padded heads are the layer's own products"""
    _, m, w = build("mixed")
    m.load_weights(w)
    layer = m.layers[1]
    h = torch.randn(5, 96)
    views = layer.proj.project(h)
    names = [n for b in layer.proj.ins for n in b.parts]
    got = torch.cat(views, 1)
    assert torch.allclose(got, torch.cat([h @ w[f"l1.{n}"].float().T for n in names], 1), atol=1e-5)
    buf, outs = layer.proj.buffers(5)
    assert all(o.data_ptr() % 16 == buf.data_ptr() % 16 for o in outs)
    want = torch.zeros(5, 96)
    for b, o in zip(layer.proj.outs, outs):
        o.view(5, b.groups, b.pitch).fill_(3.0)[..., :b.width] = torch.randn(5, b.groups, b.width)
        want += o.view(5, b.groups, b.pitch)[..., :b.width].flatten(1) @ w[f"l1.{b.name}"].float().T
    assert torch.allclose(layer.proj.out(buf), want, atol=1e-4)


def test_models_outside_the_envelope_say_so():
    from vllm_omni_amd.moe import RoutedExperts
    from vllm_omni_amd.pupopel import PupopelForCausalLM

    c, m, _ = build("odd")
    with pytest.raises(ValueError, match="bfloat16 or float32"):
        PupopelForCausalLM(c, torch.float16, "cpu")
    with pytest.raises(ValueError):
        m.quantize_int8()
    with pytest.raises(ValueError):
        RoutedExperts(64, 32, 17, 16, torch.float32)


def test_argument_validation_without_gpu():
    from vllm_omni_amd import _C

    lib = _C.lib
    buf = (ctypes.c_char * 4096)()
    p = (ctypes.addressof(buf) + 15) & ~15
    bad, no = _C.MI_ERR_INVALID_ARG, _C.MI_ERR_UNSUPPORTED
    assert lib.mi_residual_add_norm(p, None, 0, None, None, None, 0, p, 1.0, p, 0, 1e-6, 2, 8, 8, 8, 8, 0, 1, None) == bad
    assert lib.mi_residual_add_norm(p, p, 0, p, None, None, 2, p, 1.0, p, 0, 1e-6, 2, 8, 8, 8, 8, 8, 1, None) == bad     # experts without weights
    assert lib.mi_residual_add_norm(p, p, 0, None, None, None, 0, p, 1.0, p, 0, 1e-6, 2, 8, 8, 8, 8, 0, _C.MI_DTYPE_F16, None) == no
    assert lib.mi_embed_norm(p, p, p, p, p, 1.0, p, 1e-6, 2, 8, 10, 8, 8, 4, 1, None) == bad
    assert lib.mi_glu(p, p, p, 2, 8, 8, 8, 7, 1, None) == bad
    assert lib.mi_head_norm_cache(p, 100, p, p, p, 64, p, p, p, p, 2, 4, 2, 16, 16, 12, 16, 512, 32, 16, 0.0, 1, 1e-6, 1, None) == bad
    assert lib.mi_attn_rows(p, p, p, p, p, p, p, None, None, 1.0, 0, 2, 1, 3, 2, 16, 16, 1.0, 64, 64, 512, 32, 16, 4, 1, None) == bad
    dec = lambda hd, dt, bs=16: lib.mi_paged_attn_decode_biased(   # noqa: E731
        p, p, p, p, p, p, p, p, 1.0, 1, 4, 2, hd, bs, 4, 64, 1.0, 512, 512, 4096, 256, 128, 0, None, 0, dt, None)
    assert dec(32, 1) == no and dec(64, _C.MI_DTYPE_F16) == no and dec(64, 1, 8) == no
    la = {n: p for n, t in _C.LightningArgs._fields_ if t is ctypes.c_void_p}
    la.update(qkv_stride=400, gate_stride=400, out_stride=400, num_reqs=1, heads=2, dim=16, vdim=16, eps=1e-6, mul=1.0)
    call = lambda ws, **kw: lib.mi_lightning_attn(ctypes.byref(_C.LightningArgs(**{**la, **kw})), 0, 64, 64, 1, p, ws, 1, None)   # noqa: E731
    assert call(1 << 30, qkv_stride=90) == bad and call(1 << 30, dim=300, qkv_stride=2000) == no
    assert call(lib.mi_lightning_workspace_bytes(64, 1, 2, 16, 16, 1) - 1) == _C.MI_ERR_WORKSPACE
    assert lib.mi_lightning_workspace_bytes(64, 1, 2, 300, 16, 1) == 0
    assert lib.mi_moe_route(p, p, None, p, p, 2, 257, 257, 2, 1, 0, _C.MI_DTYPE_F32, -1, None) == no
    assert lib.mi_moe_pair_gemm(p, p, p, p, 4, 2, _C.MI_MOE_GATED, None, 8, 16, 2, 16, 8, 100, 1, None) == bad


# ------------------------------------------------------------------------------------------------ the restatement itself
def test_channel_rule_with_equal_channels_is_the_scalar_rule():
    from oracle import ref_dogulorn

    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(20, 2, n, generator=g, dtype=torch.float64) for n in (6, 6, 5))
    beta, dec = torch.rand(20, 2, generator=g, dtype=torch.float64), torch.rand(20, 2, generator=g, dtype=torch.float64)
    a, s = ref.channel_delta_rule(q, k, v, beta, dec[..., None].expand(20, 2, 6))
    b, t = ref_dogulorn.delta_rule(q, k, v, beta, dec)
    assert torch.allclose(a, b) and torch.allclose(s, t)


def test_attention_with_bias_and_sink_is_a_softmax_over_one_more_key():
    g = torch.Generator().manual_seed(1)
    q, k, v = torch.randn(9, 2, 4, generator=g), torch.randn(9, 1, 4, generator=g), torch.randn(9, 1, 3, generator=g)
    sink = torch.tensor([0.3, -1.0])
    got = ref.biased_sink_attention(q, k, v, 0.7, [0.5, 0.1], sink)
    for h in range(2):
        s = q[:, h] @ k[:, 0].T * 0.7 - [0.5, 0.1][h] * (torch.arange(9)[:, None] - torch.arange(9)[None])
        s = s.masked_fill(torch.triu(torch.ones(9, 9, dtype=torch.bool), 1), -math.inf)
        p = torch.softmax(torch.cat([s, sink[h].expand(9, 1)], 1), -1)[:, :9]
        assert torch.allclose(got[:, h], p @ v[:, 0], atol=1e-6)


def test_decayed_linear_attention_is_a_masked_product():
    g = torch.Generator().manual_seed(2)
    q, k, v = (torch.randn(12, 1, n, generator=g, dtype=torch.float64) for n in (5, 5, 4))
    d = torch.arange(12)[:, None] - torch.arange(12)[None]
    m = torch.where(d >= 0, torch.tensor(0.8, dtype=torch.float64) ** d.clamp(min=0), torch.zeros((), dtype=torch.float64))
    assert torch.allclose(ref.decayed_linear_attention(q, k, v, [0.8])[:, 0], (q[:, 0] @ k[:, 0].T * m) @ v[:, 0])


def test_first_tokens_of_the_temperature_and_the_convolution():
    t = ref.query_temperature(torch.arange(9, dtype=torch.float64), 0.5, 4)
    assert torch.allclose(t, 1 + 0.5 * torch.log(torch.tensor([1, 1, 1, 2, 2, 2, 2, 3, 3], dtype=torch.float64)))
    y = ref.short_conv(torch.ones(3, 1), torch.tensor([[100.0, 10.0, 1.0]]))
    assert y[:, 0].tolist() == [1.0, 11.0, 111.0]


def test_router_weighs_only_what_it_chose():
    h, w = torch.eye(3), torch.tensor([[1.0, 0, 0], [0.0, 2, 0], [3.0, 0, 0], [0.0, 0, 0]])
    idx, p = ref.route(h, w, torch.tensor([0.0, 0.0, 0.0, 0.5]), 2)
    assert idx[0].tolist() == [2, 0] and idx[1].tolist() == [1, 3] and idx[2].tolist()[0] == 3
    assert torch.allclose(p[0], torch.softmax(torch.tensor([3.0, 1.0]), 0))
