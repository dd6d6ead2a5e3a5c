"""Small Lifuzen configurations and random weights for tests (no test reads a checkpoint)."""
import torch

from dogulorn_models import Bf16Products, random_tokens, row_error  # noqa: F401  (shared by the test files)


def mamba(heads, groups, state, vdim, conv, norm_groups):
    return {"type": "mamba2", "mixer": {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": conv, "norm_groups": norm_groups}}


def attn(heads, kv_heads, dim, rot, conv, scale=None, base=1000.0):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "conv": conv,
                                           "scale": dim ** -0.5 if scale is None else scale, "rot": {"base": base, "dims": rot}}}


def moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def model(layers, loop, vocab=131, width=96, eps=1e-5, mult=0.6, cap=6.0):
    return {"architecture": "Lifuzen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "logit_softcap": cap,
            "layers": [dict(m, mlp=mlp) for m, mlp in layers],
            "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]} if loop else None}


CONFIGS = {
    # a loop in the middle that starts with either kind, layers without feed-forward of either kind, heads and groups unequal
    "mixed": model([(attn(6, 2, 48, 20, 4), moe(6, 2, 40)), (mamba(6, 2, 24, 40, 4, 3), None), (attn(4, 4, 64, 64, 3, 0.3, 77.0), None),
                    (mamba(4, 1, 40, 64, 3, 4), moe(9, 3, 24)), (mamba(2, 2, 64, 16, 4, 1), moe(4, 4, 56))], (1, 4, 3)),
    # nothing a multiple of 8, everything in the loop, one tap and two, one expert chosen
    "odd": model([(attn(3, 1, 21, 6, 2), moe(5, 1, 21)), (mamba(3, 3, 19, 13, 1, 1), moe(7, 2, 33)), (mamba(5, 1, 33, 21, 2, 5), None)], (0, 3, 2),
                 vocab=89, width=100, mult=1.0, cap=2.5),
    # a real layer's head sizes, the loop at the end and once only, many experts, parts of the norm that cross heads
    "wide": model([(mamba(8, 2, 128, 64, 4, 2), moe(40, 4, 64)), (attn(16, 2, 128, 64, 4, base=20000.0), moe(8, 8, 128)),
                   (mamba(4, 2, 64, 128, 4, 8), moe(16, 2, 128)), (attn(8, 8, 64, 16, 4), None)], (2, 4, 1), vocab=200, width=256, mult=0.4),
    # heads past the matrix-core attention's sizes, long filters, a state of many rows, a loop over the first layer
    "tall": model([(mamba(3, 1, 200, 80, 6, 1), moe(3, 2, 64)), (attn(2, 1, 160, 160, 6), moe(4, 1, 48)), (mamba(1, 1, 72, 144, 4, 2), None)],
                  (0, 1, 3), vocab=70, width=128, mult=0.9, cap=15.0),
    # no loop at all
    "flat": model([(mamba(4, 4, 32, 32, 4, 4), None), (attn(5, 5, 32, 2, 4), moe(6, 3, 32))], None, vocab=64, width=72),
}


def random_weights(cfg, seed=0, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    w, v = cfg["width"], cfg["vocab"]
    out = {}

    def mat(name, n, k, std=None):
        out[name] = (torch.randn(n, k, generator=g) * (std if std is not None else k ** -0.5)).to(dtype)

    def vec(name, n, mean=1.0, std=0.25):
        out[name] = (mean + std * torch.randn(n, generator=g)).to(dtype)

    mat("embed", v, w, 1.0)
    if cfg["loop"]:
        mat("loop.step", cfg["loop"]["times"], w, 0.7)
    for i, entry in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", entry["mixer"], entry["mlp"]
        vec(p + "norm1", w, 0.0)
        if entry["type"] == "mamba2":
            inner, ch = m["heads"] * m["vdim"], m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
            mat(p + "mix.in", inner + ch + m["heads"], w)
            mat(p + "mix.conv", ch, m["conv"], 0.7)
            vec(p + "mix.conv.b", ch, 0.0, 0.3)
            vec(p + "mix.dt_bias", m["heads"], -2.0, 1.0)
            vec(p + "mix.A_log", m["heads"], -0.5, 1.2)
            vec(p + "mix.D", m["heads"], 1.0, 0.5)
            vec(p + "mix.norm", inner)
            mat(p + "mix.o", w, inner)
        else:
            nq, nk = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
            mat(p + "mix.q", nq, w)
            mat(p + "mix.k", nk, w)
            mat(p + "mix.q.conv", nq, m["conv"], 0.7)
            mat(p + "mix.k.conv", nk, m["conv"], 0.7)
            mat(p + "mix.o", w, nq)
        if mlp:
            vec(p + "norm2", w, 0.0)
            mat(p + "mlp.router", mlp["router"]["experts"], w, 2.0 * w ** -0.5)
            for e in range(mlp["router"]["experts"]):
                mat(f"{p}mlp.e{e}.up", mlp["expert"]["ff"], w, 1.5 * w ** -0.5)
                mat(f"{p}mlp.e{e}.down", w, mlp["expert"]["ff"], 1.5 * mlp["expert"]["ff"] ** -0.5)
    vec("final.norm", w, 0.0)
    return out


def steady(weights):
    """the same weights with routers that leave no close calls: every row carries a large constant in its first column, and each
    expert weighs that column differently, so that rounding cannot turn a choice; the logits do not see the column"""
    out = dict(weights)
    out["embed"] = weights["embed"].clone()
    out["embed"][:, 0] = 6.0
    out["final.norm"] = weights["final.norm"].clone()
    out["final.norm"][0] = -1.0
    for k, v in weights.items():
        if k.endswith(("norm1", "norm2")):
            out[k] = v.clone()
            out[k][0] = 0.0
        elif k.endswith("mlp.router"):
            r = v * 0.05
            r[:, 0] = torch.linspace(-1.0, 0.6, v.shape[0])[torch.randperm(v.shape[0], generator=torch.Generator().manual_seed(v.shape[0]))]
            out[k] = r
        elif k.endswith((".o", ".down")):
            out[k] = v.clone()
            out[k][0] = 0.0          # nothing is added to the column
        elif k == "loop.step":
            out[k] = v.clone()
            out[k][:, 0] = 0.0
    return out
