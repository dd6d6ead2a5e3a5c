"""Small Pupopel configurations and random weights for tests (no test reads a checkpoint)."""
import torch

from dogulorn_models import Bf16Products, random_tokens, row_error  # noqa: F401  (shared by the test files)


def delta(heads, kv_heads, dim, vdim, conv, ranks=(8, 8)):
    """ranks: of the decay's and the gate's low-rank products; the configuration file does not have them"""
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}, ranks


def left(heads, kv_heads, dim, vdim, coef, every, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5,
            "q_temp": {"coef": coef, "every": every}}


def right(heads, dim, vdim, decay):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}


def parallel(a, r, left_scale, right_scale):
    return {"type": "parallel", "mixer": {"left": a, "right": r, "left_scale": left_scale, "right_scale": right_scale}}, None


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared}}


def model(layers, loop, vocab=131, width=96, eps=1e-5):
    """-> (configuration, ranks of the delta layers)"""
    entries = [dict(mixer, mlp=mlp) for (mixer, _), mlp in layers]
    return {"architecture": "Pupopel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": entries,
            "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]}}, [r for (_, r), _ in layers]


CONFIGS = {
    # a loop over both kinds of layers in the middle, every feed-forward kind and none, unequal sizes everywhere
    "mixed": model([(delta(4, 2, 24, 40, 3, (16, 12)), dense(72)),
                    (parallel(left(6, 2, 48, 40, 0.4, 7), right(3, 24, 32, [0.5, 0.9, 0.999]), 0.7, 1.3), moe(6, 2, 40, 56)),
                    (delta(3, 1, 32, 16, 4), None),
                    (parallel(left(4, 4, 64, 64, 0.2, 50, 0.2), right(2, 40, 24, [0.8, 1.0]), 1.0, 0.4), None),
                    (delta(2, 2, 16, 48, 2), moe(9, 3, 24, 32))], (1, 4, 2)),
    # nothing a multiple of 8, the loop over the whole model, one expert chosen, one tap
    "odd": model([(parallel(left(3, 1, 21, 35, 0.3, 5), right(2, 19, 13, [0.6, 0.97]), 1.1, 0.9), dense(77)),
                  (delta(3, 3, 18, 30, 1, (7, 5)), moe(5, 1, 21, 19)),
                  (delta(2, 1, 33, 21, 6, (3, 9)), dense(41))], (0, 3, 2), vocab=89, width=100),
    # a real layer's head sizes, the loop at the end and once only, a first layer in front of it, many experts
    "wide": model([(delta(4, 4, 64, 64, 4, (32, 16)), moe(40, 4, 64, 128)),
                   (parallel(left(16, 2, 128, 128, 0.1, 64), right(4, 128, 64, [0.3, 0.9, 0.99, 0.9995]), 0.6, 0.8), dense(128)),
                   (parallel(left(8, 1, 64, 128, 0.5, 1), right(2, 64, 128, [0.95, 0.7]), 0.5, 0.5), moe(8, 8, 128, 64))], (1, 3, 1),
                  vocab=200, width=256),
    # heads beyond the matrix-core attention's sizes, a loop over the first layer
    "tall": model([(parallel(left(2, 2, 160, 96, 0.3, 9), right(1, 136, 200, [0.98]), 0.9, 0.7), dense(64)),
                   (delta(2, 1, 136, 72, 4, (24, 24)), dense(48))], (0, 1, 3), vocab=70, width=128),
}


def random_weights(cfg, ranks, seed=0, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    w, v = cfg["width"], cfg["vocab"]
    out = {}

    def mat(name, n, k, std=None):
        out[name] = (torch.randn(n, k, generator=g) * (std if std is not None else k ** -0.5)).to(dtype)

    def vec(name, n, mean=1.0, std=0.25):
        out[name] = (mean + std * torch.randn(n, generator=g)).to(dtype)

    def glu(p, ff):
        mat(p + "gate", ff, w)
        mat(p + "up", ff, w)
        mat(p + "down", w, ff)

    mat("embed", v, w, 1.0)
    mat("loop.in", w, 2 * w)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        vec(p + "norm1", w, 0.0)
        if layer["type"] == "channel_delta":
            kd, hd, hv = m["kv_heads"] * m["dim"], m["heads"] * m["dim"], m["heads"] * m["vdim"]
            for n, c in (("q", kd), ("k", kd), ("v", hv)):
                mat(p + f"mix.{n}", c, w)
                mat(p + f"mix.{n}.conv", c, m["conv"], 0.6)
            mat(p + "mix.b", m["heads"], w)
            ra, rg = ranks[i]
            mat(p + "mix.a1", ra, w)
            mat(p + "mix.a2", hd, ra)
            mat(p + "mix.g1", rg, w)
            mat(p + "mix.g2", hv, rg)
            vec(p + "mix.A_log", m["heads"], -1.5, 0.9)
            vec(p + "mix.dt_bias", hd, 0.0, 0.8)
            vec(p + "mix.norm", m["vdim"])
            mat(p + "mix.o", w, hv)
        else:
            a, r = m["left"], m["right"]
            mat(p + "mix.left.q", a["heads"] * a["dim"], w)
            mat(p + "mix.left.k", a["kv_heads"] * a["dim"], w)
            mat(p + "mix.left.v", a["kv_heads"] * a["vdim"], w)
            vec(p + "mix.left.q.norm", a["dim"], 1.5)
            vec(p + "mix.left.k.norm", a["dim"])
            vec(p + "mix.left.sink", a["heads"], 0.5, 1.0)
            mat(p + "mix.left.o", w, a["heads"] * a["vdim"])
            hd, hv = r["heads"] * r["dim"], r["heads"] * r["vdim"]
            for n, c in (("q", hd), ("k", hd), ("v", hv), ("g", hv)):
                mat(p + "mix.right." + n, c, w)
            vec(p + "mix.right.norm", hv)
            mat(p + "mix.right.o", w, hv)
        mlp = layer["mlp"]
        if mlp and mlp["kind"] == "dense":
            glu(p + "mlp.", mlp["ff"])
        elif mlp:
            for e in range(mlp["router"]["experts"]):
                glu(f"{p}mlp.e{e}.", mlp["expert"]["ff"])
            mat(p + "mlp.router", mlp["router"]["experts"], w, 4.0 * w ** -0.5)
            vec(p + "mlp.router.b", mlp["router"]["experts"], 0.0, 0.5)
            glu(p + "mlp.shared.", mlp["shared"]["ff"])
    vec("final.norm", w, 0.0)
    mat("head", v, w)
    return out
