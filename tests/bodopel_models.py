"""Small Bodopel configurations and random weights for tests (no test reads a checkpoint)."""
import torch

from dogulorn_models import Bf16Products, random_tokens, row_error  # noqa: F401  (shared by the test files)


def layer(heads, kv_heads, dim, vdim, window, ff, softcap=20.0, scale=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window},
                                           "scale": dim ** -0.5 if scale is None else scale, "softcap": softcap},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model(layers, loop, vocab=131, width=96, eps=1e-5, taps=4, scale=3.0, positions=512):
    return {"architecture": "Bodopel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "canon": {"taps": taps}, "max_positions": positions, "layers": layers,
            "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]}}


CONFIGS = {
    # a loop in the middle, windows of different sizes (one of them a page, one longer than the prompt), a layer without feed-forward
    "mixed": model([layer(8, 2, 40, 64, 16, 120), layer(6, 3, 64, 24, 37, 0, softcap=4.0), layer(4, 4, 32, 32, 300, 64, scale=0.3),
                    layer(10, 2, 48, 56, 70, 88)], (1, 3, 3)),
    # nothing a multiple of 8, everything in the loop, one token of window, two taps
    "odd": model([layer(3, 1, 21, 35, 1, 77), layer(5, 5, 33, 19, 50, 41, softcap=2.5)], (0, 2, 2), vocab=89, width=100, taps=2, scale=0.7),
    # a real layer's head sizes, the loop over the last layers and once only, a filter longer than the kernels hold in registers
    "wide": model([layer(16, 4, 128, 128, 64, 256), layer(32, 8, 64, 64, 33, 128), layer(12, 4, 96, 128, 129, 0),
                   layer(40, 8, 64, 48, 90, 256)], (2, 4, 1), vocab=200, width=256, taps=7),
    # heads past the matrix-core kernels' sizes, one tap (no state besides the caches), a loop over the first layer
    "tall": model([layer(2, 1, 160, 96, 45, 64), layer(36, 12, 128, 40, 20, 48)], (0, 1, 3), vocab=70, width=128, taps=1, scale=1.0),
}


def random_weights(cfg, seed=0, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    w, v, taps = cfg["width"], cfg["vocab"], cfg["canon"]["taps"]
    out = {}

    def mat(name, n, k, std=None):
        out[name] = (torch.randn(n, k, generator=g) * (std if std is not None else k ** -0.5)).to(dtype)

    def vec(name, n, mean=1.0, std=0.25):
        out[name] = (mean + std * torch.randn(n, generator=g)).to(dtype)

    mat("embed", v, w, 1.0)
    mat("pos", cfg["max_positions"], w, 0.5)
    if cfg["loop"]:
        mat("loop.step", cfg["loop"]["times"], w, 1.0)
    for i, entry in enumerate(cfg["layers"]):
        p, m = f"l{i}.", entry["mixer"]
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        vec(p + "norm1", w, 0.0)
        mat(p + "canon1", w, taps, 0.5)
        for n, rows in (("q", H * D), ("k", G * D), ("v", G * V)):
            mat(p + "mix." + n, rows, w)
            vec(p + f"mix.{n}.b", rows, 0.0, 0.3)
        vec(p + "mix.q.norm", H * D, 1.4)
        vec(p + "mix.k.norm", G * D)
        out[p + "mix.r1"] = (0.2 + torch.rand(H, generator=g)).to(dtype)
        out[p + "mix.r2"] = (0.05 + 2 * torch.rand(H, generator=g)).to(dtype)
        out[p + "mix.talk"] = (torch.eye(H) + torch.randn(H, H, generator=g) * 0.5 * H ** -0.5).to(dtype)
        mat(p + "mix.g", H * V, w)
        mat(p + "mix.o", w, H * V)
        if entry["mlp"]:
            vec(p + "norm2", w, 0.0)
            mat(p + "canon2", w, taps, 0.5)
            mat(p + "mlp.up", entry["mlp"]["ff"], w)
            mat(p + "mlp.down", w, entry["mlp"]["ff"])
    vec("final.norm", w, 0.0)
    mat("head", v, w)
    return out
