"""Small Dogulorn configurations and random weights for tests (no test reads a checkpoint)."""
import torch
import torch.overrides


def attn(heads, dim, vdim, q_rank, kv_rank, window, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "mask": {"size": window},
         "scale": scale if scale is not None else dim ** -0.5}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def model(layers, vocab=131, width=96, eps=1e-5, scale=2.5, buckets=97, mul_prev=31, mul_cur=5, side=16):
    out = []
    for layer, mlp in layers:
        out.append(dict(layer, mlp=None if mlp is None else {"kind": "dense", "ff": mlp[0], "limit": mlp[1]}))
    return {"architecture": "Dogulorn", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale, "bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}},
            "token_side": {"dim": side}, "layers": out}


CONFIGS = {
    # recurrent layer first and last, caches shared across a recurrent layer and between windows, feed-forwards missing on both kinds
    "mixed": model([(delta(6, 3, 24, 40, 3), (56, 0.7)), (attn(3, 24, 40, 48, 72, 5), None),
                    (attn(2, 16, 24, 32, 72, 9, 0.31, kv_from=1), (40, 1.3)), (delta(2, 1, 16, 48, 4), None),
                    (attn(5, 32, 8, 40, 24, 21), (64, 2.0)), (attn(5, 32, 8, 40, 72, 70, kv_from=1), (64, 2.0)),
                    (delta(4, 4, 32, 32, 2), (48, 1.1))]),
    # nothing a multiple of 8, one value head per key head, one tap
    "odd": model([(attn(3, 20, 27, 33, 35, 7), (77, 0.9)), (delta(3, 3, 18, 30, 2), (41, 1.0)), (delta(2, 1, 33, 21, 1), None),
                  (attn(1, 12, 10, 14, 35, 3, kv_from=0), None)], vocab=89, width=100, side=7),
    # more than 16 and more than 32 heads, one window longer than a tile, one of a single token
    "wide": model([(attn(36, 64, 64, 96, 128, 70), (128, 1.0)), (delta(4, 2, 64, 64, 4), None), (attn(20, 32, 64, 64, 128, 1, kv_from=0), None),
                   (attn(20, 64, 128, 64, 200, 300), (96, 0.5))], vocab=200, width=192),
}


def random_weights(cfg, seed=0, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    w, v = cfg["width"], cfg["vocab"]
    out = {}

    def mat(name, n, k, std=None):
        out[name] = (torch.randn(n, k, generator=g) * (std if std is not None else k ** -0.5)).to(dtype)

    def vec(name, n, mean=1.0, std=0.25):
        out[name] = (mean + std * torch.randn(n, generator=g)).to(dtype)

    mat("embed", v, w, 0.5)
    mat("bigram", cfg["embedding"]["bigram"]["buckets"] + 1, w, 0.5)
    sd = cfg["token_side"]["dim"]
    mat("side.embed", v, sd * len(cfg["layers"]), 1.0)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        vec(p + "norm1", w)
        vec(p + "norm1b", w)
        if layer["type"] == "delta":
            kd, hv = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for n, c in (("q", kd), ("k", kd), ("v", hv)):
                mat(p + f"mix.{n}", c, w)
                mat(p + f"mix.{n}.conv", c, m["conv"], 0.6)
            mat(p + "mix.b", m["heads"], w)
            mat(p + "mix.a", m["heads"], w)
            vec(p + "mix.A_log", m["heads"], -1.5, 0.7)
            vec(p + "mix.dt_bias", m["heads"], 0.0, 0.5)
            mat(p + "mix.g", hv, w)
            vec(p + "mix.norm", m["vdim"])
            mat(p + "mix.o", w, hv)
        else:
            mat(p + "mix.dq", m["q_rank"], w)
            vec(p + "mix.dq.norm", m["q_rank"])
            mat(p + "mix.uq", m["heads"] * m["dim"], m["q_rank"], 2.0 * m["q_rank"] ** -0.5)
            if "kv_from" not in m:
                mat(p + "mix.dkv", m["kv_rank"], w)
                vec(p + "mix.dkv.norm", m["kv_rank"])
            mat(p + "mix.uk", m["heads"] * m["dim"], m["kv_rank"], 2.0 * m["kv_rank"] ** -0.5)
            mat(p + "mix.uv", m["heads"] * m["vdim"], m["kv_rank"])
            mat(p + "mix.o", w, m["heads"] * m["vdim"])
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            vec(p + "norm2", w)
            vec(p + "norm2b", w)
            mat(p + "mlp.gate", ff, w)
            mat(p + "mlp.up", ff, w)
            mat(p + "mlp.down", w, ff)
        mat(p + "side.gate", sd, w)
        mat(p + "side.proj", w, sd)
        vec(p + "side.norm", w)
    vec("final.norm", w)
    mat("head", v, w)
    return out


def random_tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


class Bf16Products(torch.overrides.TorchFunctionMode):
    """matrix products with bf16 operand and result: what rounding alone does to the plain forward"""

    def __torch_function__(self, f, types, args=(), kwargs=None):
        if f in (torch.Tensor.matmul, torch.Tensor.__matmul__, torch.matmul):
            return f(args[0].bfloat16().double(), args[1]).bfloat16().double()
        return f(*args, **(kwargs or {}))


def row_error(got, want):
    """per row: rms of the difference, mean taken off, over the spread of ``want``"""
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.std()
