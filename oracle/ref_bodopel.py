"""Plain restatement of the Bodopel decoder: one function per mechanism, loops where they make the equation plainest, in
float64 unless told otherwise.  Test infrastructure only; shares nothing with the product path.

Notation: ``x`` is the residual stream of ONE sequence, [T, width]; weights are [out, in].
"""
from __future__ import annotations

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_about_one(x, w, eps):
    """RMS norm whose weight is kept as its distance from one"""
    return rms(x, eps) * (1.0 + w)


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def relu_squared(z):
    return z.clamp(min=0) ** 2


# ------------------------------------------------------------------------------------------ the short convolution in front
def causal_conv(h, w):
    """a filter per channel over time; its last column meets the current row; zeros before the start"""
    y = torch.zeros_like(h)
    taps = w.shape[1]
    for t in range(h.shape[0]):
        for back in range(min(taps, t + 1)):
            y[t] += w[:, taps - 1 - back] * h[t - back]
    return y


def with_conv(h, w):
    return h + causal_conv(h, w)


# ------------------------------------------------------------------------------------------ attention with mixed heads
def soft_cap(s, cap):
    return s if cap is None else cap * torch.tanh(s / cap)


def log_distance(r1, r2, d):
    return r1 * torch.log(1.0 + r2 * d)


def head_weights(q, k, scale, cap, r1, r2, window):
    """q [T, H, D], k [T, G, D] -> every head's softmax weights [H, T, T], zero where a key is not visible"""
    T, H, _ = q.shape
    per = H // k.shape[1]
    d = (torch.arange(T)[:, None] - torch.arange(T)[None]).to(q.dtype)
    seen = (d >= 0) if window is None else (d >= 0) & (d < window)
    out = torch.zeros(H, T, T, dtype=q.dtype)
    for h in range(H):
        s = soft_cap((q[:, h] @ k[:, h // per].T) * scale, cap) - log_distance(r1[h], r2[h], d.clamp(min=0))
        s = s.masked_fill(~seen, float("-inf"))
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        out[h] = e / e.sum(-1, keepdim=True)
    return out


def mix_heads(p, talk):
    """[H, T, T] -> weights of head h = sum over heads g of talk[h, g] p[g]"""
    return torch.einsum("hg,gij->hij", talk, p)


def apply_weights(p, v):
    """p [H, T, T], v [T, G, V] -> [T, H, V]"""
    per = p.shape[0] // v.shape[1]
    return torch.stack([p[h] @ v[:, h // per] for h in range(p.shape[0])], dim=1)


def talking_attention(q, k, v, scale, cap, r1, r2, window, talk):
    return apply_weights(mix_heads(head_weights(q, k, scale, cap, r1, r2, window), talk), v)


def attention_mixer(h, w, m, eps):
    """``w(name)``: the mixer's tensors; ``m``: its sizes"""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (h @ w(n).T + w(n + ".b") for n in ("q", "k", "v"))
    q = rms(q, eps) * w("q.norm")
    k = rms(k, eps) * w("k.norm")
    o = talking_attention(q.view(T, H, D), k.view(T, G, D), v.view(T, G, V), m["scale"], m.get("softcap"), w("r1"), w("r2"),
                          m["mask"]["size"] if m.get("mask") else None, w("talk"))
    return (o.reshape(T, H * V) * sigmoid(h @ w("g").T)) @ w("o").T


def dense_feed_forward(h, w):
    return relu_squared(h @ w("up").T) @ w("down").T


# ------------------------------------------------------------------------------------------ the model
def layer_runs(cfg):
    """[(layer, pass it starts or None)] in the order the layers run"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return ([(i, None) for i in range(a)] + [(i, t if i == a else None) for t in range(loop["times"]) for i in range(a, b)]
            + [(i, None) for i in range(b, n)])


def embed(tokens, W, cfg):
    ids = torch.as_tensor(tokens, dtype=torch.int64)
    return W["embed"][ids] * cfg["embedding"]["scale"] + W["pos"][:len(tokens)]


def layer(x, W, p, entry, eps):
    h = with_conv(norm_about_one(x, W[p + "norm1"], eps), W[p + "canon1"])
    x = x + attention_mixer(h, lambda n: W[p + "mix." + n], entry["mixer"], eps)
    if entry.get("mlp") is not None:
        h = with_conv(norm_about_one(x, W[p + "norm2"], eps), W[p + "canon2"])
        x = x + dense_feed_forward(h, lambda n: W[p + "mlp." + n])
    return x


def forward(cfg, weights, tokens, dtype=torch.float64):
    """logits [T, vocab] and the residual stream after every layer run, a list of [T, width]"""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = embed(tokens, W, cfg)
    streams = []
    for i, start in layer_runs(cfg):
        if start is not None:
            x = x + W["loop.step"][start]
        x = layer(x, W, f"l{i}.", cfg["layers"][i], eps)
        streams.append(x)
    return norm_about_one(x, W["final.norm"], eps) @ W["head"].T, streams
