"""Plain restatement of the Dogulorn decoder: one function per mechanism, one token at a time where a recurrence or a
window makes that the clearest form, in float64 unless told otherwise.  Test infrastructure only; shares nothing with
the product path.

Notation: ``x`` is the residual stream of ONE sequence, [T, width]; weights are [out, in].
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return rms(x, eps) * w


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.log1p(torch.exp(-x.abs())) + x.clamp(min=0)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def embed(tokens, table, bigram, scale, mul_prev, mul_cur):
    """scaled token row + the row of the (previous, current) pair; the first token of a sequence takes the extra last row"""
    buckets = bigram.shape[0] - 1
    rows = []
    for i, t in enumerate(tokens):
        r = buckets if i == 0 else (int(tokens[i - 1]) * mul_prev + int(t) * mul_cur) % buckets
        rows.append(table[int(t)] * scale + bigram[r])
    return torch.stack(rows)


def causal_conv(x, w):
    """per-channel taps over time; the last column meets the current token; zeros before the start"""
    T, C = x.shape
    taps = w.shape[1]
    y = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] += w[:, j] * x[s]
    return y


def delta_rule(q, k, v, beta, g):
    """q, k [T, H, D], v [T, H, V], beta, g [T, H] -> read-outs [T, H, V] and the final state [H, D, V]"""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        S = S * g[t][:, None, None]
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def delta_mixer(h, w, m, eps):
    """``w(name)``: the layer's mixer tensors; ``m``: its sizes"""
    T = h.shape[0]
    H, K, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(causal_conv(h @ w("q").T, w("q.conv"))).view(T, K, D)
    k = silu(causal_conv(h @ w("k").T, w("k.conv"))).view(T, K, D)
    v = silu(causal_conv(h @ w("v").T, w("v.conv"))).view(T, H, V)
    q = unit(q) * D ** -0.5
    k = unit(k)
    of = [i // (H // K) for i in range(H)]
    beta = sigmoid(h @ w("b").T)
    g = torch.exp(-torch.exp(w("A_log")) * softplus(h @ w("a").T + w("dt_bias")))
    o, _ = delta_rule(q[:, of], k[:, of], v, beta, g)
    o = rms(o, eps) * w("norm") * silu(h @ w("g").T).view(T, H, V)
    return o.reshape(T, H * V) @ w("o").T


def latent(h, w, eps):
    return rms_norm(h @ w("dkv").T, w("dkv.norm"), eps)


def window_attention(q, k, v, scale, size):
    """q, k [T, H, D], v [T, H, V]; position i sees the ``size`` positions that end at i"""
    T = q.shape[0]
    out = torch.zeros_like(v)
    for i in range(T):
        j0 = max(0, i - size + 1)
        s = (q[i][None] * k[j0:i + 1]).sum(-1) * scale
        p = torch.exp(s - s.max(0).values)
        p = p / p.sum(0)
        out[i] = (p[:, :, None] * v[j0:i + 1]).sum(0)
    return out


def latent_attention_mixer(h, c, w, m, eps):
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    cq = rms_norm(h @ w("dq").T, w("dq.norm"), eps)
    q = (cq @ w("uq").T).view(T, H, D)
    k = (c @ w("uk").T).view(T, H, D)
    v = (c @ w("uv").T).view(T, H, V)
    o = window_attention(q, k, v, m["scale"], m["mask"]["size"])
    return o.reshape(T, H * V) @ w("o").T


def clamped_mlp(h, gate, up, down, limit):
    g = (h @ gate.T).clamp(max=limit)
    u = (h @ up.T).clamp(-limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def side_input(x, e, gate, proj, norm, eps):
    return rms_norm((gelu_tanh(x @ gate.T) * e) @ proj.T, norm, eps)


def forward(cfg, weights, tokens, dtype=torch.float64):
    """logits [T, vocab] and the residual stream after every layer, a list of [T, width]"""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    bg = cfg["embedding"]["bigram"]
    x = embed(tokens, W["embed"], W["bigram"], cfg["embedding"]["scale"], bg["mul_prev"], bg["mul_cur"])
    sd = cfg["token_side"]["dim"]
    side = W["side.embed"][torch.as_tensor(tokens, dtype=torch.int64)]
    streams, latents = [], {}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        w = lambda n, p=p: W[p + "mix." + n]   # noqa: E731
        m = layer["mixer"]
        h = rms_norm(x, W[p + "norm1"], eps)
        if layer["type"] == "delta":
            y = delta_mixer(h, w, m, eps)
        else:
            j = m.get("kv_from")
            if j is None:
                latents[i] = latent(h, w, eps)
            y = latent_attention_mixer(h, latents[i if j is None else j], w, m, eps)
        x = x + rms_norm(y, W[p + "norm1b"], eps)
        if layer["mlp"] is not None:
            h = rms_norm(x, W[p + "norm2"], eps)
            y = clamped_mlp(h, W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"], layer["mlp"]["limit"])
            x = x + rms_norm(y, W[p + "norm2b"], eps)
        x = x + side_input(x, side[:, i * sd:(i + 1) * sd], W[p + "side.gate"], W[p + "side.proj"], W[p + "side.norm"], eps)
        streams.append(x)
    return rms_norm(x, W["final.norm"], eps) @ W["head"].T, streams
