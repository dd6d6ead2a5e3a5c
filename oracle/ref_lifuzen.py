"""Plain restatement of the Lifuzen decoder: one function per mechanism, one token at a time wherever a recurrence makes
that the clearest form, in float64 unless told otherwise.  Test infrastructure only; shares nothing with the product
path.

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


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.log1p(torch.exp(-x.abs())) + x.clamp(min=0)


def relu_squared(z):
    return z.clamp(min=0) ** 2


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def short_conv(x, w):
    """per-channel taps over time; the last column meets the current token; zeros before the start"""
    y = torch.zeros_like(x)
    taps = w.shape[1]
    for t in range(x.shape[0]):
        for back in range(min(taps, t + 1)):
            y[t] += w[:, taps - 1 - back] * x[t - back]
    return y


# ------------------------------------------------------------------------------------------ state-space recurrence
def step_sizes(raw, bias):
    return softplus(raw + bias)


def state_space(x, B, C, dt, a_log, D):
    """x [T, H, V], B and C [T, G, N], dt [T, H] -> read-outs [T, H, V] and the final state [H, N, V]"""
    T, H, V = x.shape
    of = torch.arange(H) // (H // B.shape[1])
    S = torch.zeros(H, B.shape[2], V, dtype=x.dtype)
    y = torch.zeros_like(x)
    rate = torch.exp(a_log)
    for t in range(T):
        keep = torch.exp(-rate * dt[t])
        for h in range(H):
            S[h] = keep[h] * S[h] + dt[t, h] * torch.outer(B[t, of[h]], x[t, h])
            y[t, h] = S[h].T @ C[t, of[h]] + D[h] * x[t, h]
    return y, S


def gated_group_norm(y, z, w, groups, eps):
    """y, z [T, inner]: gate first, then the norm of each of ``groups`` equal parts"""
    g = y * silu(z)
    return rms(g.view(g.shape[0], groups, -1), eps).reshape(g.shape) * w


def mamba_mixer(h, w, m, eps):
    """``w(name)``: the mixer's tensors; ``m``: its sizes"""
    T, H, V, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * V
    z, xbc, raw = (h @ w("in").T).split([inner, inner + 2 * G * N, H], dim=1)
    xbc = silu(short_conv(xbc, w("conv")) + w("conv.b"))
    x, B, C = xbc.split([inner, G * N, G * N], dim=1)
    y, _ = state_space(x.reshape(T, H, V), B.reshape(T, G, N), C.reshape(T, G, N), step_sizes(raw, w("dt_bias")), w("A_log"), w("D"))
    return gated_group_norm(y.reshape(T, inner), z, w("norm"), m["norm_groups"], eps) @ w("o").T


# ------------------------------------------------------------------------------------------ attention whose values are its keys
def rotate(x, dims, base, first=0):
    """x [T, heads, D], positions from ``first`` on: neighbours 2i, 2i + 1 of the first ``dims`` turned by position * base^(-2i / dims)"""
    out = x.clone()
    for i in range(dims // 2):
        a = torch.arange(first, first + x.shape[0], dtype=x.dtype)[:, None] * (float(base) ** (-2.0 * i / dims))
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        out[:, :, 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return out


def sink_attention(q, k, v, scale):
    """q [T, H, D], k [T, G, D], v [T, G, V]; causal; a score of zero without a value takes part in the softmax"""
    T, H, _ = q.shape
    per = H // k.shape[1]
    future = torch.arange(T)[None, :] > torch.arange(T)[:, None]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        s = ((q[:, h] @ k[:, h // per].T) * scale).masked_fill(future, float("-inf"))
        top = s.max(-1, keepdim=True).values.clamp(min=0)
        e = torch.exp(s - top)
        out[:, h] = (e @ v[:, h // per]) / (torch.exp(-top) + e.sum(-1, keepdim=True))
    return out


def attention_mixer(h, w, m, eps):
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = short_conv(h @ w("q").T, w("q.conv")).view(T, H, D)
    v = short_conv(h @ w("k").T, w("k.conv")).view(T, G, D)
    dims, base = m["rot"]["dims"], m["rot"]["base"]
    q, k = rms(rotate(q, dims, base), eps), rms(rotate(v, dims, base), eps)
    return sink_attention(q, k, v, m["scale"]).reshape(T, H * D) @ w("o").T


# ------------------------------------------------------------------------------------------ routed experts
def route(h, router, top):
    """-> the chosen experts' numbers and scores, [T, top] each"""
    s = sigmoid(h @ router.T)
    order = torch.argsort(s, dim=-1, descending=True, stable=True)[:, :top]
    return order, torch.gather(s, 1, order)


def routed_experts(h, w, top):
    """the weight scales what an expert reads"""
    ids, weights = route(h, w("router"), top)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(top):
            e = int(ids[t, j])
            x = (h[t] * weights[t, j])[None]
            out[t] += (relu_squared(x @ w(f"e{e}.up").T) @ w(f"e{e}.down").T)[0]
    return out


# ------------------------------------------------------------------------------------------ the model
def layer_runs(cfg):
    """[(layer, pass it starts or None)] in the order the layers run"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return ([(i, None) for i in range(a)] + [(i, t if i == a else None) for t in range(loop["times"]) for i in range(a, b)]
            + [(i, None) for i in range(b, n)])


MIXERS = {"mamba2": mamba_mixer, "attention": attention_mixer}


def layer(x, W, p, entry, eps, mult):
    y = MIXERS[entry["type"]](norm_about_one(x, W[p + "norm1"], eps), lambda n: W[p + "mix." + n], entry["mixer"], eps)
    if entry.get("mlp") is not None:
        y = y + routed_experts(norm_about_one(x, W[p + "norm2"], eps), lambda n: W[p + "mlp." + n], entry["mlp"]["router"]["top"])
    return x + mult * y


def forward(cfg, weights, tokens, dtype=torch.float64):
    """logits [T, vocab] and the residual stream after every layer run, a list of [T, width]"""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    first = W["embed"][torch.as_tensor(tokens, dtype=torch.int64)]
    x, streams = first, []
    for i, start in layer_runs(cfg):
        if start is not None:
            x = x + (first if start > 0 else 0) + W["loop.step"][start]
        x = layer(x, W, f"l{i}.", cfg["layers"][i], eps, cfg["residual_mult"])
        streams.append(x)
    logits = norm_about_one(x, W["final.norm"], eps) @ W["embed"].T
    return soft_cap(logits, cfg["logit_softcap"]), streams
