"""Plain restatement of the Pupopel decoder: one function per mechanism, one token at a time wherever a recurrence makes
that the clearest form, in float64 unless told otherwise.  Test infrastructure only; shares nothing with the product
path.

Notation: ``x`` is the residual stream of ONE sequence, [T, width]; weights are [out, in].
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_about_one(x, w, eps):
    """RMS norm whose weight is kept as its distance from one"""
    return rms(x, eps) * (1.0 + w)


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


# ------------------------------------------------------------------------------------------ channel-wise gated delta rule
def short_conv(x, w):
    """per-channel taps over time; the last column meets the current token; zeros before the start"""
    y = torch.zeros_like(x)
    taps = w.shape[1]
    for t in range(x.shape[0]):
        for back in range(min(taps, t + 1)):
            y[t] += w[:, taps - 1 - back] * x[t - back]
    return y


def channel_decay(low, dt_bias, a_log, heads, dim):
    """low [T, heads * dim] -> decay per token, head and key channel"""
    rate = torch.exp(a_log)[None, :, None]
    return torch.exp(-rate * softplus(low + dt_bias).view(-1, heads, dim))


def channel_delta_rule(q, k, v, beta, g):
    """q, k, g [T, H, D], v [T, H, V], beta [T, H] -> read-outs [T, H, V] and the final state [H, D, V]"""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        S = S * g[t].unsqueeze(-1)
        seen = torch.einsum("hd,hdv->hv", k[t], S)
        u = beta[t].unsqueeze(-1) * (v[t] - seen)
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(1)
        out[t] = torch.einsum("hd,hdv->hv", q[t], S)
    return out, S


def channel_delta_mixer(h, w, m, eps):
    """``w(name)``: the mixer's tensors; ``m``: its sizes"""
    T = h.shape[0]
    H, K, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(h @ w(n).T, w(n + ".conv"))) for n in ("q", "k", "v"))
    q = unit(q.view(T, K, D)) / math.sqrt(D)
    k = unit(k.view(T, K, D))
    of = torch.arange(H) // (H // K)
    g = channel_decay((h @ w("a1").T) @ w("a2").T, w("dt_bias"), w("A_log"), H, D)
    o, _ = channel_delta_rule(q[:, of], k[:, of], v.view(T, H, V), sigmoid(h @ w("b").T), g)
    gate = sigmoid((h @ w("g1").T) @ w("g2").T).view(T, H, V)
    return (rms(o, eps) * w("norm") * gate).reshape(T, H * V) @ w("o").T


# ------------------------------------------------------------------------------------------ attention with a distance bias
def query_temperature(positions, coef, every):
    return 1.0 + coef * torch.log(torch.div(positions + 1, every, rounding_mode="floor") + 1.0)


def head_slopes(H):
    return [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]


def biased_sink_attention(q, k, v, scale, slopes, sink):
    """q [T, H, D], k [T, G, D], v [T, G, V]; causal; the sink is one more term of the denominator only"""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        for i in range(T):
            dist = i - torch.arange(i + 1, dtype=q.dtype)
            s = (k[:i + 1, h // per] @ q[i, h]) * scale - slopes[h] * dist
            top = torch.maximum(s.max(), sink[h])
            e = torch.exp(s - top)
            out[i, h] = (e @ v[:i + 1, h // per]) / (e.sum() + torch.exp(sink[h] - top))
    return out


def sink_attention_mixer(h, w, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ w("q").T).view(T, H, D), eps) * w("q.norm")
    k = rms((h @ w("k").T).view(T, G, D), eps) * w("k.norm")
    v = (h @ w("v").T).view(T, G, V)
    temp = query_temperature(torch.arange(T, dtype=h.dtype), m["q_temp"]["coef"], m["q_temp"]["every"])
    o = biased_sink_attention(q * temp[:, None, None], k, v, m["scale"], head_slopes(H), w("sink"))
    return o.reshape(T, H * V) @ w("o").T


# ------------------------------------------------------------------------------------------ decayed linear attention
def decayed_linear_attention(q, k, v, decay):
    """q, k [T, H, D], v [T, H, V], decay [H] -> read-outs [T, H, V]"""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = torch.zeros_like(v)
    lam = torch.as_tensor(decay, dtype=q.dtype)[:, None, None]
    for t in range(T):
        S = S * lam + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        out[t] = torch.einsum("hd,hdv->hv", q[t], S)
    return out


def lightning_mixer(h, w, m, eps):
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q, k = (silu(h @ w(n).T).view(T, H, D) for n in ("q", "k"))
    o = decayed_linear_attention(q, k, silu(h @ w("v").T).view(T, H, V), m["decay"]).reshape(T, H * V)
    return (rms(o, eps) * w("norm") * sigmoid(h @ w("g").T)) @ w("o").T


def parallel_mixer(h, w, m, eps):
    left = sink_attention_mixer(h, lambda n: w("left." + n), m["left"], eps)
    right = lightning_mixer(h, lambda n: w("right." + n), m["right"], eps)
    return m["left_scale"] * left + m["right_scale"] * right


# ------------------------------------------------------------------------------------------ feed-forward
def glu(h, w, act):
    return (act(h @ w("gate").T) * (h @ w("up").T)) @ w("down").T


def route(h, router, bias, top):
    """-> chosen experts [T, top] and their weights, a softmax over the chosen logits"""
    z = h @ router.T + bias
    val, idx = torch.sort(z, dim=-1, descending=True, stable=True)
    val, idx = val[:, :top], idx[:, :top]
    e = torch.exp(val - val[:, :1])
    return idx, e / e.sum(-1, keepdim=True)


def expert_mixture(h, w, mlp):
    idx, p = route(h, w("router"), w("router.b"), mlp["router"]["top"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, pe in zip(idx[t].tolist(), p[t]):
            y[t] += pe * glu(h[t:t + 1], lambda n, e=e: w(f"e{e}.{n}"), silu)[0]
    if mlp.get("shared"):
        y = y + glu(h, lambda n: w("shared." + n), silu)
    return y


def feed_forward(h, w, mlp):
    return glu(h, w, gelu_tanh) if mlp["kind"] == "dense" else expert_mixture(h, w, mlp)


# ------------------------------------------------------------------------------------------ the model
def layer_runs(cfg):
    """[(layer, starts a pass)] in the order the layers run"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return ([(i, False) for i in range(a)] + [(i, i == a) for _ in range(loop["times"]) for i in range(a, b)]
            + [(i, False) for i in range(b, n)])


MIXERS = {"channel_delta": channel_delta_mixer, "parallel": parallel_mixer}


def layer(x, W, p, entry, eps):
    h = norm_about_one(x, W[p + "norm1"], eps)
    y = MIXERS[entry["type"]](h, lambda n: W[p + "mix." + n], entry["mixer"], eps)
    if entry["mlp"] is not None:
        y = y + feed_forward(h, lambda n: W[p + "mlp." + n], entry["mlp"])
    return x + y


def forward(cfg, weights, tokens, dtype=torch.float64):
    """logits [T, vocab] and the residual stream after every layer run, a list of [T, width]"""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x0 = x = W["embed"][torch.as_tensor(tokens, dtype=torch.int64)]
    streams = []
    for i, starts in layer_runs(cfg):
        if starts:
            x = torch.cat([x, x0], -1) @ W["loop.in"].T
        x = layer(x, W, f"l{i}.", cfg["layers"][i], eps)
        streams.append(x)
    return norm_about_one(x, W["final.norm"], eps) @ W["head"].T, streams
