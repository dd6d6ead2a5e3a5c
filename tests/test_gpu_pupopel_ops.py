"""Every kernel of the layers whose sublayers run side by side, one mechanism at a time, against the plain restatement."""
import math

import pytest
import torch

from oracle import ref_pupopel as ref
from test_gpu_dogulorn_ops import DTYPES, close, rnd, tables_for, tol

pytestmark = pytest.mark.gpu


# ------------------------------------------------------------------------------------------------ rows
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [40, 100, 2304, 8192])
def test_residual_add_norm(dev, dtype, width):
    """the add, the norm about one or the cast, routed experts' rows (grouped or in their own order), a stream that starts"""
    from vllm_omni_amd import ops

    rows, top, eps = 5, 3, 3e-2                        # of the order of the rows' mean square: a misplaced eps shows
    x, y = rnd(rows, width, std=0.2, seed=1), rnd(rows, width, dtype=dtype, std=0.1, seed=2)
    w = rnd(width, dtype=dtype, std=0.3, seed=3)
    part, wt = rnd(rows * top + 4, width, dtype=dtype, std=0.1, seed=4), rnd(rows, top, seed=5).abs()
    where = torch.randperm(rows * top + 4, generator=torch.Generator().manual_seed(6))[:rows * top].to(torch.int32)
    for mapped in (None, where):
        take = part.double()[(where if mapped is not None else torch.arange(rows * top)).long()].view(rows, top, width)
        for experts in (False, True):
            for start in (False, True):
                x1 = (0 if start else x.double()) + y.double() + ((take * wt.double()[..., None]).sum(1) if experts else 0)
                for pre, want in ((w, ref.norm_about_one(x1, w.double(), eps)), (None, x1)):
                    xg = x.to(dev)
                    h = torch.full((rows, 2 * width), 5.0, dtype=dtype, device=dev)[:, :width]
                    er = ops.ExpertRows(part.to(dev), wt.to(dev), None if mapped is None else mapped.to(dev)) if experts else None
                    ops.residual_add_norm(xg, y.to(dev), None if pre is None else pre.to(dev), eps, h, er, 1.0, start)
                    close(xg, x1, rtol=1e-5, atol=1e-5)
                    close(h, want, **tol(dtype, 2.0))


def test_residual_add_norm_takes_32_bit_rows_and_partials(dev):
    from vllm_omni_amd import ops

    x, part = rnd(3, 256, seed=1), rnd(4, 3, 256, seed=2)
    h = torch.empty(3, 256, dtype=torch.bfloat16, device=dev)
    gp = part.to(dev)
    ops._LINEAR_GEN[gp.device] = ops._LINEAR_GEN.get(gp.device, 0) + 1
    p = ops.SplitKPartials(gp, 4, 3, 256, None, torch.bfloat16, (3,), gp.device, ops._LINEAR_GEN[gp.device])
    for y, want in ((p, part.double().sum(0)), (gp[1], part[1].double())):
        xg = x.to(dev)
        ops.residual_add_norm(xg, y, None, 1e-6, h)
        close(xg, x.double() + want, rtol=1e-5, atol=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [48, 50])
def test_embed_norm(dev, dtype, width):
    from vllm_omni_amd import ops

    table, w = rnd(30, width, dtype=dtype, seed=1), rnd(width, dtype=dtype, std=0.3, seed=2)
    ids = torch.tensor([3, 29, 0, 29, 30, -1])
    want = torch.cat([table.double()[ids[:4]], torch.zeros(2, width, dtype=torch.float64)])
    x = torch.empty(6, width, device=dev)
    both = torch.full((6, 2 * width), 9.0, dtype=dtype, device=dev)
    h = torch.empty(6, width, dtype=dtype, device=dev)
    ops.embed_norm(table.to(dev), ids.to(dev), x, w.to(dev), 1e-2, h, None, 1.0)
    close(x, want, rtol=0, atol=0)
    close(h, ref.norm_about_one(want, w.double(), 1e-2), **tol(dtype, 2.0))
    ops.embed_norm(table.to(dev), ids.to(dev), x, None, 1e-2, both[:, :width], both[:, width:], 1.0)
    close(both, torch.cat([want, want], 1), rtol=0, atol=0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [24, 13])
def test_glu(dev, dtype, ff):
    from vllm_omni_amd import ops

    gu = rnd(9, 2 * ff + 6, dtype=dtype, std=2.0, seed=1)
    g, u = gu[:, :ff], gu[:, ff + 3 if ff % 8 else ff:][:, :ff]
    gg = gu.to(dev)
    out = torch.zeros(9, ff + 8, dtype=dtype, device=dev)
    for act, f in (("silu", ref.silu), ("gelu_tanh", ref.gelu_tanh)):
        ops.glu(out[:, :ff], gg[:, :ff], gg[:, ff + 3 if ff % 8 else ff:][:, :ff], act)
        close(out[:, :ff], f(g.double()) * u.double(), **tol(dtype, 4.0))
    assert (out[:, ff:] == 0).all()


# ------------------------------------------------------------------------------------------------ attention
def kv_pages(k, v, tables, nb, bs, hd, dtype, dev):
    """K [T, G, D], V [T, G, V] per request -> head-major pages, heads padded to hd; pages start as garbage of finite size"""
    g = k[0].shape[1]
    t = torch.full((nb, 2, g, bs, hd), 3.0, dtype=dtype)
    t[..., k[0].shape[2]:] = 0
    t[:, 1, :, :, v[0].shape[2]:] = 0
    for kk, vv, tab in zip(k, v, tables):
        for i in range(kk.shape[0]):
            t[tab[i // bs], 0, :, i % bs, :kk.shape[2]] = kk[i].to(dtype)
            t[tab[i // bs], 1, :, i % bs, :vv.shape[2]] = vv[i].to(dtype)
    t = t.to(dev)
    return t[:, 0].permute(0, 2, 1, 3), t[:, 1].permute(0, 2, 1, 3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(4, 2, 64, 64, 64), (3, 1, 21, 35, 40), (8, 2, 128, 64, 128), (2, 2, 160, 96, 160), (5, 5, 48, 40, 64)],
                         ids=lambda s: "x".join(map(str, s)))
def test_head_norm_cache(dev, dtype, sizes):
    from vllm_omni_amd import ops

    h, g, d, vd, hd = sizes
    rows, bs, eps, coef, every = 7, 16, 2e-2, 0.7, 3
    x = rnd(rows, (h + g) * d + g * vd, dtype=dtype, std=0.2, seed=1)
    wq, wk = rnd(d, dtype=dtype, seed=2), rnd(d, dtype=dtype, seed=3)
    pos = torch.tensor([0, 1, 2, 5, 600, 8, 9])
    slots = torch.tensor([17, 3, -1, 47, 32, 16, 0])
    cache = torch.zeros(3, 2, g, bs, hd, dtype=dtype, device=dev)
    kc, vc = cache[:, 0].permute(0, 2, 1, 3), cache[:, 1].permute(0, 2, 1, 3)
    q = ops.head_norm_cache(x.to(dev), wq.to(dev), wk.to(dev), kc, vc, slots.to(dev), pos.to(dev), h, d, vd, eps, coef, every)
    xd = x.double()
    qw = ref.rms(xd[:, :h * d].view(rows, h, d), eps) * wq.double() * ref.query_temperature(pos.double(), coef, every)[:, None, None]
    kw = ref.rms(xd[:, h * d:(h + g) * d].view(rows, g, d), eps) * wk.double()
    vw = xd[:, (h + g) * d:].view(rows, g, vd)
    q = q.view(rows, h, hd)
    close(q[..., :d], qw, **tol(dtype, 2.0))
    assert (q[..., d:] == 0).all()
    for i, s in enumerate(slots.tolist()):
        if s >= 0:
            close(kc[s // bs, s % bs, :, :d], kw[i], **tol(dtype, 2.0))
            close(vc[s // bs, s % bs, :, :vd], vw[i], rtol=0, atol=0)
    assert int((cache != 0).any(-1).sum()) == 6 * 2 * g            # the row without a slot wrote nothing
    plain = ops.head_norm_cache(x.to(dev), None, None, kc, vc, slots.to(dev), pos.to(dev), h, d, vd, eps)
    close(plain.view(rows, h, hd)[..., :d], xd[:, :h * d].view(rows, h, d), rtol=0, atol=0)


def attention_case(h, g, d, vd, lens, dtype, seed, far=()):
    """per request q, k, v with a few keys made to stand out against the distance: (request, query, key)"""
    out = []
    slopes = ref.head_slopes(h)
    for r, n in enumerate(lens):
        q, k, v = rnd(n, h, d, seed=seed + 3 * r), rnd(n, g, d, seed=seed + 3 * r + 1), rnd(n, g, vd, seed=seed + 3 * r + 2)
        for rr, i, j in far:
            if rr == r:
                kh = rnd(g, d, seed=seed + 999)
                k[j] = kh
                for hh in range(h):      # a score that makes up for the distance, at scale d^-1/2
                    u = kh[hh // (h // g)]
                    q[i, hh] = u / (u * u).sum() * (slopes[hh] * (i - j) + 6.0) * math.sqrt(d)
        out.append((q.to(dtype), k.to(dtype), v.to(dtype)))
    return out


ATTN = [(8, 2, 64, 64, 64, 16), (5, 1, 48, 40, 64, 16), (16, 4, 128, 128, 128, 16), (7, 1, 128, 96, 128, 32), (3, 3, 40, 64, 64, 16),
        (32, 2, 64, 32, 64, 16)]


@pytest.mark.parametrize("case", ATTN, ids=lambda s: "x".join(map(str, s)))
def test_biased_sink_attention_kernels(dev, case):
    """prompts, portions and decoding on scattered pages: far keys that matter, sinks from negligible to dominant, short
    portions (the kernel for at most 16 rows) and long ones, contexts split or not"""
    from vllm_omni_amd import ops

    h, g, d, vd, hd, bs = case
    lens = [300, 33, 1, 130, 64]
    far = [(0, 299, 0), (0, 40, 31), (0, 200, 16), (3, 129, 15), (3, 64, 0), (1, 32, 0), (4, 63, 47)]
    reqs = attention_case(h, g, d, vd, lens, torch.bfloat16, 100, far)
    sink = torch.linspace(-30.0, 6.0, h)
    scale, mul = d ** -0.5, 0.6
    want = [ref.biased_sink_attention(*(t.double() for t in r), scale, ref.head_slopes(h), sink.double()) * mul for r in reqs]
    tabs, table, nb = tables_for(lens, bs, seed=4)
    kc, vc = kv_pages([r[1] for r in reqs], [r[2] for r in reqs], tabs, nb, bs, hd, torch.bfloat16, dev)
    slopes = torch.tensor(ref.head_slopes(h), device=dev)
    bias = dict(slopes=slopes, sinks=sink.to(dev), out_scale=mul)
    table = table.to(dev)
    i32 = dict(dtype=torch.int32, device=dev)

    def rows(parts):
        """parts: (request, first row, rows) -> padded q, seq_lens, query_start_loc, table"""
        q = torch.zeros(sum(n for _, _, n in parts), h, hd, dtype=torch.bfloat16)
        at = 0
        for r, a, n in parts:
            q[at:at + n, :, :d] = reqs[r][0][a:a + n]
            at += n
        qsl = torch.tensor([0] + [n for _, _, n in parts]).cumsum(0).to(**i32)
        return q.flatten(1).to(dev), torch.tensor([a + n for _, a, n in parts], **i32), qsl, table[[r for r, _, _ in parts]]

    def compare(out, parts):
        out, at = out.view(-1, h, hd), 0
        for r, a, n in parts:
            close(out[at:at + n, :, :vd], want[r][a:a + n], rtol=2 ** -6, atol=0.01)
            assert (out[at:at + n, :, vd:] == 0).all()
            at += n

    plans = [[(i, 0, n) for i, n in enumerate(lens)], [(0, 100, 90), (3, 0, 129)], [(0, 190, 2), (1, 30, 3), (3, 115, 15)], [(0, 284, 16)]]
    for parts in plans:
        q, seq, qsl, tab = rows(parts)
        longest = max(n for _, _, n in parts)
        for kw in (dict(), dict(max_seq_len=300), dict(max_seq_len=300, segments=3)):
            out = torch.full_like(q, 7.0)
            ops.paged_attn_prefill(out, q, kc, vc, tab, seq, qsl, longest, scale, **kw, **bias)
            compare(out, parts)
        out = torch.full_like(q, 7.0)
        ops.attn_rows(out, q, kc, vc, tab, seq, qsl, scale, **bias)
        compare(out, parts)
    for parts in ([(i, n - 1, 1) for i, n in enumerate(lens)], [(0, 40, 1), (0, 200, 1), (3, 64, 1)]):
        q, seq, qsl, tab = rows(parts)
        for kw in (dict(), dict(partition_size=64), dict(partition_size=32)):
            out = torch.full_like(q, 7.0)
            ops.paged_attn_decode(out, q, kc, vc, tab, seq, 300, scale, **kw, **bias)
            compare(out, parts)
    # padded rows of a graph replay: no tokens, zeros
    out = torch.full_like(q, 7.0)
    ops.paged_attn_decode(out, q, kc, vc, tab, torch.zeros_like(seq), 300, scale, **bias)
    assert (out == 0).all()


def test_attention_rows_in_32_bit(dev):
    from vllm_omni_amd import ops

    h, g, d, vd, hd, bs = 6, 3, 33, 21, 40, 16
    lens = [280, 20]
    reqs = attention_case(h, g, d, vd, lens, torch.float32, 7, [(0, 279, 2), (0, 256, 255)])
    sink = torch.linspace(-3.0, 4.0, h)
    tabs, table, nb = tables_for(lens, bs, seed=1)
    kc, vc = kv_pages([r[1] for r in reqs], [r[2] for r in reqs], tabs, nb, bs, hd, torch.float32, dev)
    q = torch.zeros(300, h, hd)
    q[..., :d] = torch.cat([r[0] for r in reqs])
    i32 = dict(dtype=torch.int32, device=dev)
    args = (q.flatten(1).to(dev), kc, vc, table.to(dev), torch.tensor(lens, **i32), torch.tensor([0, 280, 300], **i32), d ** -0.5)
    slopes = torch.tensor(ref.head_slopes(h), device=dev)
    for kw, sl, sk in ((dict(slopes=slopes, sinks=sink.to(dev)), ref.head_slopes(h), sink), (dict(sinks=sink.to(dev)), [0.0] * h, sink),
                       (dict(slopes=slopes), ref.head_slopes(h), torch.full((h,), -1e30))):
        out = torch.zeros(300, h * hd, device=dev)
        ops.attn_rows(out, *args, **kw)
        want = torch.cat([ref.biased_sink_attention(*(t.double() for t in r), d ** -0.5, sl, sk.double()) for r in reqs])
        close(out.view(300, h, hd)[..., :vd], want, rtol=2e-5, atol=2e-5)


# ------------------------------------------------------------------------------------------------ channel-wise gated delta rule
class ChannelCase:
    def __init__(self, h, kvh, dim, vdim, taps, dtype, dev, slots=5, a_std=1.0, a_log=-1.5):
        self.h, self.kvh, self.dim, self.vdim, self.dtype, self.dev, self.a_std = h, kvh, dim, vdim, dtype, dev, a_std
        self.kd, self.hd, self.hv = kvh * dim, h * dim, h * vdim
        self.ch = 2 * self.kd + self.hv
        self.conv = rnd(self.ch, taps, dtype=dtype, std=0.6, seed=1)
        self.a_log, self.dt = rnd(h, std=0.7, seed=2) + a_log, rnd(self.hd, std=0.8, seed=3)
        self.norm = rnd(vdim, dtype=dtype, std=0.3, seed=4) + 1
        self.state = torch.full((slots, h, dim, vdim), 7.0, device=dev)         # slots start dirty
        self.ring = torch.full((slots, taps, self.ch), 7.0, dtype=dtype, device=dev)

    def rows(self, n, seed):
        """qkv, decay projection, gate, b"""
        return [rnd(n, c, dtype=self.dtype, std=s, seed=seed + 1000 * j)
                for j, (c, s) in enumerate(((self.ch, 1.0), (self.hd, self.a_std), (self.hv, 1.0), (self.h, 1.0)))]

    def want(self, rows):
        p, a, gate, b = (t.double() for t in rows)
        t, c = p.shape[0], self.conv.double()
        q, k, v = (ref.silu(ref.short_conv(p[:, lo:hi], c[lo:hi])) for lo, hi in ((0, self.kd), (self.kd, 2 * self.kd), (2 * self.kd, self.ch)))
        of = torch.arange(self.h) // (self.h // self.kvh)
        q, k = ref.unit(q.view(t, self.kvh, -1)) / math.sqrt(self.dim), ref.unit(k.view(t, self.kvh, -1))
        g = ref.channel_decay(a, self.dt.double(), self.a_log.double(), self.h, self.dim)
        o, s = ref.channel_delta_rule(q[:, of], k[:, of], v.view(t, self.h, -1), ref.sigmoid(b), g)
        return (ref.rms(o, 1e-5) * self.norm.double() * ref.sigmoid(gate).view(t, self.h, -1)).reshape(t, self.hv), s

    def run(self, parts, chunked):
        """parts: [(slot, rows, tokens before them)] in one call -> output rows per part"""
        from vllm_omni_amd import ops

        dev, i32 = self.dev, torch.int32
        p, a, gate, b = (torch.cat([r[j] for _, r, _ in parts]).to(dev) for j in range(4))
        lens = [r[0].shape[0] for _, r, _ in parts]
        qsl = torch.tensor([0] + lens).cumsum(0).to(i32).to(dev)
        seq = torch.tensor([n0 + n for (_, _, n0), n in zip(parts, lens)], dtype=i32, device=dev)
        slots = torch.tensor([s for s, _, _ in parts], dtype=i32, device=dev)
        out = torch.full((p.shape[0], self.hv + 8), 5.0, dtype=self.dtype, device=dev)
        args = (p, self.conv.to(dev), self.a_log.to(dev), self.dt.to(dev), self.norm.to(dev), self.state, self.ring, slots, qsl, seq,
                self.kvh, 1e-5, out[:, :self.hv])
        kw = dict(gate=gate, beta=b, decay=a, sigmoid_gate=True)
        if chunked:
            ops.gated_delta_chunked(*args, 0, len(parts), 0, max(lens), **kw)
        else:
            ops.gated_delta_step(*args, 0, len(parts), **kw)
        assert (out[:, self.hv:] == 5.0).all()
        return list(out[:, :self.hv].split(lens))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(4, 2, 32, 64, 4), (6, 3, 24, 40, 3), (3, 3, 18, 30, 2), (2, 1, 33, 21, 1), (9, 3, 64, 128, 4),
                                   (2, 2, 128, 64, 6), (2, 1, 128, 256, 4), (2, 1, 136, 72, 4)], ids=lambda s: "x".join(map(str, s)))
def test_channel_delta(dev, dtype, sizes):
    """whole prompts, portions cut anywhere (down to single tokens) and unequal batches, chunked and token by token"""
    t = dict(rtol=2 ** -6, atol=0.03) if dtype == torch.bfloat16 else dict(rtol=1e-4, atol=1e-4)
    c = ChannelCase(*sizes, dtype, dev)
    lens = [1, 64, 65, 150, 2]
    ps = [c.rows(n, 50 + i) for i, n in enumerate(lens)]
    wants = [c.want(p) for p in ps]
    for chunked in (False, True):
        outs = c.run([(4 - i, p, 0) for i, p in enumerate(ps)], chunked)
        for i in range(len(lens)):
            close(outs[i], wants[i][0], **t)
            close(c.state[4 - i], wants[i][1], rtol=1e-4, atol=2e-5)
    cuts = [0, 2, 3, 5, 70, 72, 73, 137, 138, 139, 140, 150]
    for n, (a, b) in enumerate(zip(cuts, cuts[1:])):
        parts = [(2, [x[a:b] for x in ps[3]], a)]
        if n < 4:
            parts.append((0, [x[16 * n:16 * n + 16] for x in ps[1]], 16 * n))
        outs = c.run(parts, chunked=n % 3 != 2)
        close(outs[0], wants[3][0][a:b], **t)
        if n < 4:
            close(outs[1], wants[1][0][16 * n:16 * n + 16], **t)
    close(c.state[2], wants[3][1], rtol=1e-4, atol=2e-5)


@pytest.mark.parametrize("a_std,a_log", [(6.0, 2.0), (20.0, 4.5), (3.0, -6.0)])
def test_channel_decays_of_every_strength(dev, a_std, a_log):
    """from channels that forget everything within a token (e^-1000 and less) to channels that forget nothing, beside each
    other: no factor of the chunked form may overflow or vanish where the product does not"""
    c = ChannelCase(3, 1, 48, 32, 4, torch.float32, dev, a_std=a_std, a_log=a_log)
    p = c.rows(200, 9)
    w, s = c.want(p)
    for chunked in (False, True):
        close(c.run([(0, p, 0)], chunked)[0], w, rtol=2e-4, atol=2e-4)
        close(c.state[0], s, rtol=2e-4, atol=5e-5)


def test_channel_delta_repeated_keys_stay_exact(dev):
    """equal tokens give equal keys: the chunk's triangular system is then as far from the identity as it gets"""
    c = ChannelCase(2, 1, 32, 32, 4, torch.float32, dev)
    p = [x.repeat(200, 1) for x in c.rows(1, 5)]
    p[1] = p[1] - 8.0       # hardly any decay
    p[3][:] = 4.0           # write strength near 1
    w, s = c.want(p)
    close(c.run([(0, p, 0)], True)[0], w, rtol=1e-3, atol=1e-3)
    close(c.state[0], s, rtol=1e-3, atol=1e-4)


# ------------------------------------------------------------------------------------------------ decayed linear attention
class LightningCase:
    def __init__(self, h, d, v, dtype, dev, slots=5):
        self.h, self.d, self.v, self.dtype, self.dev = h, d, v, dtype, dev
        self.decay = [1.0, 0.999, 0.3, 0.9, 0.01, 0.99][:h]
        self.norm = rnd(h * v, dtype=dtype, std=0.3, seed=4) + 1
        self.state = torch.full((slots, h, d, v), 7.0, device=dev)

    def rows(self, n, seed):
        return [rnd(n, self.h * (2 * self.d + self.v), dtype=self.dtype, seed=seed), rnd(n, self.h * self.v, dtype=self.dtype, seed=seed + 1000)]

    def want(self, rows):
        p, gate = (t.double() for t in rows)
        t, hd = p.shape[0], self.h * self.d
        q, k, v = ref.silu(p[:, :hd]).view(t, self.h, -1), ref.silu(p[:, hd:2 * hd]).view(t, self.h, -1), ref.silu(p[:, 2 * hd:]).view(t, self.h, -1)
        o = ref.decayed_linear_attention(q, k, v, self.decay).reshape(t, -1)
        return ref.rms(o, 1e-2) * self.norm.double() * ref.sigmoid(gate) * 0.7

    def run(self, parts, chunked, row0=0):
        from vllm_omni_amd import ops

        dev, i32 = self.dev, torch.int32
        p, gate = (torch.cat([r[j] for _, r, _ in parts]).to(dev) for j in range(2))
        lens = [r[0].shape[0] for _, r, _ in parts]
        qsl = torch.tensor([0] + lens).cumsum(0).to(i32).to(dev)
        seq = torch.tensor([n0 + n for (_, _, n0), n in zip(parts, lens)], dtype=i32, device=dev)
        slots = torch.tensor([s for s, _, _ in parts], dtype=i32, device=dev)
        out = torch.full((p.shape[0], self.h * self.v + 8), 5.0, dtype=self.dtype, device=dev)
        dec = torch.tensor(self.decay, device=dev)
        ops.lightning_attn(p, gate, self.norm.to(dev), dec, dec.double().log2().float(), self.state, slots, qsl, seq, 1e-2, out[:, :-8], 0,
                           len(parts), 0, p.shape[0], max(lens), 0.7, chunked=chunked)
        assert (out[:, -8:] == 5.0).all()
        return list(out[:, :-8].split(lens))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(2, 64, 64), (3, 24, 40), (2, 19, 13), (6, 128, 128), (1, 136, 200), (4, 32, 256), (1, 300, 20)],
                         ids=lambda s: "x".join(map(str, s)))
def test_lightning_attention(dev, dtype, sizes):
    t = dict(rtol=2 ** -6, atol=0.03) if dtype == torch.bfloat16 else dict(rtol=1e-4, atol=1e-4)
    c = LightningCase(*sizes, dtype, dev)
    lens = [1, 64, 65, 150, 2]
    ps = [c.rows(n, 70 + i) for i, n in enumerate(lens)]
    wants = [c.want(p) for p in ps]
    for chunked in (False, True):
        for got, w in zip(c.run([(4 - i, p, 0) for i, p in enumerate(ps)], chunked), wants):
            close(got, w, **t)
    cuts = [0, 2, 3, 5, 70, 72, 73, 137, 138, 139, 140, 150]
    for n, (a, b) in enumerate(zip(cuts, cuts[1:])):
        parts = [(2, [x[a:b] for x in ps[3]], a)]
        if n < 4:
            parts.append((0, [x[16 * n:16 * n + 16] for x in ps[1]], 16 * n))
        outs = c.run(parts, chunked=n % 3 != 2)
        close(outs[0], wants[3][a:b], **t)
        if n < 4:
            close(outs[1], wants[1][16 * n:16 * n + 16], **t)


@pytest.mark.parametrize("sizes", [(2, 64, 64), (3, 24, 40), (1, 128, 128)], ids=lambda s: "x".join(map(str, s)))
def test_lightning_attention_in_segments(dev, sizes):
    """long portions: chunks run in segments side by side; requests of unequal length, then a second portion from the states"""
    c = LightningCase(*sizes, torch.float32, dev)
    c.decay = [1.0, 0.999, 0.9997][:sizes[0]]
    lens = [2100, 70, 1030, 512]
    ps = [c.rows(n, 30 + i) for i, n in enumerate(lens)]
    wants = [c.want(p) for p in ps]
    cut = [1500, 60, 1000, 1]
    for got, w, n in zip(c.run([(i, [x[:n] for x in p], 0) for i, (p, n) in enumerate(zip(ps, cut))], True), wants, cut):
        close(got, w[:n], rtol=2e-4, atol=2e-4)
    for got, w, n in zip(c.run([(i, [x[n:] for x in p], n) for i, (p, n) in enumerate(zip(ps, cut))], True), wants, cut):
        close(got, w[n:], rtol=2e-4, atol=2e-4)


# ------------------------------------------------------------------------------------------------ routed experts
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("t,width,experts,top,ff", [(7, 96, 6, 2, 40), (70, 128, 8, 3, 64), (33, 100, 5, 1, 21), (300, 320, 9, 4, 96),
                                                    (90, 256, 40, 4, 64), (20, 128, 130, 16, 16), (3, 200, 4, 4, 24),
                                                    (1500, 72, 20, 2, 16)])
def test_routed_experts(dev, dtype, t, width, experts, top, ff):
    from vllm_omni_amd import ops
    from vllm_omni_amd.moe import RoutedExperts

    m = RoutedExperts(width, experts, top, ff, dtype, dev)
    w = {"router": rnd(experts, width, dtype=dtype, std=4 * width ** -0.5, seed=1), "router.b": rnd(experts, std=0.7, seed=2)}
    for e in range(experts):
        for j, (n, a, b) in enumerate((("gate", ff, width), ("up", ff, width), ("down", width, ff))):
            w[f"e{e}.{n}"] = rnd(a, b, dtype=dtype, std=b ** -0.5, seed=10 + 3 * e + j)
    for name, dst in m.named_weights(""):
        assert tuple(dst.shape) == tuple(w[name].shape)
        dst.copy_(w[name])
    h = rnd(t, width, dtype=dtype, seed=5)
    hg = torch.full((t, width + 8), 9.0, dtype=dtype, device=dev)[:, :width]
    hg.copy_(h)
    wd = {k: v.double() for k, v in w.items()}
    idx, p = ref.route(h.double(), wd["router"], wd["router.b"], top)
    logits = ops.moe_router_logits(hg, m.router)
    close(logits, h.double() @ wd["router"].T, rtol=1e-5, atol=2e-5)      # 32-bit whatever the rows are
    ids, wt, _ = ops.moe_route(logits, top, True, want_counts=False, bias=m.router_b)
    assert torch.equal(ids.cpu().long().sort(-1).values, idx.sort(-1).values)
    got = torch.zeros(t, experts, dtype=torch.float64).scatter_(1, ids.cpu().long(), wt.cpu().double())
    close(got, torch.zeros(t, experts, dtype=torch.float64).scatter_(1, idx, p), rtol=1e-5, atol=1e-6)
    er = m(hg)
    x = torch.zeros(t, width, device=dev)
    ops.residual_add_norm(x, torch.zeros(t, width, dtype=dtype, device=dev), None, 1e-6, torch.empty(t, width, dtype=dtype, device=dev), er)
    want = ref.expert_mixture(h.double(), lambda n: wd[n], {"router": {"top": top}})
    close(x, want, **(dict(rtol=2 ** -6, atol=0.02) if dtype == torch.bfloat16 else dict(rtol=1e-4, atol=2e-5)))
