"""Every kernel of the state-space layers, of attention whose values are its keys and of the rows around them, one mechanism at
a time, against the plain restatement."""
import pytest
import torch

from oracle import ref_lifuzen as ref
from test_gpu_dogulorn_ops import DTYPES, close, rnd, tables_for, tol
from test_gpu_pupopel_ops import kv_pages

pytestmark = pytest.mark.gpu


# ------------------------------------------------------------------------------------------------ rows
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [40, 100, 2304, 8192])
def test_stream_norm2(dev, dtype, width):
    """the multiplied add, a pass's vector and the embedding output, experts' rows (weighted or not), both norms, a stream that starts"""
    from vllm_omni_amd import ops

    rows, top, eps, mult = 5, 3, 3e-2, 0.45            # eps of the order of the rows' mean square: a misplaced one shows
    x, y = rnd(rows, width, std=0.2, seed=1), rnd(rows, width, dtype=dtype, std=0.3, seed=2)
    w1, w2, step = (rnd(width, dtype=dtype, std=0.3, seed=3 + i) for i in range(3))
    table, ids = rnd(30, width, dtype=dtype, std=0.2, seed=6), torch.tensor([3, 29, 0, 30, -1])
    emb = torch.cat([table.double()[ids[:3]], torch.zeros(2, width, dtype=torch.float64)])       # ids outside the table: zeros
    part, wt = rnd(rows * top + 4, width, dtype=dtype, std=0.2, seed=7), rnd(rows, top, seed=8).abs()
    where = torch.randperm(rows * top + 4, generator=torch.Generator().manual_seed(9))[:rows * top].to(torch.int32)
    g = lambda t: None if t is None else t.to(dev)     # noqa: E731
    for start in (False, True):
        for experts in ((None,) if start else (None, "own", "mapped", "plain")):
            for with_table, row, second in ((True, step, True), (start, None, False), (start, step, True)):
                want = torch.zeros(rows, width, dtype=torch.float64)
                er = None
                if not start:
                    add = y.double()
                    if experts:
                        take = part.double()[(torch.arange(rows * top) if experts == "own" else where).long()].view(rows, top, width)
                        add = add + (take * (1.0 if experts == "plain" else wt.double()[..., None])).sum(1)
                        er = ops.ExpertRows(g(part), None if experts == "plain" else g(wt), None if experts == "own" else g(where), top)
                    want = x.double() + mult * add
                want = want + (emb if with_table else 0) + (row.double() if row is not None else 0)
                xg = g(x)
                h = torch.full((2, rows, width + 8), 5.0, dtype=dtype, device=dev)[:, :, :width]
                ops.stream_norm2(xg, None if start else g(y), g(w1), g(w2) if second else None, eps, h[0], h[1] if second else None, 1.0, mult,
                                 er, g(table) if with_table else None, g(ids), g(row))
                close(xg, want, rtol=1e-5, atol=1e-5)            # the stream stays 32-bit in both modes
                close(h[0], ref.norm_about_one(want, w1.double(), eps), **tol(dtype, 2.0))
                if second:
                    close(h[1], ref.norm_about_one(want, w2.double(), eps), **tol(dtype, 2.0))


def test_stream_norm2_takes_32_bit_rows_and_partials(dev):
    from vllm_omni_amd import ops

    x, part, w = rnd(3, 256, seed=1), rnd(4, 3, 256, seed=2), rnd(256, dtype=torch.bfloat16, seed=3).to(dev)
    h = torch.empty(3, 256, dtype=torch.bfloat16, device=dev)
    gp = part.to(dev)
    ops._LINEAR_GEN[gp.device] = ops._LINEAR_GEN.get(gp.device, 0) + 1
    p = ops.SplitKPartials(gp, 4, 3, 256, None, torch.bfloat16, (3,), gp.device, ops._LINEAR_GEN[gp.device])
    for y, want in ((p, part.double().sum(0)), (gp[1], part[1].double())):
        xg = x.to(dev)
        ops.stream_norm2(xg, y, w, None, 1e-6, h, mult=0.5)
        close(xg, x.double() + 0.5 * want, rtol=1e-5, atol=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("vocab", [131, 1000, 20000])
def test_soft_cap_argmax(dev, dtype, vocab):
    from vllm_omni_amd import ops

    lg = rnd(6, vocab, dtype=dtype, std=4.0, seed=1)
    lg[2, 7] = lg[2, 90] = lg[2].max() + 1              # the first of equals
    want = ref.soft_cap(lg.double(), 5.0)
    buf = torch.full((6, vocab + 8), 3.0, dtype=dtype, device=dev)
    out = buf[:, :vocab]
    out.copy_(lg)
    ids = ops.soft_cap_argmax(out, 5.0)
    close(out, want, **(dict(rtol=2 ** -7, atol=1e-3) if dtype == torch.bfloat16 else dict(rtol=1e-6, atol=1e-6)))
    assert (buf[:, vocab:] == 3.0).all()
    o = out.float().cpu()
    assert ids.tolist() == [int((r == r.max()).nonzero()[0]) for r in o] and ids[2] == 7
    out.copy_(lg)
    assert ops.soft_cap_argmax(out, 5.0, greedy=False) is None and torch.equal(out.float().cpu(), o)


# ------------------------------------------------------------------------------------------------ filter, rotation, norm, cache
class ConvRopeCase:
    def __init__(self, h, g, d, hd, rot, taps, dtype, dev, slots=4, bs=16, blocks=40):
        self.h, self.g, self.d, self.hd, self.rot, self.taps, self.dtype, self.dev, self.bs = h, g, d, hd, rot, taps, dtype, dev, bs
        self.w = rnd((h + g) * d, taps, dtype=dtype, std=0.6, seed=1)
        self.ring = torch.full((slots, taps, (h + g) * d), 9.0, dtype=dtype, device=dev)        # dirty: nothing is ever cleared
        self.cache = torch.full((blocks, 2, g, bs, hd), 8.0, dtype=dtype, device=dev)
        freq = 300.0 ** (-torch.arange(0, rot, 2, dtype=torch.float64) / max(rot, 1))
        self.freq = freq.float().to(dev) if rot else None

    def rows(self, n, seed):
        return rnd(n, (self.h + self.g) * self.d, dtype=self.dtype, seed=seed)

    def want(self, x, first=0):
        """rows that start a sequence, or (``first``) whose sequence had zeros before them"""
        y = ref.short_conv(x.double(), self.w.double())
        t = y.shape[0]
        q, v = y[:, :self.h * self.d].view(t, self.h, self.d), y[:, self.h * self.d:].view(t, self.g, self.d)
        return [ref.rms(ref.rotate(a, self.rot, 300.0, first), 2e-2) for a in (q, v)] + [v]

    def run(self, parts, split=True):
        """parts: (slot, rows, rows before them); pages of a slot follow each other"""
        from vllm_omni_amd import ops

        i32 = dict(dtype=torch.int32, device=self.dev)
        x = torch.full((sum(p.shape[0] for _, p, _ in parts), (self.h + self.g) * self.d + 8), 3.0, dtype=self.dtype, device=self.dev)
        x = x[:, :-8] if self.d % 8 == 0 else x[:, 3:-5]
        x.copy_(torch.cat([p for _, p, _ in parts]))
        lens = [p.shape[0] for _, p, _ in parts]
        qsl = torch.tensor([0] + lens).cumsum(0).to(**i32)
        seq = torch.tensor([a + n for (_, _, a), n in zip(parts, lens)], **i32)
        slots = torch.tensor([s for s, _, _ in parts], **i32)
        at = torch.cat([s * 160 + (torch.arange(a, a + n) % 160) for (s, _, a), n in zip(parts, lens)]).to(self.dev)
        q = torch.full((x.shape[0], self.h * self.hd), 7.0, dtype=self.dtype, device=self.dev)
        kc, vc = self.cache[:, 0].permute(0, 2, 1, 3), self.cache[:, 1].permute(0, 2, 1, 3)
        ops.conv_rope_cache(x, self.w.to(self.dev), self.ring, q, kc, vc, self.freq, slots, qsl, seq, at, self.h, self.d, 2e-2, 0, len(parts),
                            max(lens))
        k, v = kc[at // 16, at % 16], vc[at // 16, at % 16]
        return [t.split(lens) for t in (q.view(-1, self.h, self.hd), k, v)]

    def compare(self, got, i, want, lo, hi):
        for g, w in zip(got, want):
            close(g[i][..., :self.d], w[lo:hi], **tol(self.dtype, 3.0))
            assert (g[i][..., self.d:] == 0).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(6, 1, 64, 64, 32, 4), (3, 1, 21, 64, 6, 2), (4, 4, 48, 64, 20, 4), (2, 2, 128, 128, 128, 4), (3, 1, 96, 128, 0, 1),
                                   (40, 8, 40, 64, 40, 3), (2, 1, 160, 160, 160, 6), (5, 5, 33, 40, 32, 4), (1, 1, 300, 304, 100, 4)],
                         ids=lambda s: "x".join(map(str, s)))
def test_conv_rope_cache(dev, dtype, sizes):
    c = ConvRopeCase(*sizes, dtype, dev)
    lens = [1, 40, 9, 70]
    xs = [c.rows(n, 20 + i) for i, n in enumerate(lens)]
    wants = [c.want(x) for x in xs]
    got = c.run([(3 - i, x, 0) for i, x in enumerate(xs)])
    for i, (w, n) in enumerate(zip(wants, lens)):
        c.compare(got, i, w, 0, n)
    # the same sequences again in portions and one by one, in slots that held others: the first tokens, lengths around the taps
    for plan in ([1] * 20, [2] * 8, [1, 2, 3, 1, 5, 4, 1, 1, 8, 9, 1], [7, 17, 16], [33, 1, 1, 5]):
        at = 0
        for n in plan:
            parts = [(0, xs[3][at:at + n], at)] + ([(2, xs[1][at:at + 1], at)] if n == 1 and at < 40 and set(plan) == {1} else [])
            got = c.run(parts)
            c.compare(got, 0, wants[3], at, at + n)
            if len(parts) > 1:
                c.compare(got, 1, wants[1], at, at + 1)
            at += n


@pytest.mark.parametrize("dtype", DTYPES)
def test_angles_of_far_positions(dev, dtype):
    """zeros in front, so that the filter of the rows looked at starts there; angles in the tens of thousands"""
    c = ConvRopeCase(2, 1, 64, 64, 64, 4, dtype, dev)
    c.freq = (300.0 ** (-torch.arange(0, 64, 2, dtype=torch.float64) / 64)).float().to(dev)
    x = c.rows(20, 3)
    for first in (1000, 70000):
        c.ring.zero_()
        want = c.want(x, first)
        got = c.run([(1, x[:5], first)])
        for g, w in zip(got, want):
            close(g[0], w[:5], **(tol(dtype, 3.0) if dtype == torch.bfloat16 else dict(rtol=1e-4, atol=2e-2 if first > 5000 else 1e-3)))


def test_rows_without_a_slot_write_nothing(dev):
    """padded rows of a graph replay"""
    from vllm_omni_amd import ops

    c = ConvRopeCase(2, 1, 64, 64, 32, 4, torch.bfloat16, dev)
    before, ring = c.cache.clone(), c.ring.clone()
    i32 = dict(dtype=torch.int32, device=dev)
    q = torch.zeros(2, 128, dtype=torch.bfloat16, device=dev)
    kc, vc = c.cache[:, 0].permute(0, 2, 1, 3), c.cache[:, 1].permute(0, 2, 1, 3)
    ops.conv_rope_cache(c.rows(2, 1).to(dev), c.w.to(dev), c.ring, q, kc, vc, c.freq, torch.tensor([3, 3], **i32), torch.tensor([0, 1, 2], **i32),
                        torch.zeros(2, **i32), torch.full((2,), -1, dtype=torch.int64, device=dev), 2, 64, 1e-5, 0, 2, 1)
    assert torch.equal(c.cache, before) and torch.equal(c.ring, ring) and q.isfinite().all()


# ------------------------------------------------------------------------------------------------ attention with a sink of score 0
ATTN = [(6, 2, 64, 64, 16), (5, 1, 48, 64, 16), (16, 4, 128, 128, 16), (7, 7, 21, 64, 32), (12, 1, 96, 128, 16), (32, 2, 40, 64, 16)]


@pytest.mark.parametrize("case", ATTN, ids=lambda s: "x".join(map(str, s)))
def test_sink_attention_kernels(dev, case):
    """prompts, portions and decoding on scattered pages: keys far away and at page borders that stand out, rows whose scores are so
    low that the sink takes nearly all, the first tokens"""
    from vllm_omni_amd import ops

    h, g, d, hd, bs = case
    lens, scale = [300, 33, 1, 130, 64], d ** -0.5
    far = [(0, 299, 0), (0, 40, 31), (0, 200, 16), (3, 129, 15), (3, 64, 0), (1, 32, 0), (4, 63, 47), (0, 17, 17)]
    reqs = []
    for r, n in enumerate(lens):
        q, v = rnd(n, h, d, seed=3 * r), rnd(n, g, d, seed=3 * r + 1)
        k = ref.rms(v, 0.0)
        q = ref.rms(q, 0.0) * 1.5
        for rr, i, j in far:
            if rr == r:
                q[i] = k[j].repeat_interleave(h // g, 0) * 14.0 / (scale * d)        # score 14 there, a few elsewhere
        if n > 50:
            q[20:24] *= 0.01
            k[5:9] *= -1.0
            q[25] = -k[:26].mean(0).repeat_interleave(h // g, 0) * 30.0              # all scores below the sink's on the average
        reqs.append((q.to(torch.bfloat16), k.to(torch.bfloat16), v.to(torch.bfloat16)))
    want = [ref.sink_attention(*(t.double() for t in r), scale) for r in reqs]
    tabs, table, nb = tables_for(lens, bs, seed=4)
    kc, vc = kv_pages([r[1] for r in reqs], [r[2] for r in reqs], tabs, nb, bs, hd, torch.bfloat16, dev)
    bias = dict(sinks=torch.zeros(h, device=dev))
    table = table.to(dev)
    i32 = dict(dtype=torch.int32, device=dev)

    def rows(parts):
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
            close(out[at:at + n, :, :d], want[r][a:a + n], rtol=2 ** -6, atol=0.012)
            at += n

    for parts in ([(i, 0, n) for i, n in enumerate(lens)], [(0, 100, 90), (3, 0, 129)], [(0, 190, 2), (1, 30, 3), (3, 115, 15)], [(0, 284, 16)]):
        q, seq, qsl, tab = rows(parts)
        for kw in (dict(), dict(max_seq_len=300), dict(max_seq_len=300, segments=3)):
            out = torch.full_like(q, 7.0)
            ops.paged_attn_prefill(out, q, kc, vc, tab, seq, qsl, max(n for _, _, n in parts), scale, **kw, **bias)
            compare(out, parts)
        out = torch.full_like(q, 7.0)
        ops.attn_rows(out, q, kc, vc, tab, seq, qsl, scale, **bias)
        compare(out, parts)
    for parts in ([(i, n - 1, 1) for i, n in enumerate(lens)], [(0, 40, 1), (0, 200, 1), (3, 64, 1), (0, 25, 1), (0, 17, 1)]):
        q, seq, qsl, tab = rows(parts)
        for kw in (dict(), dict(partition_size=64), dict(partition_size=32)):
            out = torch.full_like(q, 7.0)
            ops.paged_attn_decode(out, q, kc, vc, tab, seq, 300, scale, **kw, **bias)
            compare(out, parts)


# ------------------------------------------------------------------------------------------------ state space
class SsmCase:
    def __init__(self, h, g, n, v, taps, parts, dtype, dev, slots=5, a_log=(-0.5, 1.2), bias=(-2.0, 1.0)):
        self.h, self.g, self.n, self.v, self.taps, self.parts, self.dtype, self.dev = h, g, n, v, taps, parts, dtype, dev
        self.inner, self.ch = h * v, h * v + 2 * g * n
        self.w, self.b = rnd(self.ch, taps, dtype=dtype, std=0.7, seed=1), rnd(self.ch, dtype=dtype, std=0.3, seed=2)
        self.a_log, self.bias = rnd(h, std=a_log[1], seed=3) + a_log[0], rnd(h, std=bias[1], seed=4) + bias[0]
        self.d, self.norm = rnd(h, seed=5) + 0.5, rnd(self.inner, dtype=dtype, std=0.3, seed=6) + 1
        self.norm = self.norm.to(dtype)
        self.state = torch.full((slots, h, n, v), 7.0, device=dev)                   # dirty: nothing is ever cleared
        self.ring = torch.full((slots, taps, self.ch), 9.0, dtype=dtype, device=dev)

    def rows(self, t, seed, std=1.0):
        return rnd(t, self.inner + self.ch + self.h, dtype=self.dtype, std=std, seed=seed)

    def want(self, x):
        z, xbc, raw = x.double().split([self.inner, self.ch, self.h], 1)
        t = x.shape[0]
        xbc = ref.silu(ref.short_conv(xbc, self.w.double()) + self.b.double()).to(self.dtype).double()
        xs, b, c = xbc.split([self.inner, self.g * self.n, self.g * self.n], 1)
        y, s = ref.state_space(xs.reshape(t, self.h, self.v), b.reshape(t, self.g, self.n), c.reshape(t, self.g, self.n),
                               ref.step_sizes(raw, self.bias.double()), self.a_log.double(), self.d.double())
        return ref.gated_group_norm(y.reshape(t, -1), z, self.norm.double(), self.parts, 1e-2), s

    def run(self, parts, chunked):
        from vllm_omni_amd import ops

        i32 = dict(dtype=torch.int32, device=self.dev)
        x = torch.cat([p for _, p, _ in parts])
        pad = -x.shape[1] % 16
        xg = torch.full((x.shape[0], x.shape[1] + pad), 3.0, dtype=self.dtype, device=self.dev)
        xg[:, :x.shape[1]] = x.to(self.dev)
        lens = [p.shape[0] for _, p, _ in parts]
        qsl = torch.tensor([0] + lens).cumsum(0).to(**i32)
        seq = torch.tensor([a + n for (_, _, a), n in zip(parts, lens)], **i32)
        out = torch.full((x.shape[0], self.inner + 8), 5.0, dtype=self.dtype, device=self.dev)
        at = self.inner + self.ch
        f = lambda t: t.to(self.dev)   # noqa: E731
        ops.state_space(xg[:, self.inner:at], xg[:, :self.inner], xg[:, at:at + self.h], f(self.w), f(self.b), f(self.bias), f(self.a_log),
                        f(self.d), f(self.norm), self.state, self.ring, torch.tensor([s for s, _, _ in parts], **i32), qsl, seq, self.g,
                        self.parts, 1e-2, out[:, :-8], 0, len(parts), 0, x.shape[0], max(lens), chunked=chunked)
        assert (out[:, -8:] == 5.0).all()
        return list(out[:, :-8].split(lens))


def ssm_tol(dtype):
    return dict(rtol=2 ** -6, atol=0.03) if dtype == torch.bfloat16 else dict(rtol=1e-4, atol=1e-4)


def state_tol(dtype):
    """the state is 32-bit in both modes; 16-bit filter outputs may round the other way here and there"""
    return dict(rtol=4e-3, atol=4e-3) if dtype == torch.bfloat16 else dict(rtol=1e-4, atol=1e-4)


SSM = [(4, 2, 32, 48, 4, 1), (6, 2, 24, 40, 4, 3), (3, 3, 19, 13, 1, 1), (5, 1, 33, 21, 2, 5), (8, 2, 128, 64, 4, 2), (2, 1, 64, 128, 4, 8),
       (2, 2, 200, 80, 6, 1), (1, 1, 72, 144, 4, 2), (3, 1, 256, 16, 3, 1), (2, 1, 300, 20, 4, 2), (2, 1, 16, 256, 4, 16)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", SSM, ids=lambda s: "x".join(map(str, s)))
def test_state_space(dev, dtype, sizes):
    """whole sequences in a batch, chunked and token by token; then portions of every small size, in slots that held others"""
    c = SsmCase(*sizes, dtype, dev)
    lens = [1, 64, 65, 150, 2]
    ps = [c.rows(n, 70 + i) for i, n in enumerate(lens)]
    wants = [c.want(p) for p in ps]
    for chunked in (False, True):
        for i, (got, (w, s)) in enumerate(zip(c.run([(4 - i, p, 0) for i, p in enumerate(ps)], chunked), wants)):
            close(got, w, **ssm_tol(dtype))
            close(c.state[4 - i], s, **state_tol(dtype))
    cuts = [0, 2, 3, 5, 70, 72, 73, 137, 138, 139, 140, 150]
    for n, (a, b) in enumerate(zip(cuts, cuts[1:])):
        parts = [(2, ps[3][a:b], a)]
        if n < 4:
            parts.append((0, ps[1][16 * n:16 * n + 16], 16 * n))
        outs = c.run(parts, chunked=n % 3 != 2)
        close(outs[0], wants[3][0][a:b], **ssm_tol(dtype))
        if n < 4:
            close(outs[1], wants[1][0][16 * n:16 * n + 16], **ssm_tol(dtype))
    for i in range(12):                                                # decoding from the first token on, two requests side by side
        outs = c.run([(3, ps[2][i:i + 1], i), (1, ps[1][i:i + 1], i)], chunked=False)
        close(outs[0], wants[2][0][i:i + 1], **ssm_tol(dtype))
        close(outs[1], wants[1][0][i:i + 1], **ssm_tol(dtype))


@pytest.mark.parametrize("sizes", [(2, 1, 64, 64, 4, 1), (3, 3, 24, 40, 3, 2), (1, 1, 128, 128, 4, 1)], ids=lambda s: "x".join(map(str, s)))
def test_state_space_in_segments(dev, sizes):
    """long portions: chunks run in segments side by side; requests of unequal length, then a second portion from the states; slow
    decays, so that the first tokens reach the end"""
    c = SsmCase(*sizes, torch.bfloat16, dev, a_log=(-5.0, 0.5), bias=(-1.0, 0.5))
    lens = [2100, 70, 1030, 512]
    ps = [c.rows(n, 30 + i) for i, n in enumerate(lens)]
    wants = [c.want(p) for p in ps]
    cut = [1500, 60, 1000, 1]
    for got, (w, _), n in zip(c.run([(i, p[:n], 0) for i, (p, n) in enumerate(zip(ps, cut))], True), wants, cut):
        close(got, w[:n], **ssm_tol(torch.bfloat16))
    for i, (got, (w, s), n) in enumerate(zip(c.run([(i, p[n:], n) for i, (p, n) in enumerate(zip(ps, cut))], True), wants, cut)):
        close(got, w[n:], **ssm_tol(torch.bfloat16))
        close(c.state[i], s, **state_tol(torch.bfloat16))


@pytest.mark.parametrize("a_log,bias", [((4.0, 1.0), (3.0, 2.0)), ((-6.0, 0.1), (-4.0, 0.5)), ((0.0, 4.0), (0.0, 4.0))])
def test_decays_of_every_strength(dev, a_log, bias):
    """from a state that is gone at the next token to one that hardly fades, beside each other in a chunk; big step projections"""
    c = SsmCase(6, 2, 32, 48, 4, 2, torch.bfloat16, dev, a_log=a_log, bias=bias)
    x = c.rows(200, 9)
    x[:, -6:] *= 3.0
    w, s = c.want(x)
    for chunked in (True, False):
        close(c.run([(1, x, 0)], chunked)[0], w, **ssm_tol(torch.bfloat16))
        close(c.state[1], s, **state_tol(torch.bfloat16))


def test_chunked_state_is_32_bit(dev):
    """the chunked form's state against a float64 recurrence over the same filtered rows: no trace of 16-bit products"""
    c = SsmCase(4, 2, 64, 64, 4, 1, torch.bfloat16, dev, a_log=(-3.0, 0.5), bias=(-1.0, 0.5))
    x = c.rows(640, 4)
    _, s = c.want(x)
    c.run([(0, x, 0)], True)
    e = (c.state[0].double().cpu() - s).abs() / s.abs().max()
    assert e.median() < 1e-6 and e.max() < 1e-3, (float(e.median()), float(e.max()))      # (the worst: an input rounded the other way)


def test_one_early_token_reaches_the_end(dev):
    """a state that does not fade: the row that stands out comes back when C asks for it, across chunks, portions and decoding"""
    c = SsmCase(2, 1, 64, 32, 1, 1, torch.bfloat16, dev, a_log=(-12.0, 0.0), bias=(0.0, 0.0))
    x = c.rows(300, 8, std=0.05)
    x[3] = c.rows(1, 9)[0] * 3
    for i in (63, 64, 65, 128, 299):
        x[i, c.inner + c.inner + c.n:c.inner + c.inner + 2 * c.n] = x[3, c.inner + c.inner:c.inner + c.inner + c.n]     # C of this row: B of that
    w, _ = c.want(x)
    y = c.want(torch.cat([x[:3], x[3:4] * 0, x[4:]]))[0]
    assert (w[299] - y[299]).abs().max() > 0.3
    close(c.run([(1, x, 0)], True)[0], w, **ssm_tol(torch.bfloat16))
    outs = [c.run([(2, x[a:b], a)], True)[0] for a, b in ((0, 60), (60, 62), (62, 127), (127, 129), (129, 290))]
    outs += [c.run([(2, x[i:i + 1], i)], False)[0] for i in range(290, 300)]
    close(torch.cat(outs), w, **ssm_tol(torch.bfloat16))


# ------------------------------------------------------------------------------------------------ routed experts
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("t,width,experts,top,ff", [(7, 96, 6, 2, 40), (70, 128, 8, 3, 128), (33, 100, 5, 1, 21), (300, 320, 9, 4, 96),
                                                    (90, 256, 40, 4, 64), (20, 128, 130, 16, 16), (3, 200, 4, 4, 24),
                                                    (1500, 72, 20, 2, 16), (1400, 256, 4, 2, 256), (1, 176, 11, 1, 72)])
def test_routed_experts(dev, dtype, t, width, experts, top, ff):
    """sigmoid scores that scale what an expert reads, squared relu, no gate; widely spread router logits"""
    from vllm_omni_amd import ops
    from vllm_omni_amd.moe import RoutedExperts

    m = RoutedExperts(width, experts, top, ff, dtype, dev, act="relu_squared", scores="sigmoid", bias=False, weigh_input=True)
    w = {"router": rnd(experts, width, dtype=dtype, std=4 * width ** -0.5, seed=1)}
    for e in range(experts):
        w[f"e{e}.up"], w[f"e{e}.down"] = rnd(ff, width, dtype=dtype, std=width ** -0.5, seed=10 + 2 * e), rnd(width, ff, dtype=dtype, std=ff ** -0.5, seed=11 + 2 * e)
    for name, dst in m.named_weights(""):
        assert tuple(dst.shape) == tuple(w[name].shape)
        dst.copy_(w[name])
    assert len(dict(m.named_weights(""))) == len(w)
    h = rnd(t, width, dtype=dtype, seed=5)
    hg = torch.full((t, width + 8), 9.0, dtype=dtype, device=dev)[:, :width]
    hg.copy_(h)
    wd = {k: v.double() for k, v in w.items()}
    idx, p = ref.route(h.double(), wd["router"], top)
    ids, wt, _ = ops.moe_route(ops.moe_router_logits(hg, m.router), top, False, want_counts=False, sigmoid=True)
    assert torch.equal(ids.cpu().long().sort(-1).values, idx.sort(-1).values)
    got = torch.zeros(t, experts, dtype=torch.float64).scatter_(1, ids.cpu().long(), wt.cpu().double())
    close(got, torch.zeros(t, experts, dtype=torch.float64).scatter_(1, idx, p), rtol=1e-5, atol=1e-6)
    er = m(hg)
    assert er.weights is None and er.top == top
    x = torch.zeros(t, width, device=dev)
    ops.stream_norm2(x, torch.zeros(t, width, dtype=dtype, device=dev), torch.zeros(width, dtype=dtype, device=dev), None, 1e-6,
                     torch.empty(t, width, dtype=dtype, device=dev), experts=er)
    close(x, ref.routed_experts(h.double(), lambda n: wd[n], top), **(dict(rtol=2 ** -6, atol=0.06) if dtype == torch.bfloat16
                                                                     else dict(rtol=1e-4, atol=2e-5)))


def test_sigmoid_routing_of_far_logits(dev):
    """chosen by the logits, so that scores which round to 0 or 1 still have an order; normalised on request; a bias"""
    from vllm_omni_amd import ops

    lg = torch.tensor([[30.0, 40.0, 35.0, -5.0], [-120.0, -110.0, -130.0, -115.0], [80.0, -90.0, -100.0, -95.0]], device=dev)
    ids, w, counts = ops.moe_route(lg, 2, False, sigmoid=True)
    assert ids.tolist() == [[1, 2], [1, 3], [0, 1]] and counts.tolist() == [1, 3, 1, 1]
    close(w, torch.sigmoid(lg.double().cpu()).gather(1, ids.cpu().long()), rtol=1e-5, atol=1e-30)
    ids, w, _ = ops.moe_route(lg, 2, True, want_counts=False, sigmoid=True, bias=torch.tensor([0.0, -20.0, 0.0, 0.0], device=dev))
    assert ids.tolist()[0] == [2, 0]
    close(w[0].sum(), torch.tensor(1.0), rtol=1e-6, atol=0)
