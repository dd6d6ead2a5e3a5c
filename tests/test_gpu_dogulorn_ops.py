"""Every kernel of the 32-bit-residual decoders against the plain restatement, one mechanism at a time."""
import pytest
import torch

from oracle import ref_dogulorn as ref

pytestmark = pytest.mark.gpu
DTYPES = [torch.bfloat16, torch.float32]


def tol(dtype, scale=1.0):
    return dict(rtol=2 ** -7, atol=0.012 * scale) if dtype == torch.bfloat16 else dict(rtol=2e-5, atol=2e-5 * scale)


def rnd(*shape, dtype=torch.float32, std=1.0, seed=0):
    return (torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * std).to(dtype)


def close(got, want, **kw):
    torch.testing.assert_close(got.double().cpu(), want.double(), **kw)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [40, 100, 2304, 8192])
def test_residual_norm(dev, dtype, width):
    from vllm_omni_amd import ops

    x, y = rnd(5, width, std=3.0, seed=1), rnd(5, width, dtype=dtype, std=0.01, seed=2)
    a, b = rnd(width, dtype=dtype, seed=3), rnd(width, dtype=dtype, seed=4)
    eps = 3e-5                                         # of the order of y's own mean square: a misplaced eps shows
    x1 = x.double() + ref.rms_norm(y.double(), a.double(), eps)
    for pre, h_want in ((b, ref.rms_norm(x1, b.double(), eps)), (None, x1)):
        xg = x.to(dev)
        h = ops.residual_norm(xg, y.to(dev), a.to(dev), None if pre is None else pre.to(dev), eps)
        close(xg, x1, rtol=1e-5, atol=1e-5)            # the stream stays 32-bit in both modes
        close(h, h_want, **tol(dtype, 4.0))
    xg = x.to(dev)
    assert ops.residual_norm(xg, y.to(dev), a.to(dev), None, eps, want_h=False) is None
    close(xg, x1, rtol=1e-5, atol=1e-5)


def test_residual_norm_takes_split_k_partials(dev):
    from vllm_omni_amd import ops

    x, part = rnd(3, 256, seed=1), rnd(4, 3, 256, seed=2)
    a = rnd(256, dtype=torch.bfloat16, seed=3)
    gp = part.to(dev)
    ops._LINEAR_GEN[gp.device] = ops._LINEAR_GEN.get(gp.device, 0) + 1
    p = ops.SplitKPartials(gp, 4, 3, 256, None, torch.bfloat16, (3,), gp.device, ops._LINEAR_GEN[gp.device])
    xg = x.to(dev)
    ops.residual_norm(xg, p, a.to(dev), None, 1e-6)
    close(xg, x.double() + ref.rms_norm(part.double().sum(0), a.double(), 1e-6), rtol=1e-5, atol=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [48, 50])
def test_pair_embed_norm(dev, dtype, width):
    from vllm_omni_amd import ops

    vocab, buckets, mp, mc = 70, 53, 41, 13
    table, pairs, w = rnd(vocab, width, dtype=dtype, seed=1), rnd(buckets + 1, width, dtype=dtype, seed=2), rnd(width, dtype=dtype, seed=3)
    toks = [3, 69, 69, 0, 17, 5]
    want = ref.embed(toks, table.double(), pairs.double(), 2.5, mp, mc)
    ids = torch.tensor(toks, device=dev)
    # a whole prompt (the previous tokens given), then the same tokens one by one through the slot
    prev = torch.tensor([-1] + toks[:-1], device=dev)
    slots = torch.full((6,), -1, dtype=torch.int32, device=dev)
    slots[-1] = 2
    last = torch.full((4,), 11, dtype=torch.int64, device=dev)
    x, h = ops.pair_embed_norm(table.to(dev), pairs.to(dev), w.to(dev), ids, prev, slots, last, torch.arange(6, device=dev), 2.5, mp, mc, 1e-5)
    close(x, want, rtol=1e-6, atol=1e-6)
    close(h, ref.rms_norm(want, w.double(), 1e-5), **tol(dtype, 3.0))
    assert last.tolist() == [11, 11, 5, 11]
    one = torch.tensor([1], dtype=torch.int32, device=dev)
    for i, t in enumerate(toks):      # the slot holds another request's token at first: position 0 ignores it
        x, _ = ops.pair_embed_norm(table.to(dev), pairs.to(dev), w.to(dev), torch.tensor([t], device=dev), None, one, last,
                                   torch.tensor([i], device=dev), 2.5, mp, mc, 1e-5)
        close(x[0], want[i], rtol=1e-6, atol=1e-6)
        assert last[1].item() == t


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim", [24, 13])
def test_gates(dev, dtype, dim):
    from vllm_omni_amd import ops

    z, table = rnd(9, dim, dtype=dtype, std=2.0, seed=1), rnd(30, 4 * dim, dtype=dtype, seed=2)
    ids = torch.tensor([0, 29, 4, 4, 7, 1, 2, 3, 28])
    got = ops.gelu_lookup_mul(z.to(dev), table.to(dev), ids.to(dev), 2 * dim)
    close(got, ref.gelu_tanh(z.double()) * table.double()[ids, 2 * dim:3 * dim], **tol(dtype))
    gu = rnd(9, 2 * dim, dtype=dtype, std=3.0, seed=3)
    g, u = gu.double().split(dim, 1)
    eye = torch.eye(dim, dtype=torch.float64)
    for limit in (0.6, 4.0):      # the gate has no lower clamp, the up projection has both
        want = (g.clamp(max=limit) * ref.sigmoid(1.702 * g.clamp(max=limit)) * (u.clamp(-limit, limit) + 1)) @ eye
        close(ops.clamped_glu(gu.to(dev), 1.702, limit), want, **tol(dtype, 4.0))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nq,nc", [(48, 64), (33, 35), (1536, 512), (24, 0)])
def test_latent_norm_cache(dev, dtype, nq, nc):
    from vllm_omni_amd import ops

    x = rnd(5, nq + nc, dtype=dtype, std=0.02, seed=1)
    wq, wc = rnd(nq, dtype=dtype, seed=2), rnd(max(nc, 1), dtype=dtype, seed=3)
    cache = torch.zeros(4, 8, max(nc, 1), dtype=dtype, device=dev)
    slots = torch.tensor([9, -1, 31, 8, 16], device=dev)
    got = ops.latent_norm_cache(x.to(dev), wq.to(dev), wc.to(dev) if nc else None, cache if nc else None, slots if nc else None, 1e-4)
    close(got, ref.rms_norm(x[:, :nq].double(), wq.double(), 1e-4), **tol(dtype, 3.0))
    if nc:
        want = torch.zeros(32, nc, dtype=torch.float64)
        for i, s in enumerate(slots.tolist()):
            if s >= 0:
                want[s] = ref.rms_norm(x[i, nq:].double(), wc.double(), 1e-4)
        close(cache.view(32, nc), want, **tol(dtype, 3.0))


@pytest.mark.parametrize("rows,h,n,k", [(1, 3, 40, 24), (70, 2, 128, 512), (130, 5, 72, 200), (64, 36, 64, 128)])
def test_head_gemm(dev, rows, h, n, k):
    from vllm_omni_amd import ops

    for dtype in DTYPES:
        x, w = rnd(rows, h * k, dtype=dtype, seed=1), rnd(h, n, k, dtype=dtype, std=k ** -0.5, seed=2)
        want = torch.stack([x.view(rows, h, k)[:, i].double() @ w[i].double().T for i in range(h)], 1).reshape(rows, h * n)
        close(ops.head_gemm(x.to(dev), w.to(dev)), want, **tol(dtype, 2.0))
        close(ops.head_gemm(x.to(dev), w.transpose(1, 2).contiguous().to(dev), transposed=True), want, **tol(dtype, 2.0))
        if dtype == torch.bfloat16:
            close(ops.head_gemm_nt(x.to(dev), w.to(dev)), want, **tol(dtype, 2.0))


def rows_close(got, want):
    # a wrong window moves the rows whose outstanding key it is about by the spread of the values itself
    e = (got.double().cpu() - want).pow(2).mean(-1).sqrt() / want.std()
    assert e.max() < 0.04 and e.mean() < 0.012, (e.max(), e.mean(), int(e.argmax()))


def paged(lat, tables, bs, nb, dtype, dev):
    """cache holding each request's latents at its table's blocks; everything else is poison"""
    cache = torch.full((nb, bs, lat[0].shape[1]), 40.0, dtype=dtype)
    for c, t in zip(lat, tables):
        for i in range(c.shape[0]):
            cache[t[i // bs], i % bs] = c[i].to(dtype)
    return cache.to(dev)


def tables_for(lens, bs, seed=0):
    need = [-(-n // bs) for n in lens]
    perm = (torch.randperm(sum(need), generator=torch.Generator().manual_seed(seed)) + 1).tolist()
    out, at = [], 0
    for n in need:
        out.append(perm[at:at + n])
        at += n
    t = torch.zeros(len(lens), max(need), dtype=torch.int32)
    for i, b in enumerate(out):
        t[i, :len(b)] = torch.tensor(b)
    return out, t, sum(need) + 1


@pytest.mark.parametrize("h,dim,vdim,rank,window,bs", [(4, 32, 64, 64, 40, 16), (3, 24, 40, 72, 5, 8), (20, 64, 128, 512, 300, 16),
                                                       (36, 64, 64, 128, 1, 16), (16, 128, 128, 256, 64, 32), (40, 16, 8, 8, 65, 16)])
def test_latent_attention_kernels_agree_with_the_direct_form(dev, h, dim, vdim, rank, window, bs):
    """decode, prompt portions of several sizes and the any-size kernel on one paged cache, against attention on expanded
    k and v; keys just inside and just outside the window get a score that stands out"""
    from vllm_omni_amd import ops

    dt, scale = torch.bfloat16, dim ** -0.5
    lens = [1, 7, window, window + 1, 333, 450]
    lat = [rnd(n, rank, dtype=dt, seed=10 + i) for i, n in enumerate(lens)]
    uk, uv = rnd(h, dim, rank, dtype=dt, std=rank ** -0.5, seed=1), rnd(h, vdim, rank, dtype=dt, std=rank ** -0.5, seed=2)
    # a key that a query meets at the window's last place (distance window - 1) and one at the first place outside
    for c in lat:
        n = c.shape[0]
        for d in (window - 1, window):
            if n > d:
                c[n - 1 - d] *= 4.0
    bt, table, nb = tables_for(lens, bs)
    cache = paged(lat, bt, bs, nb, dt, dev)
    qs = [rnd(n, h * dim, dtype=dt, seed=30 + i) for i, n in enumerate(lens)]

    def want(i):
        c = lat[i].double()
        k = torch.stack([c @ uk[j].double().T for j in range(h)], 1)
        v = torch.stack([c @ uv[j].double().T for j in range(h)], 1)
        return ref.window_attention(qs[i].double().view(-1, h, dim), k, v, scale, window).reshape(-1, h * vdim)

    wants = [want(i) for i in range(len(lens))]
    ukt = uk.transpose(1, 2).contiguous().to(dev)
    n = len(lens)
    sl = torch.tensor(lens, dtype=torch.int32, device=dev)
    tb = table.to(dev)
    # decode: the last token of every request (and a padded row); the launch bound far above the lengths as in a graph
    q1 = torch.cat([q[-1:] for q in qs] + [qs[0][:1]]).to(dev)
    sl1 = torch.cat([sl, torch.zeros(1, dtype=torch.int32, device=dev)])
    tb1 = torch.cat([tb, torch.zeros_like(tb[:1])])
    qa = ops.head_gemm_nt(q1, ukt)
    for bound in (max(lens), 4096):
        oa = ops.latent_decode(qa, cache, tb1, sl1, h, window, bound, scale)
        o = ops.head_gemm_nt(oa, uv.to(dev))
        rows_close(o[:n], torch.cat([w[-1:] for w in wants]))
        assert not o[n].any()
    qsl1 = torch.arange(n + 2, dtype=torch.int32, device=dev)
    rows = ops.latent_attn_rows(qa, cache, tb1, sl1, qsl1, h, window, scale)
    rows_close(ops.head_gemm_nt(rows, uv.to(dev))[:n], torch.cat([w[-1:] for w in wants]))
    # prompt portions: the last m tokens of every request in one launch
    for portion in (2, 63, 129, 450):
        m = [min(portion, k) for k in lens]
        qsl = torch.tensor([0] + m).cumsum(0).to(torch.int32)
        q = torch.cat([x[-k:] for x, k in zip(qs, m)]).to(dev)
        seen = [min(ln, k + window - 1) for ln, k in zip(lens, m)]
        start = torch.tensor([0] + [-(-s // 64) * 64 for s in seen]).cumsum(0).to(torch.int32)
        ctx = ops.latent_gather(cache, start.to(dev), int(start[-1]), tb, sl, qsl.to(dev), window)
        for i in range(n):
            a = int(start[i])
            assert torch.equal(ctx[a:a + seen[i]].cpu(), lat[i][lens[i] - seen[i]:]) and not ctx[a + seen[i]:int(start[i + 1])].any()
        kk = torch.nn.functional.linear(ctx, uk.view(h * dim, rank).to(dev))
        vt = torch.nn.functional.linear(uv.view(h * vdim, rank).to(dev), ctx)
        out = torch.zeros(q.shape[0], h * vdim, dtype=dt, device=dev)
        ops.latent_prefill(out, q, kk, vt, start.to(dev), sl, qsl.to(dev), max(m), h, window, scale)
        rows_close(out, torch.cat([w[-k:] for w, k in zip(wants, m)]))


@pytest.mark.parametrize("h,dim,vdim,rank,window", [(3, 20, 27, 35, 7), (2, 32, 16, 64, 300)])
def test_latent_rows_in_32_bit(dev, h, dim, vdim, rank, window):
    from vllm_omni_amd import ops

    lens, scale = [1, 12, 301, 320], 0.4
    lat = [rnd(n, rank, seed=10 + i) for i, n in enumerate(lens)]
    uk, uv = rnd(h, dim, rank, std=rank ** -0.5, seed=1), rnd(h, vdim, rank, std=rank ** -0.5, seed=2)
    bt, table, nb = tables_for(lens, 16)
    cache = paged(lat, bt, 16, nb, torch.float32, dev)
    qs = [rnd(n, h * dim, std=2.0, seed=30 + i) for i, n in enumerate(lens)]
    qsl = torch.tensor([0] + lens).cumsum(0).to(torch.int32).to(dev)
    qa = ops.head_gemm(torch.cat(qs).to(dev), uk.to(dev), transposed=True)
    oa = ops.latent_attn_rows(qa, cache, table.to(dev), torch.tensor(lens, dtype=torch.int32, device=dev), qsl, h, window, scale)
    got = ops.head_gemm(oa, uv.to(dev))
    want = []
    for i, c in enumerate(lat):
        k = torch.stack([c.double() @ uk[j].double().T for j in range(h)], 1)
        v = torch.stack([c.double() @ uv[j].double().T for j in range(h)], 1)
        want.append(ref.window_attention(qs[i].double().view(-1, h, dim), k, v, scale, window).reshape(-1, h * vdim))
    close(got, torch.cat(want), rtol=1e-5, atol=2e-5)


class DeltaCase:
    """one gated-delta layer's tensors, with the plain mixer around the same projections"""

    def __init__(self, h, kvh, dim, vdim, taps, dtype, dev, slots=5, seed=0):
        self.h, self.kvh, self.dim, self.vdim, self.taps, self.dtype, self.dev = h, kvh, dim, vdim, taps, dtype, dev
        kd, hv = kvh * dim, h * vdim
        self.ch, self.cols = 2 * kd + hv, 2 * kd + 2 * hv + 2 * h
        self.ld = -(-self.cols // 16) * 16
        self.conv = rnd(self.ch, taps, dtype=dtype, std=0.6, seed=seed + 1)
        self.a_log, self.dt = rnd(h, std=0.7, seed=seed + 2) - 1.5, rnd(h, std=0.5, seed=seed + 3)
        self.norm = rnd(vdim, dtype=dtype, std=0.3, seed=seed + 4) + 1
        self.state = torch.full((slots, h, dim, vdim), 7.0, device=dev)         # slots start dirty
        self.ring = torch.full((slots, taps, self.ch), 7.0, dtype=dtype, device=dev)

    def proj(self, n, seed):
        p = rnd(n, self.ld, dtype=self.dtype, seed=seed)
        p[:, self.cols:] = 9.0
        return p

    def want(self, p):
        t, kd, hv, h = p.shape[0], self.kvh * self.dim, self.h * self.vdim, self.h
        p = p.double()
        c = self.conv.double()
        q = ref.silu(ref.causal_conv(p[:, :kd], c[:kd])).view(t, self.kvh, self.dim)
        k = ref.silu(ref.causal_conv(p[:, kd:2 * kd], c[kd:2 * kd])).view(t, self.kvh, self.dim)
        v = ref.silu(ref.causal_conv(p[:, 2 * kd:self.ch], c[2 * kd:])).view(t, h, self.vdim)
        of = [i // (h // self.kvh) for i in range(h)]
        q, k = ref.unit(q) * self.dim ** -0.5, ref.unit(k)
        gate, b, a = p[:, self.ch:self.ch + hv], p[:, self.ch + hv:self.ch + hv + h], p[:, self.ch + hv + h:self.cols]
        g = torch.exp(-torch.exp(self.a_log.double()) * ref.softplus(a + self.dt.double()))
        o, s = ref.delta_rule(q[:, of], k[:, of], v, ref.sigmoid(b), g)
        return (ref.rms(o, 1e-5) * self.norm.double() * ref.silu(gate).view(t, h, self.vdim)).reshape(t, hv), s

    def run(self, parts, chunked):
        """parts: [(slot, projection rows, tokens before them)] in one call -> output rows per part"""
        from vllm_omni_amd import ops

        dev, i32 = self.dev, torch.int32
        p = torch.cat([x for _, x, _ in parts]).to(dev)
        lens = [x.shape[0] for _, x, _ in parts]
        qsl = torch.tensor([0] + lens).cumsum(0).to(i32).to(dev)
        seq = torch.tensor([b + n for (_, _, b), n in zip(parts, lens)], dtype=i32, device=dev)
        slots = torch.tensor([s for s, _, _ in parts], dtype=i32, device=dev)
        out = torch.zeros(p.shape[0], self.h * self.vdim, dtype=self.dtype, device=dev)
        args = (p, self.conv.to(dev), self.a_log.to(dev), self.dt.to(dev), self.norm.to(dev), self.state, self.ring, slots, qsl, seq,
                self.kvh, 1e-5, out)
        if chunked:
            ops.gated_delta_chunked(*args, 0, len(parts), 0, max(lens))
        else:
            ops.gated_delta_step(*args, 0, len(parts))
        return list(out.split(lens))


DELTA_SIZES = [(4, 2, 32, 64, 4), (6, 3, 24, 40, 3), (3, 3, 18, 30, 2), (2, 1, 33, 21, 1), (9, 3, 64, 128, 4), (2, 2, 128, 64, 6), (2, 1, 256, 256, 4)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", DELTA_SIZES, ids=lambda s: "x".join(map(str, s)))
def test_gated_delta(dev, dtype, sizes):
    """whole prompts, portions cut anywhere (down to single tokens) and unequal batches, chunked and token by token"""
    t = dict(rtol=2 ** -6, atol=0.03) if dtype == torch.bfloat16 else dict(rtol=1e-4, atol=1e-4)
    c = DeltaCase(*sizes, dtype, dev)
    lens = [1, 64, 65, 150, 2]
    ps = [c.proj(n, 50 + i) for i, n in enumerate(lens)]
    wants = [c.want(p) for p in ps]
    for chunked in (False, True):
        outs = c.run([(4 - i, p, 0) for i, p in enumerate(ps)], chunked)
        for i in range(len(lens)):
            close(outs[i], wants[i][0], **t)
            close(c.state[4 - i], wants[i][1], rtol=1e-4, atol=2e-5)
    # cut: portions of changing size, the two kernels in turn, beside another request in the same call
    cuts = [0, 2, 3, 5, 70, 72, 73, 137, 138, 139, 140, 150]
    for k, (a, b) in enumerate(zip(cuts, cuts[1:])):
        parts = [(2, ps[3][a:b], a)]
        if k < 4:
            parts.append((0, ps[1][16 * k:16 * k + 16], 16 * k))
        outs = c.run(parts, chunked=k % 3 != 2)
        close(outs[0], wants[3][0][a:b], **t)
        if k < 4:
            close(outs[1], wants[1][0][16 * k:16 * k + 16], **t)
    close(c.state[2], wants[3][1], rtol=1e-4, atol=2e-5)


def test_gated_delta_repeated_keys_stay_exact(dev):
    """equal tokens give equal keys: the chunk's triangular system is then as far from the identity as it gets"""
    c = DeltaCase(2, 1, 32, 32, 4, torch.float32, dev)
    p = c.proj(1, 5).repeat(200, 1)
    p[:, c.ch + 64:c.ch + 66] = 4.0      # write strength near 1
    p[:, c.ch + 66:c.ch + 68] = -6.0     # hardly any decay
    w, s = c.want(p)
    close(c.run([(0, p, 0)], True)[0], w, rtol=1e-3, atol=1e-3)
    close(c.state[0], s, rtol=1e-3, atol=1e-4)
