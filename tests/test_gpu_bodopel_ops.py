"""Every kernel of attention with mixed heads and of the filters in front of sublayers, one mechanism at a time, against the
plain restatement."""
import pytest
import torch

from oracle import ref_bodopel as ref
from test_gpu_dogulorn_ops import DTYPES, close, rnd, tables_for, tol

pytestmark = pytest.mark.gpu


def bf(x):
    return x.bfloat16().float()


# ------------------------------------------------------------------------------------------------ rows
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,taps", [(40, 4), (100, 2), (2304, 7), (64, 1), (4100, 3)])
def test_filter_in_portions_and_token_by_token(dev, dtype, width, taps):
    """unequal requests in portions (1 and 2 tokens, fewer than the taps, longer than a workgroup's rows), rings dirty from
    the start, a slot that is used again; then one-token rows in the residual add's launch"""
    from vllm_omni_amd import ops

    w = rnd(width, taps, dtype=dtype, std=0.5, seed=1)
    ring = torch.full((4, taps - 1, width), 77.0, dtype=dtype, device=dev) if taps > 1 else None
    conv = ops.ConvRing(w.t().contiguous().to(dev), ring)
    slots = torch.tensor([2, 0, 3], dtype=torch.int32)
    for again in range(2):
        seqs = [rnd(n, width, dtype=dtype, seed=10 * again + i) for i, n in enumerate((80, 49, 9))]
        want = [ref.with_conv(s.double(), w.double()) for s in seqs]
        at = [0, 0, 0]
        for sizes in ((33, 1, 2), (2, 40, 1), (1, 2, 2), (35, 3, 1)):
            qsl = torch.tensor([0, *torch.tensor(sizes).cumsum(0).tolist()], dtype=torch.int32)
            lens = torch.tensor([a + n for a, n in zip(at, sizes)], dtype=torch.int32)
            h = torch.cat([s[a:a + n] for s, a, n in zip(seqs, at, sizes)]).to(dev)
            y = ops.input_conv(h, conv, slots.to(dev), qsl.to(dev), lens.to(dev), 3, max(sizes))
            close(y, torch.cat([x[a:a + n] for x, a, n in zip(want, at, sizes)]), **tol(dtype, 2.0))
            at = [a + n for a, n in zip(at, sizes)]
        for _ in range(3):      # one row each: the stream's add, norm and filter together
            rows = torch.stack([s[a] for s, a in zip(seqs, at)])
            pos = torch.tensor(at)
            x, y = torch.zeros(3, width, device=dev), torch.empty(3, width, dtype=dtype, device=dev)
            ops.residual_add_norm_conv(x, rows.to(dev), None, 1e-6, y, conv=conv, slots=slots.to(dev), positions=pos.to(dev))
            close(y, torch.stack([v[a] for v, a in zip(want, at)]), **tol(dtype, 2.0))
            at = [a + 1 for a in at]


@pytest.mark.parametrize("dtype", DTYPES)
def test_filter_of_the_first_tokens_one_by_one(dev, dtype):
    """from position 0 on, in a dirty ring: nothing before the start counts"""
    from vllm_omni_amd import ops

    width, taps = 48, 4
    w, s = rnd(width, taps, dtype=dtype, seed=1), rnd(9, width, dtype=dtype, seed=2)
    want = ref.with_conv(s.double(), w.double())
    for fused in (True, False):
        conv = ops.ConvRing(w.t().contiguous().to(dev), torch.full((2, taps - 1, width), 50.0, dtype=dtype, device=dev))
        slot = torch.tensor([1], dtype=torch.int32, device=dev)
        for t in range(9):
            row = s[t:t + 1].to(dev)
            if fused:
                y = torch.empty_like(row)
                ops.residual_add_norm_conv(torch.zeros(1, width, device=dev), row, None, 1e-6, y, conv=conv, slots=slot,
                                           positions=torch.tensor([t], device=dev))
            else:
                y = ops.input_conv(row, conv, slot, torch.tensor([0, 1], dtype=torch.int32, device=dev),
                                   torch.tensor([t + 1], dtype=torch.int32, device=dev), 1, 1)
            close(y, want[t:t + 1], **tol(dtype, 2.0))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [40, 100, 8192])
def test_residual_add_with_a_row_for_all(dev, dtype, width):
    from vllm_omni_amd import ops

    x, y, step = rnd(5, width, std=0.2, seed=1), rnd(5, width, dtype=dtype, std=0.1, seed=2), rnd(width, dtype=dtype, std=0.2, seed=3)
    w, eps = rnd(width, dtype=dtype, std=0.3, seed=4), 3e-2       # of the order of the rows' mean square: a misplaced eps shows
    for add in (None, step):
        x1 = x.double() + y.double() + (0 if add is None else add.double())
        xg, h = x.to(dev), torch.empty(5, width, dtype=dtype, device=dev)
        ops.residual_add_norm_conv(xg, y.to(dev), w.to(dev), eps, h, 1.0, None if add is None else add.to(dev))
        close(xg, x1, rtol=1e-5, atol=1e-5)
        close(h, ref.norm_about_one(x1, w.double(), eps), **tol(dtype, 2.0))


def test_residual_add_and_squared_relu_take_partials(dev):
    from vllm_omni_amd import ops

    x, part = rnd(3, 256, seed=1), rnd(4, 3, 256, seed=2)
    gp = part.to(dev)
    ops._LINEAR_GEN[gp.device] = ops._LINEAR_GEN.get(gp.device, 0) + 1
    p = ops.SplitKPartials(gp, 4, 3, 256, None, torch.bfloat16, (3,), gp.device, ops._LINEAR_GEN[gp.device])
    xg, h = x.to(dev), torch.empty(3, 256, dtype=torch.bfloat16, device=dev)
    ops.residual_add_norm_conv(xg, p, None, 1e-6, h)
    close(xg, x.double() + part.double().sum(0), rtol=1e-5, atol=1e-5)
    close(ops.relu_squared(p), ref.relu_squared(part.double().sum(0)), **tol(torch.bfloat16))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [24, 13])
def test_squared_relu(dev, dtype, ff):
    from vllm_omni_amd import ops

    z = rnd(9, ff, dtype=dtype, std=2.0, seed=1)
    close(ops.relu_squared(z.to(dev)), ref.relu_squared(z.double()), **tol(dtype))


@pytest.mark.parametrize("m,n,k", [(1, 256, 256), (7, 48, 512), (32, 6144, 2048), (200, 1024, 128), (5, 64, 16384)])
def test_up_projection_with_squared_relu(dev, m, n, k):
    """with and without slabs to sum"""
    from vllm_omni_amd import ops

    x, w = rnd(m, k, dtype=torch.bfloat16, seed=1), rnd(n, k, dtype=torch.bfloat16, std=k ** -0.5, seed=2)
    close(ops.linear_relu_squared(x.to(dev), w.to(dev)), ref.relu_squared(x.double() @ w.double().T), **tol(torch.bfloat16))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [48, 50])
def test_embedding_with_positions(dev, dtype, width):
    """scaled token rows, position rows that are not scaled, a pass's row, tokens and positions outside their tables, filter"""
    from vllm_omni_amd import ops

    table, pos_t, step = rnd(30, width, dtype=dtype, seed=1), rnd(20, width, dtype=dtype, seed=2), rnd(width, dtype=dtype, seed=3)
    w, eps = rnd(width, dtype=dtype, std=0.3, seed=4), 0.5
    ids, pos = torch.tensor([3, 29, 0, 29, 30, 5]), torch.tensor([0, 19, 7, 7, 2, 20])
    known = torch.cat([table.double()[ids[:4]] * 2.5, torch.zeros(1, width, dtype=torch.float64), table.double()[5:6] * 2.5])
    placed = torch.cat([pos_t.double()[pos[:5]], torch.zeros(1, width, dtype=torch.float64)])
    for add in (None, step):
        want = known + placed + (0 if add is None else add.double())
        x, h = torch.empty(6, width, device=dev), torch.empty(6, width, dtype=dtype, device=dev)
        ops.embed_pos_norm(table.to(dev), ids.to(dev), x, w.to(dev), eps, h, pos.to(dev), 2.5, pos_t.to(dev),
                           None if add is None else add.to(dev), 1.0)
        close(x, want, rtol=1e-6, atol=1e-6)
        close(h, ref.norm_about_one(want, w.double(), eps), **tol(dtype, 2.0))
    cw = rnd(width, 2, dtype=dtype, std=0.5, seed=5)
    ring = rnd(6, 1, width, dtype=dtype, seed=6)
    x, h = torch.empty(6, width, device=dev), torch.empty(6, width, dtype=dtype, device=dev)
    rg = ring.to(dev)
    ops.embed_pos_norm(table.to(dev), ids.to(dev), x, w.to(dev), eps, h, pos.to(dev), 2.5, pos_t.to(dev), None, 1.0,
                       ops.ConvRing(cw.t().contiguous().to(dev), rg), torch.arange(6, dtype=torch.int32, device=dev))
    n = ref.norm_about_one(known + placed, w.double(), eps)
    before = torch.where(pos[:, None] > 0, ring[:, 0].double(), torch.zeros(1, dtype=torch.float64))
    close(h, n + cw[:, 1].double() * n + cw[:, 0].double() * before, **tol(dtype, 4.0))
    close(rg[:, 0], n, **tol(dtype, 2.0))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("h,g,dim,vdim,hd", [(6, 2, 40, 24, 64), (5, 1, 21, 35, 40), (32, 8, 128, 128, 128), (4, 4, 16, 64, 64)])
def test_row_norm_and_cache_write(dev, dtype, h, g, dim, vdim, hd):
    from vllm_omni_amd import ops

    rows, bs, eps = 7, 16, 0.3
    n = (h + g) * dim + g * vdim
    x = rnd(rows, n + 8, dtype=dtype, seed=1)[:, :n]
    wq, wk = rnd(h * dim, dtype=dtype, seed=2), rnd(g * dim, dtype=dtype, seed=3)
    kc, vc = (torch.full((3, bs, g, hd), 9.0, dtype=dtype, device=dev) for _ in range(2))
    slots = torch.tensor([0, 47, 16, 17, 31, -1, 5])
    q = ops.row_norm_cache(x.to(dev), wq.to(dev), wk.to(dev), kc, vc, slots.to(dev), h, dim, vdim, eps)
    xd = x.double()
    wantq = ref.rms(xd[:, :h * dim], eps) * wq.double()
    wantk = ref.rms(xd[:, h * dim:(h + g) * dim], eps) * wk.double()
    q = q.view(rows, h, hd)
    close(q[..., :dim].reshape(rows, -1), wantq, **tol(dtype, 2.0))
    assert not q[..., dim:].any()
    live = slots >= 0
    kk, vv = (c.view(-1, g, hd)[slots[live].to(dev)] for c in (kc, vc))
    close(kk[..., :dim].reshape(int(live.sum()), -1), wantk[live], **tol(dtype, 2.0))
    close(vv[..., :vdim].reshape(int(live.sum()), -1), xd[live][:, (h + g) * dim:], rtol=0, atol=0)
    assert not kk[..., dim:].any() and not vv[..., vdim:].any()
    untouched = torch.ones(3 * bs, dtype=torch.bool)
    untouched[slots[live]] = False
    assert (kc.view(-1, g, hd)[untouched.to(dev)] == 9).all() and (vc.view(-1, g, hd)[untouched.to(dev)] == 9).all()


# ------------------------------------------------------------------------------------------------ attention
def attention_case(lens, h, g, dim, vdim, hd, window, dtype, seed=0, loud=()):
    """per request q, k, v; ``loud``: (request, row, key) whose product stands out in one head"""
    out = []
    for i, n in enumerate(lens):
        q, k, v = (rnd(n, x, d, dtype=dtype, seed=seed + 10 * i + j) for j, (x, d) in enumerate(((h, dim), (g, dim), (g, vdim))))
        out.append([q.float(), k.float(), v.float()])
    for r, i, j in loud:
        q, k, _ = out[r]
        hh = (i + j) % h
        q[i, hh] = bf(k[j, hh // (h // g)] * 4)
    return out


def paged(reqs, lens, bs, g, hd, dtype, dev, seed=4):
    tabs, table, nb = tables_for(lens, bs, seed=seed)
    kc, vc = (torch.full((nb, bs, g, hd), 1e4, dtype=dtype) for _ in range(2))     # rows of no request: would show at once
    for (q, k, v), t in zip(reqs, tabs):
        for p in range(k.shape[0]):
            at = t[p // bs], p % bs
            kc[at], vc[at] = 0, 0
            kc[at][:, :k.shape[2]], vc[at][:, :v.shape[2]] = k[p], v[p]
    return kc.to(dev), vc.to(dev), table.to(dev)


def laid_out(q, hd, dtype, dev):
    out = torch.zeros(q.shape[0], q.shape[1], hd, dtype=dtype)
    out[..., :q.shape[2]] = q
    return out.flatten(1).to(dev)


CASES = [  # heads, kv heads, dim, vdim, laid out, window, cap, block
    (6, 2, 40, 48, 64, 40, 6.0, 16), (8, 1, 64, 64, 64, 16, 20.0, 16), (32, 8, 128, 128, 128, 130, 10.0, 16),
    (5, 5, 24, 21, 64, 64, 3.0, 32), (12, 4, 96, 128, 128, 1, 5.0, 16), (40, 8, 64, 56, 64, 300, 0.0, 16),
    (18, 6, 128, 72, 128, 2**31 - 1, 2.0, 64), (16, 1, 64, 64, 64, 257, 8.0, 16), (3, 1, 21, 35, 64, 47, 2.5, 16),
    (22, 2, 120, 128, 128, 200, 15.0, 16), (64, 4, 64, 64, 64, 96, 30.0, 16), (2, 2, 128, 8, 128, 65, 1.5, 16)]


def expected_rows(req, th, rows):
    q, k, v = (x.double() for x in req)
    talk, r1, r2, scale, cap, window = th
    o = ref.talking_attention(q, k, v, scale, cap or None, r1.double(), r2.double(), None if window > 10**6 else window, talk.double())
    return o[rows].flatten(1)


def check_rows(got, want, dtype):
    """element by element against the row's own spread: values are sums of many terms of both signs"""
    err = (got.double().cpu() - want).abs()
    lim = (0.012 if dtype == torch.bfloat16 else 2e-5) * want.abs().amax(-1, keepdim=True) + \
          (2 ** -8 if dtype == torch.bfloat16 else 1e-6) * want.abs() + 1e-6
    assert (err <= lim).all(), float((err / lim).max())


@pytest.mark.parametrize("form", ["rows32", "rows16", "matrix"])
@pytest.mark.parametrize("case", CASES, ids=lambda c: "-".join(map(str, c)))
def test_talking_attention(dev, case, form):
    """decode rows of unequal requests, prompt portions of 2 to 80 rows (their keys at page and window edges and far away made
    to stand out), gate and all, by the any-size kernel in both types and by the matrix-core kernels"""
    from vllm_omni_amd import ops

    h, g, dim, vdim, hd, window, cap, bs = case
    dtype = torch.float32 if form == "rows32" else torch.bfloat16
    if form == "matrix":
        assert ops.talking_attn_supported(dtype, h, g, hd, vdim, bs, cap)
    lens = [1, 2, 17, 90, 333, 420]
    w = min(window, 333)
    loud = [(4, 332, 332 - w + 1), (4, 331, max(331 - w, 0)), (4, 320, max(320 - w + 1, 0)), (4, 330, max(330 - w, 0)), (5, 419, 400),
            (5, 419, 384), (5, 416, 415), (5, 405, max(405 - w + 1, 0)), (5, 406, max(406 - w, 0)), (5, 390, 3), (3, 89, 15), (3, 80, 16)]
    reqs = attention_case(lens, h, g, dim, vdim, hd, window, torch.bfloat16, loud=loud)
    talk = bf(torch.eye(h) + rnd(h, h, std=0.6 * h ** -0.5, seed=91))
    r1, r2 = bf(0.1 + rnd(h, seed=92).abs()), bf(0.02 + rnd(h, seed=93).abs())
    scale = 1.3 * dim ** -0.5
    th = ops.TalkingHeads(talk.to(dev), r1.to(dev), r2.to(dev), scale, cap, window, vdim)
    kc, vc, table = paged(reqs, lens, bs, g, hd, dtype, dev)
    pars = (talk, r1, r2, scale, cap, window)
    full = [expected_rows(r, pars, slice(None)) for r in reqs]
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=dev)   # noqa: E731
    sig = lambda x: 1 / (1 + torch.exp(-x.double()))   # noqa: E731

    def gate_for(n, seed):
        return rnd(n, h * vdim + 8, dtype=dtype, seed=seed)[:, :h * vdim]

    # one row per request, the last one; longest context bound exact, larger, and one padded row (no request)
    q = torch.stack([r[0][-1] for r in reqs])
    want = torch.stack([f[-1] for f in full])
    gate = gate_for(len(lens) + 1, 70)
    qg = laid_out(torch.cat([q, q[:1]]), hd, dtype, dev)
    n1 = len(lens) + 1
    tb = torch.cat([table, torch.zeros_like(table[:1])])
    sl, qsl = i32(lens + [0]), i32(list(range(n1 + 1)))
    for bound in (max(lens), 2000):
        for gg in (gate, None):
            out = torch.full((n1, h * vdim), 7.0, dtype=dtype, device=dev)
            if form == "matrix":
                ops.talking_decode(out, qg, kc, vc, tb, sl, qsl, th, bound, n1, None if gg is None else gg.to(dev))
            else:
                ops.talking_attn_rows(out, qg, kc, vc, tb, sl, qsl, th, None if gg is None else gg.to(dev))
            check_rows(out[:-1], want * (1 if gg is None else sig(gg[:-1])), dtype)
            assert not out[-1].any()
    # portions: the last n rows of each request, behind three rows that belong to somebody else
    for sizes in ([1, 2, 2, 3, 33, 80], [1, 2, 17, 90, 16, 5]):
        rows = sum(sizes) + 3
        q = torch.cat([torch.zeros(3, h, dim)] + [r[0][-n:] for r, n in zip(reqs, sizes)])
        want = torch.cat([f[-n:] for f, n in zip(full, sizes)])
        gate = gate_for(rows, 71)
        starts = [3]
        for n in sizes:
            starts.append(starts[-1] + n)
        out = torch.full((rows, h * vdim), 7.0, dtype=dtype, device=dev)
        args = (out, laid_out(q, hd, dtype, dev), kc, vc, table, i32(lens), i32(starts), th)
        if form == "matrix":
            ctx = [0]
            for L, n in zip(lens, sizes):
                ctx.append(ctx[-1] + -(-(L - max(0, L - n - window + 1)) // 64) * 64)
            ops.talking_prefill(*args, i32(ctx), ctx[-1], max(sizes), gate.to(dev))
        else:
            ops.talking_attn_rows(*args, gate.to(dev), row0=3)
        check_rows(out[3:], want * sig(gate[3:]), dtype)
        assert (out[:3] == 7).all()


def test_long_decode_context_in_parts(dev):
    """few requests with long contexts and many with short ones: other part sizes, parts past a request's end"""
    from vllm_omni_amd import ops

    h, g, dim, window, bs = 8, 2, 64, 1500, 16
    talk, r1, r2 = bf(torch.eye(h) + rnd(h, h, std=0.2, seed=1)), bf(0.1 + rnd(h, seed=2).abs()), bf(rnd(h, seed=3).abs())
    th = ops.TalkingHeads(talk.to(dev), r1.to(dev), r2.to(dev), 0.2, 12.0, window, dim)
    for lens in ([1900], [1, 1700, 64, 65], list(range(1, 260, 3)) + [1501]):
        reqs = attention_case(lens, h, g, dim, dim, dim, window, torch.bfloat16)
        kc, vc, table = paged(reqs, lens, bs, g, dim, torch.bfloat16, dev)
        q = torch.stack([r[0][-1] for r in reqs])
        want = []
        for r, n in zip(reqs, lens):
            lo = max(0, n - window)
            one = (r[0][-1:].double(), r[1][lo:].double(), r[2][lo:].double())
            d = torch.arange(n - 1 - lo, -1, -1, dtype=torch.float64)
            p = torch.stack([torch.softmax(ref.soft_cap(one[1][:, i // (h // g)] @ one[0][0, i] * 0.2, 12.0)
                                           - ref.log_distance(r1[i].double(), r2[i].double(), d), 0) for i in range(h)])
            want.append(ref.apply_weights(ref.mix_heads(p[:, None], talk.double()), one[2]).flatten())
        out = torch.empty(len(lens), h * dim, dtype=torch.bfloat16, device=dev)
        ops.talking_decode(out, laid_out(q, dim, torch.bfloat16, dev), kc, vc, table, torch.tensor(lens, dtype=torch.int32, device=dev),
                           torch.arange(len(lens) + 1, dtype=torch.int32, device=dev), th, 2048, len(lens))
        check_rows(out, torch.stack(want), torch.bfloat16)


def test_no_bias_at_all(dev):
    from vllm_omni_amd import ops

    lens, h, g, dim, bs = [70, 33], 4, 2, 64, 16
    reqs = attention_case(lens, h, g, dim, dim, dim, 50, torch.bfloat16)
    talk = bf(rnd(h, h, seed=1))
    zero = torch.zeros(h)
    th = ops.TalkingHeads(talk.to(dev), None, None, 0.125, 4.0, 50, dim)
    kc, vc, table = paged(reqs, lens, bs, g, dim, torch.bfloat16, dev)
    q = torch.cat([r[0] for r in reqs])
    want = torch.cat([expected_rows(r, (talk, zero, zero, 0.125, 4.0, 50), slice(None)) for r in reqs])
    out = torch.empty(103, h * dim, dtype=torch.bfloat16, device=dev)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=dev)   # noqa: E731
    args = (out, laid_out(q, dim, torch.bfloat16, dev), kc, vc, table, i32(lens), i32([0, 70, 103]), th)
    ops.talking_prefill(*args, i32([0, 128, 192]), 192, 70)
    check_rows(out, want, torch.bfloat16)
    ops.talking_attn_rows(*args)
    check_rows(out, want, torch.bfloat16)
