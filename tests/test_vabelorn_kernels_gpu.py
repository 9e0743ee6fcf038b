"""Each mechanism of the Vabelorn design alone, against the plain functions of ``plain_vabelorn.py`` in 64-bit, at sizes that are no multiples
of the kernels' tiles: the sum of a normed branch output with mixes of neighbouring tokens (portions, several requests, rows of a slot), the
sum handed on without a norm, the products of several mixes in one launch, decays per key channel, the recurrence with a bonus (portions
against single steps to the bit, slots used again, one key made to stand out hundreds of tokens back), the norm and rotation of queries,
keys and values with a magnitude straight into the pages, the attention that adds one and turns its output back (every position a query,
portions down to two tokens, scrambled pages with NaN wherever nothing was written, a far key that carries the weight), and the gate
against a token's own row."""
import pytest
import torch

import plain_vabelorn as plain

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]


def _tol(dtype, loose=1.0):
    return dict(atol=2e-5 * loose, rtol=2e-5 * loose) if dtype == torch.float32 else dict(atol=2e-2 * loose, rtol=2e-2 * loose)


def _i32(x):
    return torch.tensor(x, dtype=torch.int32, device="cuda")


def _batch(spans):
    """``spans``: per request its ``(first, last + 1)`` positions in the step -> (indptr, token_req, positions, ctx_lens) on the GPU."""
    lens = [b - a for a, b in spans]
    indptr = [0] + torch.tensor(lens).cumsum(0).tolist()
    return (_i32(indptr), _i32([i for i, n in enumerate(lens) for _ in range(n)]), _i32([p for a, b in spans for p in range(a, b)]), _i32([a for a, _ in spans]))


def _steps(lengths, cuts):
    """The steps of requests cut at ``cuts[r]``: per step the live requests with their spans of positions."""
    edges = [[0] + c + [n] for c, n in zip(cuts, lengths)]
    for s in range(max(len(e) for e in edges) - 1):
        spans = {r: (e[s], e[s + 1]) for r, e in enumerate(edges) if s + 1 < len(e) and e[s + 1] > e[s]}
        if spans:
            yield spans


# ------------------------------------------------------------------ sums and mixes

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden, kind", [(42, "whole"), (64, "slabs"), (37, "slabs"), (1028, "whole"), (96, "plain"), (50, "nothing"), (5000, "whole"), (9004, "slabs"), (4102, "slabs")])
def test_sum_and_mixes_of_neighbouring_tokens(dtype, hidden, kind):
    """Two requests in portions, the rows of the tokens before in scrambled slots at an odd offset; the pending output normed, added as it is,
    in slabs, or absent."""
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(hidden)
    lengths, cuts, slots = [29, 11], [[7, 8, 20], [1, 3]], [4, 1]
    eps, off = 1e-5, 5
    w = 1.0 + torch.randn(hidden, generator=g) * 0.3
    mu = torch.rand(5, hidden, generator=g)
    x0 = [torch.randn(n, hidden, generator=g) * 3 for n in lengths]
    y = [torch.randn(n, hidden, generator=g) * 5 for n in lengths]
    slabs = [torch.randn(3, n, hidden, generator=g) for n in lengths]
    state = torch.full((6, off + hidden + 2), float("nan"), device="cuda")
    for s in slots:
        state[s, off: off + hidden] = 0.0
    want_x = []
    for r in range(2):
        if kind == "nothing":
            want_x.append(x0[r].double())
            continue
        b = slabs[r].double().sum(0) if kind == "slabs" else y[r].to(dtype).double()
        want_x.append(x0[r].double() + (b if kind == "plain" else plain.rms(b, eps) * w.double()))
    for spans in _steps(lengths, cuts):
        live = list(spans)
        indptr, token_req, _, _ = _batch(list(spans.values()))
        cat = lambda xs, dim=0: torch.cat([xs[r][spans[r][0]: spans[r][1]] if dim == 0 else xs[r][:, spans[r][0]: spans[r][1]] for r in live], dim)
        pending = None if kind == "nothing" else (cat(slabs, 1).contiguous().cuda() if kind == "slabs" else cat(y).to(dtype).cuda())
        res = cat(x0).cuda()
        T = res.shape[0]
        mixes = torch.full((5, T, hidden), float("nan"), dtype=dtype, device="cuda")
        sl = _i32([slots[r] for r in live])
        x = ops.settle_shift(res, pending, None if kind in ("plain", "nothing") else w.cuda(), eps, state, off, sl, indptr, token_req, mu.cuda(), mixes)
        assert (x is res) == (kind == "nothing")
        at = 0
        for r in live:
            a, b = spans[r]
            torch.testing.assert_close(x[at: at + b - a].cpu().double(), want_x[r][a:b], atol=3e-5, rtol=1e-5)
            want = torch.stack([plain.token_shift(want_x[r], m.double())[a:b] for m in mu])
            torch.testing.assert_close(mixes[:, at: at + b - a].cpu().double(), want, **_tol(dtype, 3))
            at += b - a
            state[slots[r], off: off + hidden] = x[at - 1]


@pytest.mark.parametrize("T", [2100, 800, 5])
def test_sum_and_mixes_of_long_prompts(T):
    """Work-groups that take several rows, with requests that begin inside one."""
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(T)
    hidden, first = 40, T // 2 + 1
    x0, y, mu = torch.randn(T, hidden, generator=g), torch.randn(T, hidden, generator=g), torch.rand(2, hidden, generator=g)
    w = 1.0 + torch.randn(hidden, generator=g) * 0.3
    state = torch.randn(2, hidden, generator=g)
    mixes = torch.empty(2, T, hidden, device="cuda")
    indptr, token_req, _, _ = _batch([(0, first), (0, T - first)])
    x = ops.settle_shift(x0.cuda(), y.cuda(), w.cuda(), 1e-6, state.cuda(), 0, _i32([1, 0]), indptr, token_req, mu.cuda(), mixes)
    want = x0.double() + plain.rms(y.double(), 1e-6) * w.double()
    before = torch.cat((state[1:2].double(), want[:-1]))
    before[first] = state[0].double()
    torch.testing.assert_close(x.cpu().double(), want, atol=2e-5, rtol=1e-5)
    torch.testing.assert_close(mixes.cpu().double(), want[None] + (before - want)[None] * mu.double()[:, None], atol=3e-5, rtol=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("parts, H", [(0, 150), (3, 150), (5, 152), (0, 4104), (2, 9000), (8, 2048)])
def test_sum_of_a_normed_branch_handed_on_without_a_norm(dtype, parts, H):
    from torchlet_amd.config.base import OffsetRMSNormSpec
    from torchlet_amd.parts import NORMS, Stream
    g = torch.Generator().manual_seed(3)
    T, eps = 6, 1e-5
    norm = NORMS.build(OffsetRMSNormSpec(dim=H, eps=eps, offset=0.0, weight_name=""), dtype, torch.device("cuda"))
    w = (1.0 + torch.randn(H, generator=g) * 0.3).to(torch.bfloat16)
    norm.load_weights({"": w})
    x = torch.randn(T, H, generator=g) * 3
    y = torch.randn(parts, T, H, generator=g) if parts else (torch.randn(T, H, generator=g) * 7).to(dtype)
    stream = Stream(x.cuda(), y.cuda())
    stream.post = (norm.weight, norm.eps)
    h = norm.settle(stream)
    new = x.double() + plain.rms(y.double().sum(0) if parts else y.double(), eps) * w.double()
    torch.testing.assert_close(stream.residual.cpu().double(), new, atol=2e-5, rtol=1e-5)
    torch.testing.assert_close(h.cpu().double(), new, **_tol(dtype, 1 if dtype == torch.float32 else 0.5))
    assert stream.pending is None and stream.post is None
    rows = torch.tensor([4, 0, 4], dtype=torch.int32, device="cuda")         # and the norm of some rows of a sum still pending, the stream left as it is
    stream.pending, stream.post = y.cuda(), (norm.weight, norm.eps)
    few = norm.forward(stream, rows=rows, gain=0.7)
    b = y.double().sum(0) if parts else y.double()
    want = plain.rms((stream.residual.cpu().double() + plain.rms(b, eps) * w.double())[[4, 0, 4]], eps) * w.double() * 0.7
    torch.testing.assert_close(few.cpu().double(), want, **_tol(dtype, 3))
    torch.testing.assert_close(stream.residual.cpu().double(), new, atol=2e-5, rtol=1e-5)
    stream.pending = stream.post = None
    again = norm.settle(stream)                                  # nothing pending: the residual as it is
    torch.testing.assert_close(again.cpu(), stream.residual.to(dtype).cpu(), atol=0.0, rtol=0.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M", [1, 3, 16, 17, 40, 64, 130, 600])
@pytest.mark.parametrize("G, N, K", [(4, 21, 42), (4, 96, 64), (2, 200, 136), (4, 256, 512)])
def test_products_of_several_mixes_in_one_launch(dtype, M, G, N, K):
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(M * K)
    x, w = torch.randn(G, M, K, generator=g).to(dtype), (torch.randn(G, N, K, generator=g) * K ** -0.5).to(dtype)
    wide = torch.full((M, G * N + 8), float("nan"), dtype=dtype, device="cuda")
    ops.linear_groups(x.cuda(), w.cuda(), wide[:, : G * N])
    want = torch.cat([x[i].double() @ w[i].double().T for i in range(G)], 1)
    torch.testing.assert_close(wide[:, : G * N].cpu().double(), want, **_tol(dtype))
    assert bool(torch.isnan(wide[:, G * N:]).all())


# ------------------------------------------------------------------ decays and the recurrence

@pytest.mark.parametrize("T, rank, channels", [(1, 1, 1), (3, 5, 21), (9, 16, 300), (700, 7, 513), (1030, 64, 256), (2, 1024, 40)])
def test_decays_per_key_channel(T, rank, channels):
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(T)
    z, w2, w0 = torch.randn(T, rank, generator=g) * 2, torch.randn(channels, rank, generator=g) * rank ** -0.5, torch.rand(channels, generator=g) * 8 - 6
    out = torch.full((T, channels), float("nan"), device="cuda")
    ops.channel_decay(z.cuda(), w2.T.contiguous().cuda(), w0.cuda(), out)
    want = torch.exp(-torch.exp(torch.tanh(z.double()) @ w2.double().T + w0.double()))
    torch.testing.assert_close(out.cpu().double(), want, atol=2e-6, rtol=1e-5)


def _recur(dtype, data, lengths, cuts, slots, heads, dim, vdim, state, off, rows, max_new=None):
    """The recurrence over the steps of ``cuts``; returns the outputs per request."""
    from torchlet_amd.kernels import ops
    r, k, v, w, u = data
    outs = [torch.zeros(n, heads * vdim) for n in lengths]
    pad = 3 if dim % 4 else 4
    for spans in _steps(lengths, cuts):
        live = list(spans)
        indptr, _, _, _ = _batch(list(spans.values()))
        cat = lambda xs: torch.cat([xs[q][spans[q][0]: spans[q][1]] for q in live])
        T = int(indptr[-1])
        rkv = torch.cat((cat(r), cat(k), torch.zeros(T, pad), cat(v), torch.zeros(T, pad)), 1).to(dtype).cuda()
        out = torch.full((T, heads * vdim), float("nan"), device="cuda")
        K = heads * dim
        ops.wkv_scan(rkv, K, 2 * K + pad, cat(w).cuda(), u.reshape(-1).cuda(), state, _i32([slots[q] for q in live]), indptr, out, heads, dim, vdim,
                     max_new_tokens=max(b - a for a, b in spans.values()), last_rows=cat(rows).cuda(), tail_off=off)
        at = 0
        for q in live:
            n = spans[q][1] - spans[q][0]
            outs[q][spans[q][0]: spans[q][1]] = out[at: at + n].cpu()
            at += n
            assert torch.equal(state[slots[q], off: off + rows[q].shape[1]].cpu(), rows[q][spans[q][1] - 1])
    return outs


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, dim, vdim", [(3, 7, 7), (2, 64, 64), (1, 1, 1), (2, 36, 50), (1, 100, 20), (2, 192, 17), (1, 256, 33), (3, 130, 16)])
def test_recurrence_with_a_bonus_against_plain_and_portions_to_the_bit(dtype, heads, dim, vdim):
    """Whole requests, portions of every batch size of the kernel (down to two tokens and single ones), requests side by side in scrambled
    slots of a wider state: the same bits; against the plain recurrence within rounding."""
    g = torch.Generator().manual_seed(dim)
    lengths, slots, width = [45, 19], [2, 0], 11
    K, off = heads * dim, heads * dim * vdim + 3
    r, k = ([torch.randn(n, K, generator=g).to(dtype).float() for n in lengths] for _ in range(2))
    v = [torch.randn(n, heads * vdim, generator=g).to(dtype).float() for n in lengths]
    w = [torch.exp(-torch.exp(torch.rand(n, K, generator=g) * 8 - 6)) for n in lengths]
    u = torch.randn(heads, dim, generator=g)
    rows = [torch.randn(n, width, generator=g) for n in lengths]
    results = []
    for cuts in ([[], []], [[16, 32, 33, 34, 36, 40], [2, 4, 7, 9, 10, 11]], [list(range(1, 45)), list(range(1, 19))], [[3, 30], [17]]):
        state = torch.full((4, off + width + 1), float("nan"), device="cuda")
        for s in slots:
            state[s, : heads * dim * vdim] = 0.0
        outs = _recur(dtype, (r, k, v, w, u), lengths, cuts, slots, heads, dim, vdim, state, off, rows)
        results.append((outs, [state[s, : heads * dim * vdim].cpu() for s in slots]))
    for outs, states in results[1:]:
        for a, b in zip(outs + states, results[0][0] + results[0][1]):
            assert torch.equal(a, b)
    for q, n in enumerate(lengths):
        f = lambda x, m: x.double().view(n, heads, m)
        want, S = plain.wkv_recurrence(f(r[q], dim), f(k[q], dim), f(v[q], vdim), f(w[q], dim), u.double())
        scale = float(want.abs().max())
        torch.testing.assert_close(results[0][0][q].double(), want.reshape(n, -1), atol=2e-6 * scale, rtol=1e-5)
        torch.testing.assert_close(results[0][1][q].double().view(heads, vdim, dim).transpose(1, 2), S, atol=1e-6 * float(S.abs().max()), rtol=1e-5)


def test_recurrence_remembers_one_token_far_back():
    """One key that stands out and decays close to one: its value is read 400 tokens later through the state, with the decay it has gone
    through; and the bonus holds for the current token only."""
    g = torch.Generator().manual_seed(9)
    heads, dim, vdim, n, at = 1, 32, 20, 420, 13
    r, k, v = (torch.randn(n, m, generator=g) * 0.01 for m in (dim, dim, vdim))
    w = torch.full((n, dim), 0.999)
    k[at], r[n - 1], v[at] = 5.0, 1.0, torch.arange(vdim).float()
    u = torch.full((1, dim), -3.0)
    state = torch.zeros(1, dim * vdim + 1, device="cuda")
    out = _recur(torch.float32, ([r], [k], [v], [w], u), [n], [[200, 202]], [0], heads, dim, vdim, state, dim * vdim, [torch.zeros(n, 1)])[0]
    torch.testing.assert_close(out[n - 1], 5.0 * dim * 0.999 ** (n - 2 - at) * v[at], atol=0.1, rtol=1e-2)
    now = -3.0 * float((r[at] * k[at]).sum())                   # at the token itself: the state before it, and the bonus times its value
    torch.testing.assert_close(out[at], now * v[at], atol=0.05, rtol=0.02)


# ------------------------------------------------------------------ attention

def _tables(lengths, page, g):
    blocks = [-(-n // page) for n in lengths]
    pages = sum(blocks) + 1
    order = (torch.randperm(pages - 1, generator=g) + 1).tolist()
    table = torch.zeros(len(lengths), max(blocks + [1]) + 1, dtype=torch.int32)
    for r, b in enumerate(blocks):
        for i in range(b):
            table[r, i] = order.pop()
    return table, pages


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("halves", [False, True])
@pytest.mark.parametrize("H, G, dim, vdim, dims, vdims", [(6, 2, 10, 14, 6, 14), (4, 4, 96, 32, 96, 32), (1, 1, 8, 6, 2, 4), (3, 1, 128, 256, 64, 0)])
def test_norm_and_rotation_straight_into_the_pages(dtype, halves, H, G, dim, vdim, dims, vdims):
    """Queries stay in place; keys (with a magnitude on cosine and sine) and values (no weight, a rotation of their own) go to their pages, and
    nothing else of a page is touched; a token whose block is the sentinel writes nothing."""
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(dim)
    page, eps, mag, base = 4, 1e-4, 1.2, 500.0
    spans = [(3, 9), (0, 2), (30, 31)]
    indptr, token_req, positions, _ = _batch(spans)
    T = int(indptr[-1])
    x = (torch.randn(T, (H + G) * dim + G * vdim + 5, generator=g) * 3).to(dtype)
    wq, wk = (1.0 + torch.randn(dim, generator=g) * 0.3 for _ in range(2))
    fq = torch.tensor(plain.plain_frequencies(dims, base), dtype=torch.float32)
    fv = torch.tensor(plain.plain_frequencies(vdims, base), dtype=torch.float32)
    table, pages = _tables([9, 2, 31], page, g)
    table[2, 30 // page] = 0                                     # the third request's block is the sentinel
    nan = float("nan")
    kp = torch.full((pages, G, page, dim), nan, dtype=dtype, device="cuda")
    vp = torch.full((pages, G, vdim, page), nan, dtype=dtype, device="cuda")
    xs = x.cuda()
    width = (H + G) * dim + G * vdim
    ops.head_norm_rotate(xs[:, :width], H, G, dim, wq.cuda(), wk.cuda(), eps, positions, fq.cuda(), dims, halves, magnitude=mag,
                         values=(G, vdim, True, fv.cuda() if vdims else None, vdims, halves), pages=(token_req, table.cuda(), kp, vp, page))
    assert torch.equal(xs[:, H * dim:].cpu(), x[:, H * dim:])
    pos = positions.cpu().long()

    def turn(t, freqs, magnitude):
        if not len(freqs):
            return t
        freqs = [float(f) for f in freqs]
        if not halves:
            return plain.rotate_pairs(t, pos, freqs, magnitude)
        n = len(freqs)
        order = [i for m in range(n) for i in (m, m + n)]        # halves are pairs of another order
        back = [order.index(i) for i in range(2 * n)]
        y = plain.rotate_pairs(torch.cat((t[..., order], t[..., 2 * n:]), -1), pos, freqs, magnitude)
        return torch.cat((y[..., back], y[..., 2 * n:]), -1)
    q = turn(plain.rms(x[:, : H * dim].double().view(T, H, dim), eps) * wq.double(), fq, mag)
    k = turn(plain.rms(x[:, H * dim: (H + G) * dim].double().view(T, G, dim), eps) * wk.double(), fq, mag)
    v = turn(plain.rms(x[:, (H + G) * dim: width].double().view(T, G, vdim), eps), fv, 1.0)
    loose = 3 if dtype == torch.float32 else 1.5
    torch.testing.assert_close(xs[:, : H * dim].cpu().double().view(T, H, dim), q, **_tol(dtype, loose))
    seen_k, seen_v = torch.zeros_like(kp, dtype=torch.bool).cpu(), torch.zeros_like(vp, dtype=torch.bool).cpu()
    for t in range(T):
        p, pg = int(pos[t]), int(table[int(token_req[t]), int(pos[t]) // page])
        if pg == 0:
            continue
        torch.testing.assert_close(kp[pg, :, p % page].cpu().double(), k[t], **_tol(dtype, loose))
        torch.testing.assert_close(vp[pg, :, :, p % page].cpu().double(), v[t], **_tol(dtype, loose))
        seen_k[pg, :, p % page] = True
        seen_v[pg, :, :, p % page] = True
    assert torch.equal(~torch.isnan(kp.cpu()), seen_k) and torch.equal(~torch.isnan(vp.cpu()), seen_v)


def _attend(dtype, H, G, dim, vdim, page, lengths, cuts, g, q, k, v, scale, freqs, halves, gain=1.0):
    """Keys and values (turned already) go to scrambled pages in steps, every token of every step is a query; the outputs per request by the
    general kernel and, where built, by the matrix-core kernel."""
    from torchlet_amd.kernels import ops
    table, pages = _tables(lengths, page, g)
    table = table.cuda()
    nan = float("nan")
    kp = torch.full((pages, G, page, dim), nan, dtype=dtype, device="cuda")
    vp = torch.full((pages, G, vdim, page), nan, dtype=dtype, device="cuda")
    fits = ops.local_attention_mfma_fits(dtype, dim, vdim, page)
    outs = {m: [torch.zeros(n, H * vdim) for n in lengths] for m in (False, True)}
    f = torch.tensor(freqs, dtype=torch.float32).cuda()
    for spans in _steps(lengths, cuts):
        live = list(spans)
        indptr, token_req, positions, ctx = _batch(list(spans.values()))
        cat = lambda xs: torch.cat([xs[r][spans[r][0]: spans[r][1]] for r in live]).to(dtype).cuda()
        tab = table[live].contiguous()
        ops.kv_cache_write(cat(k), cat(v), token_req, positions, tab, kp, vp, page)
        lens = [b - a for a, b in spans.values()]
        for use_mfma in ((False, True) if fits else (False,)):
            out = torch.full((int(indptr[-1]), H * vdim + 3), nan, dtype=dtype, device="cuda")
            tiles = None
            if use_mfma:
                tile_req = [i for i, n in enumerate(lens) for _ in range(-(-n // 16))]
                tiles = (indptr, ctx, _i32(tile_req), _i32([16 * j for n in lens for j in range(-(-n // 16))]), len(tile_req))
            ops.local_attention(cat(q), out[:, : H * vdim], kp, vp, tab, token_req, positions, H, G, dim, vdim, page, scale, 0.0, 0, 0, gain, tiles=tiles,
                                sink=torch.zeros(H, device="cuda"), turn_back=(f, 2 * len(freqs), halves))
            at = 0
            for r, n in zip(live, lens):
                outs[use_mfma][r][spans[r][0]: spans[r][1]] = out[at: at + n, : H * vdim].float().cpu()
                at += n
            assert bool(torch.isnan(out[:, H * vdim:]).all())
    return outs, fits


def _plain_attention(q, k, v, H, G, dim, vdim, scale, freqs, dtype):
    n = q.shape[0]
    f = lambda t, h, m: t.to(dtype).double().view(n, h, m)
    qq, kk, vv = f(q, H, dim), f(k, G, dim), f(v, G, vdim)
    o = torch.stack([plain.off_by_one_attention(qq[:, h], kk[:, h // (H // G)], vv[:, h // (H // G)], scale) for h in range(H)], 1)
    return plain.rotate_pairs(o, torch.arange(n), [float(x) for x in torch.tensor(freqs, dtype=torch.float32)], sign=-1.0).reshape(n, -1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, G, dim, vdim, page, vdims", [(6, 2, 10, 14, 4, 14), (4, 2, 64, 32, 16, 32), (2, 1, 32, 96, 8, 96), (3, 3, 128, 16, 16, 8), (1, 1, 4, 2, 8, 2)])
def test_attention_that_adds_one_and_turns_its_output_back(dtype, H, G, dim, vdim, page, vdims):
    g = torch.Generator().manual_seed(5)
    lengths, cuts = [83, 41], [[30, 32, 47, 48, 49, 50, 70], [2, 25, 26, 27]]
    q, k, v = ([torch.randn(n, h * m, generator=g) for n in lengths] for h, m in ((H, dim), (G, dim), (G, vdim)))
    freqs = plain.plain_frequencies(vdims, 40.0)
    outs, fits = _attend(dtype, H, G, dim, vdim, page, lengths, cuts, g, q, k, v, 0.3, freqs, False)
    assert fits == (dtype == torch.bfloat16 and dim % 32 == 0)
    for r in range(2):
        want = _plain_attention(q[r], k[r], v[r], H, G, dim, vdim, 0.3, freqs, dtype)
        for use_mfma in ((False, True) if fits else (False,)):
            torch.testing.assert_close(outs[use_mfma][r].double(), want, **_tol(dtype, 2 if dtype == torch.float32 else 1.5))


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_key_carries_the_weight_and_its_value_arrives_turned_by_the_distance(dtype):
    """One key of 900 stands out for the last query: the output is that key's value turned by minus the distance, in a prompt's portion and
    decoded alone; scores far below zero leave next to nothing, since one is added to the denominator; the halves layout likewise."""
    g = torch.Generator().manual_seed(6)
    H = G = 1
    dim, vdim, n, at, page = 32, 32, 900, 37, 16
    q, k, v = torch.zeros(n, dim), torch.zeros(n, dim), torch.randn(n, vdim, generator=g).to(dtype).float()
    k[:, 0] = -1.0
    k[at, 0] = 1.0
    q[:, 0] = 12.0
    freqs = plain.plain_frequencies(vdim, 30.0)
    for halves in (False, True):
        order = [i for m in range(vdim // 2) for i in (m, m + vdim // 2)] if halves else list(range(vdim))
        for cuts in ([[]], [[n - 1]], [[500, n - 2]]):
            outs, fits = _attend(dtype, H, G, dim, vdim, page, [n], cuts, g, [q], [k], [v], 1.0, freqs, halves, gain=0.5)
            for use_mfma in ((False, True) if fits else (False,)):
                got = outs[use_mfma][0].double()
                want = plain.rotate_pairs(v[at].double()[order].view(1, 1, -1), torch.tensor([n - 1]), [float(f) for f in torch.tensor(freqs, dtype=torch.float32)], sign=-1.0).view(-1) * 0.5
                torch.testing.assert_close(got[n - 1][order], want, **_tol(dtype, 5 if dtype == torch.float32 else 1))
                assert float(got[at - 1].abs().max()) < 1e-3      # every score -12 there: nearly all weight lies on the one that was added


@pytest.mark.parametrize("dtype", DTYPES)
def test_gate_against_a_tokens_own_row(dtype):
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(8)
    V, n, layers = 40, 13, 3
    table = torch.randn(V, layers * n, generator=g).to(dtype)
    z, ids = torch.randn(9, n, generator=g) * 2, torch.randint(0, V, (9,), generator=g)
    for i in range(layers):
        out = torch.full((9, n), float("nan"), dtype=dtype, device="cuda")
        ops.token_gate(z.cuda(), _i32(ids.tolist()), table.cuda()[:, i * n: (i + 1) * n], out)
        torch.testing.assert_close(out.cpu().double(), plain.gelu_tanh(z.double()) * table.double()[ids, i * n: (i + 1) * n], **_tol(dtype))


def test_operands_that_do_not_fit_are_refused():
    from torchlet_amd.kernels import ops
    z = lambda *s, dt=torch.float32: torch.zeros(*s, dtype=dt, device="cuda")
    i = lambda *v: _i32(list(v))
    with pytest.raises(ops.KernelError):         # the slots hold no row behind the states
        ops.wkv_scan(z(2, 12), 4, 8, z(2, 4), z(4), z(2, 16), i(0), i(0, 2), z(2, 4), 1, 4, 4, last_rows=z(2, 6), tail_off=16)
    with pytest.raises(ops.KernelError):         # decays of another size
        ops.wkv_scan(z(2, 12), 4, 8, z(2, 3), z(4), z(2, 16), i(0), i(0, 2), z(2, 4), 1, 4, 4)
    with pytest.raises(ops.KernelError):
        ops.settle_shift(z(2, 6), None, None, 0.0, z(2, 5), 0, i(0), i(0, 2), i(0, 0), z(5, 6), z(5, 2, 6))
    with pytest.raises(ops.KernelError):
        ops.channel_decay(z(2, 3), z(3, 5), z(4), z(2, 4))
    with pytest.raises(ops.KernelError):         # more value heads than key heads for the pages
        ops.head_norm_rotate(z(1, 16), 1, 1, 4, None, None, 1e-5, i(0), None, 0, False, values=(2, 4, True, None, 0, False), pages=(i(0), _i32([[1]]), z(2, 1, 4, 4), z(2, 1, 4, 4), 4))
    with pytest.raises(ops.KernelError):         # a turn over more columns than a value has
        ops.local_attention(z(1, 4), z(1, 4), z(2, 1, 4, 4), z(2, 1, 4, 4), _i32([[1]]), i(0), i(0), 1, 1, 4, 4, 4, 1.0, turn_back=(z(3), 6, False))
    with pytest.raises(ops.KernelError):
        ops.linear_groups(z(2, 3, 4), z(2, 5, 4), z(3, 11))
