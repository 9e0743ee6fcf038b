"""Each mechanism of the Tilalorn design alone, against the plain functions of ``plain_tilalorn.py`` in 64-bit, at sizes that are no multiples of
the kernels' tiles: the norm that adds a branch times a factor, the cache row with its rotated part and the queries' rotated parts turned by
the same kernel (halves and pairs, a rotation over a part of the numbers), attention over cached rows in a window (every position a query,
portions down to two tokens, pages in scrambled order with NaN wherever nothing was written, latents that do not split evenly over the
waves, rows at the window's edges made to carry the weight), products over heads with a gate per number, unit queries and keys with a
temperature in place and into the pages, causal attention with a cap and a gate per head (a key far back that carries the weight), the choice
among the experts of the best groups (ties, many groups, every kind of score), the feed-forward gated by gelu."""
import pytest
import torch

import plain_tilalorn as plain

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]


def _tol(dtype, loose=1.0):
    return dict(atol=2e-5 * loose, rtol=2e-5 * loose) if dtype == torch.float32 else dict(atol=2e-2 * loose, rtol=2e-2 * loose)


def _i32(x):
    return torch.tensor(x, dtype=torch.int32, device="cuda")


def _tables(lengths, page, g):
    """Block tables of requests of the given lengths over pages handed out in scrambled order."""
    blocks = [-(-n // page) for n in lengths]
    pages = sum(blocks) + 1
    order = (torch.randperm(pages - 1, generator=g) + 1).tolist()
    table = torch.zeros(len(lengths), max(blocks + [1]) + 1, dtype=torch.int32)
    for r, b in enumerate(blocks):
        for i in range(b):
            table[r, i] = order.pop()
    return table, pages


def _steps(lengths, cuts):
    """The steps of requests cut at ``cuts[r]``: per step the live requests with their spans of positions."""
    edges = [[0] + c + [n] for c, n in zip(cuts, lengths)]
    for s in range(max(len(e) for e in edges) - 1):
        spans = {r: (e[s], e[s + 1]) for r, e in enumerate(edges) if s + 1 < len(e) and e[s + 1] > e[s]}
        if spans:
            yield spans


# ------------------------------------------------------------------ a factor on the branch

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("parts, H", [(0, 150), (3, 150), (5, 152), (0, 4104), (2, 4102), (8, 2048)])
def test_branch_enters_the_stream_times_a_factor(dtype, parts, H):
    """The branch as one tensor or as slabs of partial sums, times the factor, added and normed; the row alone (a selection leaves the stream as it
    is); the sum without a norm; a branch that is normed first."""
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(3)
    T, eps, m = 7, 1e-5, 0.37
    x, w, post = torch.randn(T, H, generator=g), torch.randn(H, generator=g) * 0.3, torch.randn(H, generator=g)
    pending = torch.randn(parts, T, H, generator=g) if parts else torch.randn(T, H, generator=g).to(dtype)
    y = pending.double().sum(0) if parts else pending.double()
    rows = torch.tensor([5, 0, 6])
    for kind in ("plain", "rows", "no norm", "normed branch"):
        branch = plain.rms(y, 1e-4) * post.double() if kind == "normed branch" else y
        r = x.double() + m * branch
        want = r if kind == "no norm" else plain.offset_rms_norm(r, w.double(), eps)
        res = x.cuda()
        out = torch.full((3 if kind == "rows" else T, H), float("nan"), dtype=dtype, device="cuda")
        ops.sandwich_norm(res, pending.cuda(), post.cuda() if kind == "normed branch" else None, 1e-4, None, None if kind == "no norm" else (1.0 + w).cuda(), eps, out,
                          _i32(rows.tolist()) if kind == "rows" else None, branch_gain=m)
        torch.testing.assert_close(out.cpu().double(), want[rows] if kind == "rows" else want, **_tol(dtype))
        torch.testing.assert_close(res.cpu().double(), x.double() if kind == "rows" else r, atol=2e-6, rtol=2e-6)


# ------------------------------------------------------------------ the cache row and the queries' rotated parts

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("halves", [True, False])
@pytest.mark.parametrize("H, dim, rot, dims, rank", [(3, 6, 4, 4, 10), (5, 32, 16, 16, 80), (1, 7, 10, 6, 5), (20, 128, 64, 64, 512), (2, 8, 258, 130, 300)])
def test_cache_rows_and_queries_rotated_parts_in_one_kernel(dtype, halves, H, dim, rot, dims, rank):
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(4)
    lengths, page, eps, base = [23, 9], 4, 1e-5, 70.0
    table, pages = _tables([n + 3000 for n in lengths], page, g)
    positions = torch.cat([torch.arange(n) + c for n, c in zip(lengths, (0, 2991))])
    T, head, D, pad = sum(lengths), dim + rot, rank + rot, 5
    down = torch.randn(T, H * head + D + pad, generator=g).to(dtype)
    w = (torch.randn(rank, generator=g) * 0.3 + 1.0).to(dtype)
    inv = (torch.tensor(base, dtype=torch.float64) ** (-2.0 * torch.arange(dims // 2) / dims)).float()
    plane = torch.full((pages, 1, page, D), float("nan"), dtype=dtype, device="cuda")
    rows = torch.full((T, H * D), float("nan"), dtype=dtype, device="cuda")
    token_req = _i32([0] * lengths[0] + [1] * lengths[1])
    ops.latent_prepare(down.cuda(), 0, rank, rot, dims, None, w.cuda(), eps, _i32(positions.tolist()), inv.cuda(), None, token_req, table.cuda(), plane, page,
                       kv_off=H * head, halves=halves, queries=(rows, H, head, dim))

    def turned(x):          # [T, ..., rot]; the angles as the kernels take them, in 32-bit
        order = [i for m in range(dims // 2) for i in (m, m + dims // 2)] if not halves else None
        if order:           # neighbours to halves, turn, and back
            there = [2 * m for m in range(dims // 2)] + [2 * m + 1 for m in range(dims // 2)] + list(range(dims, rot))
            y = plain.rotate_halves(x[..., there], positions, dims, base)
            back = torch.empty_like(y)
            back[..., there] = y
            return back
        return plain.rotate_halves(x, positions, dims, base)

    d = down.double()
    tol = dict(atol=6e-4, rtol=1e-3) if dtype == torch.float32 else _tol(dtype)      # angles up to 3000 turns of 32-bit products
    want = turned(torch.stack([d[:, h * head + dim: (h + 1) * head] for h in range(H)], 1))
    got = rows.cpu().double().view(T, H, D)
    torch.testing.assert_close(got[:, :, rank:], want, **tol)
    assert bool(torch.isnan(got[:, :, :rank]).all())             # the unrotated parts are another kernel's
    c = plain.rms(d[:, H * head: H * head + rank], eps) * w.double()
    kr = turned(d[:, H * head + rank: H * head + D])
    for t in range(T):
        row = plane[int(table[int(token_req[t]), int(positions[t]) // page]), 0, int(positions[t]) % page].cpu().double()
        torch.testing.assert_close(row[:rank], c[t], **_tol(dtype))
        torch.testing.assert_close(row[rank:], kr[t], **tol)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rot, dims", [(10, 10), (12, 4), (64, 64)])
def test_rotation_in_halves_from_one_row_to_another(dtype, rot, dims):
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(5)
    T, H, src_head, src_off, dst_head, dst_off, base = 11, 3, rot + 7, 5, rot + 9, 2, 300.0
    src = torch.randn(T, H * src_head + 3, generator=g).to(dtype)
    dst = torch.zeros(T, H * dst_head, dtype=dtype, device="cuda")
    positions = torch.arange(T) * 17
    inv = (torch.tensor(base, dtype=torch.float64) ** (-2.0 * torch.arange(dims // 2) / dims)).float()
    ops.rotate_pairs(src.cuda(), src_head, src_off, dst, dst_head, dst_off, _i32(positions.tolist()), inv.cuda(), H, rot, halves=True)
    got = dst.cpu().double().view(T, H, dst_head)
    for h in range(H):
        want = plain.rotate_halves(src.double()[:, h * src_head + src_off: h * src_head + src_off + rot], positions, dims, base)
        torch.testing.assert_close(got[:, h, dst_off: dst_off + rot], want, **_tol(dtype, 3))
    assert float(got[:, :, :dst_off].abs().max()) == 0.0 and float(got[:, :, dst_off + rot:].abs().max()) == 0.0


# ------------------------------------------------------------------ attention over cached rows with a rotated part

def _latent_attend(dtype, H, rank, rot, page, window, lengths, cuts, g, scale, q, c):
    """``q[r] [n, H * D]`` queries against the cached rows ``c[r] [n, D]`` (D = rank + rot); outputs of the general kernel and, where it is built, of
    the matrix-core kernel, whole and with the keys dealt to three work-groups."""
    from torchlet_amd.kernels import ops
    D = rank + rot
    table, pages = _tables(lengths, page, g)
    table = table.cuda()
    plane = torch.full((pages, 1, page, D), float("nan"), dtype=dtype, device="cuda")
    fits = ops.latent_attention_mfma_fits(dtype, H, rank, rot)
    outs = {m: [torch.zeros(n, H * rank) for n in lengths] for m in (False, True)}
    for spans in _steps(lengths, cuts):
        live = list(spans)
        lens = [spans[r][1] - spans[r][0] for r in live]
        indptr = [0] + torch.tensor(lens).cumsum(0).tolist()
        ctx = _i32([spans[r][0] for r in live])
        queries = torch.cat([q[r][spans[r][0]: spans[r][1]] for r in live]).to(dtype).cuda()
        tab = table[live].contiguous()
        for i, r in enumerate(live):
            for p in range(*spans[r]):
                plane[int(tab[i, p // page]), 0, p % page] = c[r][p].to(dtype).cuda()
            if window:              # pages behind the window are gone
                tab[i, : max(0, spans[r][0] - window + 1) // page] = 0
        for use_mfma in ((False, True) if fits else (False,)):
            tq = ops.latent_tile_tokens(H, ops.LATENT_MFMA_ROWS if use_mfma else ops.LATENT_ATTENTION_ROWS)
            tile_req = [i for i, n in enumerate(lens) for _ in range(-(-n // tq))]
            tile_tok0 = [tq * j for n in lens for j in range(-(-n // tq))]
            for splits in (1, 3):
                out = torch.full((int(indptr[-1]), H * rank), float("nan"), dtype=dtype, device="cuda")
                ops.latent_attention(queries, out, plane, tab, _i32(indptr), ctx, _i32(tile_req), _i32(tile_tok0), len(tile_req), tq, H, rank, rot,
                                     page, scale, None, splits, general=not use_mfma, max_new_tokens=max(lens), window=window)
                for i, r in enumerate(live):
                    got = out[indptr[i]: indptr[i + 1]].float().cpu()
                    if splits == 1:
                        outs[use_mfma][r][spans[r][0]: spans[r][1]] = got
                    else:
                        torch.testing.assert_close(got, outs[use_mfma][r][spans[r][0]: spans[r][1]], **_tol(dtype, 2))
    return outs, fits


def _plain_latent(q, c, H, rank, rot, window, dtype, scale):
    n, D = q.shape[0], rank + rot
    rounded = lambda t: t.to(dtype).double()
    qq, cc = rounded(q).view(n, H, D), rounded(c)
    mask = plain.mask_matrix(n, window or None)
    return torch.cat([torch.softmax(qq[:, h] @ cc.T * scale + mask, -1) @ cc[:, :rank] for h in range(H)], -1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, rank, rot, page, window", [(3, 12, 4, 4, 9), (4, 80, 16, 16, 40), (2, 16, 16, 16, 33), (20, 112, 16, 8, 1), (2, 48, 16, 16, 0), (5, 208, 16, 8, 96),
                                                          (16, 512, 64, 16, 57), (6, 24, 40, 8, 30), (1, 336, 48, 16, 21)])
def test_latent_attention_in_a_window(dtype, H, rank, rot, page, window):
    """Every position a query, whole, in portions down to two tokens and in single tokens, two requests side by side over scrambled pages, the
    pages behind the window gone; latents of any multiple of 16 numbers on the matrix cores."""
    g = torch.Generator().manual_seed(7)
    lengths, cuts, D = [83, 41], [[30, 32, 47, 48, 49, 50, 70], [2, 25, 26, 27]], rank + rot
    q, c = [torch.randn(n, H * D, generator=g) for n in lengths], [torch.randn(n, D, generator=g) for n in lengths]
    scale = 1.2 * D ** -0.5
    outs, fits = _latent_attend(dtype, H, rank, rot, page, window, lengths, cuts, g, scale, q, c)
    assert fits == (dtype == torch.bfloat16 and D % 32 == 0 and rank % 16 == 0)
    for r in range(len(lengths)):
        want = _plain_latent(q[r], c[r], H, rank, rot, window, dtype, scale)
        for use_mfma in ((False, True) if fits else (False,)):
            torch.testing.assert_close(outs[use_mfma][r].double(), want, **_tol(dtype, 2 if dtype == torch.float32 else 1.5))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("rank, rot", [(48, 16), (64, 32)])
def test_rows_at_the_window_edge_carry_the_weight_or_none(dtype, decoded, rank, rot):
    """One query at the end of 300 tokens (in a portion, or decoded alone) whose first head matches the rotated part of one cached row: at the
    window's first position and at a page border inside it that row comes through whole; just outside the window, and far back, it does not
    show at all."""
    H, page, window, n, D = 2, 16, 40, 300, rank + rot
    last = n - 1
    g = torch.Generator().manual_seed(8)
    for what, at, shows in (("first of the window", last - window + 1, True), ("just outside the window", last - window, False),
                            ("page border inside", 288, True), ("far back", 0, False)):
        q, c = torch.randn(n, H * D, generator=g) * 0.2, torch.randn(n, D, generator=g) * 0.2
        c[at] = torch.randn(D, generator=g)
        q[last, rank: D] = c[at, rank:] * 5.0
        outs, fits = _latent_attend(dtype, H, rank, rot, page, window, [n], [[n - 1]] if decoded else [[150, 290]], g, 1.0, [q], [c])
        want = _plain_latent(q, c, H, rank, rot, window, dtype, 1.0)[last]
        for use_mfma in ((False, True) if fits else (False,)):
            got = outs[use_mfma][0][last].double()
            torch.testing.assert_close(got, want, **_tol(dtype, 3))
            near = float((got[:rank] - c[at, :rank].to(dtype).double()).abs().max())
            assert (near < 0.05) == shows, (what, use_mfma, near)


# ------------------------------------------------------------------ products over heads with a gate per number

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("G, N, K, T", [(3, 10, 12, 5), (4, 48, 96, 33), (5, 21, 64, 70), (2, 128, 512, 8), (16, 32, 32, 129)])
def test_products_over_heads_with_a_gate_per_number(dtype, G, N, K, T):
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(9)
    x, w = torch.randn(T, G * K, generator=g).to(dtype), (torch.randn(G, N, K, generator=g) * K ** -0.5).to(dtype)
    wide = torch.randn(T, G * N + 11, generator=g).to(dtype).cuda() * 2
    want = torch.cat([x.double()[:, h * K: (h + 1) * K] @ w[h].double().T for h in range(G)], -1) * torch.sigmoid(wide.cpu().double()[:, 3: 3 + G * N])
    for general in (False, True):
        out = torch.full((T, G * N), float("nan"), dtype=dtype, device="cuda")
        ops.heads_linear(x.cuda(), K, w.cuda(), out, N, general=general, gate=wide[:, 3: 3 + G * N])
        torch.testing.assert_close(out.cpu().double(), want, **_tol(dtype))


# ------------------------------------------------------------------ unit queries and keys, the temperature

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, G, dim, vdim", [(6, 2, 10, 14), (4, 4, 96, 72), (1, 1, 8, 6), (3, 1, 130, 256)])
@pytest.mark.parametrize("heat", [(0.6, 6), (0.3, 1), (0.5, 4096), None])
def test_unit_queries_and_keys_with_a_temperature(dtype, H, G, dim, vdim, heat):
    """Queries in place, keys and values into scrambled pages, nothing beyond them touched; the queries alone (a mixer that reads another's
    cache); queries and keys in place; positions on both sides of the temperature's steps."""
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(10)
    lengths, starts, page, eps = [14, 9], [0, 4088], 8, 1e-3
    table, pages = _tables([n + s for n, s in zip(lengths, starts)], page, g)
    positions = torch.cat([torch.arange(n) + s for n, s in zip(lengths, starts)])
    T, width, pad = sum(lengths), (H + G) * dim + G * vdim, 3
    x = (torch.randn(T, width + pad, generator=g) * 2).to(dtype)
    d = x.double()
    q, k, v = d[:, : H * dim].view(T, H, dim), d[:, H * dim: (H + G) * dim].view(T, G, dim), d[:, (H + G) * dim: width].view(T, G, vdim)
    grown = plain.query_temperature(positions, *heat)[:, None, None] if heat else 1.0
    want_q, want_k = (plain.rms(q, eps) * grown).reshape(T, -1), plain.rms(k, eps).reshape(T, -1)
    pos, token_req = _i32(positions.tolist()), _i32([0] * lengths[0] + [1] * lengths[1])
    k_plane = torch.full((pages, G, page, dim), float("nan"), dtype=dtype, device="cuda")
    v_plane = torch.full((pages, G, vdim, page), float("nan"), dtype=dtype, device="cuda")
    y = x.cuda()
    ops.head_norm_rotate(y[:, :width], H, G, dim, None, None, eps, pos, None, 0, False, values=(G, vdim, False, None, 0, False),
                         pages=(token_req, table.cuda(), k_plane, v_plane, page), unit=True, heat=heat)
    torch.testing.assert_close(y.cpu().double()[:, : H * dim], want_q, **_tol(dtype))
    assert torch.equal(y[:, H * dim:].cpu(), x[:, H * dim:])
    for t in range(T):
        p = int(positions[t])
        at = int(table[int(token_req[t]), p // page])
        torch.testing.assert_close(k_plane[at, :, p % page].cpu().double().reshape(-1), want_k[t], **_tol(dtype))
        assert torch.equal(v_plane[at, :, :, p % page].cpu(), x[t, (H + G) * dim: width].view(G, vdim))
    written = torch.isfinite(k_plane.float()).all(-1).sum()
    assert int(written) == T * G
    y = x.cuda()
    ops.head_norm_rotate(y[:, : H * dim], H, 0, dim, None, None, eps, pos, None, 0, False, unit=True, heat=heat)
    torch.testing.assert_close(y.cpu().double()[:, : H * dim], want_q, **_tol(dtype))
    assert torch.equal(y[:, H * dim:].cpu(), x[:, H * dim:])
    y = x.cuda()
    ops.head_norm_rotate(y[:, : (H + G) * dim], H, G, dim, None, None, eps, pos, None, 0, False, unit=True, heat=heat)
    torch.testing.assert_close(y.cpu().double()[:, : (H + G) * dim], torch.cat((want_q, want_k), -1), **_tol(dtype))


# ------------------------------------------------------------------ causal attention with a cap and a gate per head

def _attend(dtype, H, G, dim, vdim, page, lengths, cuts, g, q, k, v, gate, scale, cap):
    from torchlet_amd.kernels import ops
    table, pages = _tables(lengths, page, g)
    table = table.cuda()
    k_plane = torch.full((pages, G, page, dim), float("nan"), dtype=dtype, device="cuda")
    v_plane = torch.full((pages, G, vdim, page), float("nan"), dtype=dtype, device="cuda")
    fits = ops.local_attention_mfma_fits(dtype, dim, vdim, page)
    outs = {m: [torch.zeros(n, H * vdim) for n in lengths] for m in (False, True)}
    for spans in _steps(lengths, cuts):
        live = list(spans)
        lens = [spans[r][1] - spans[r][0] for r in live]
        indptr = [0] + torch.tensor(lens).cumsum(0).tolist()
        cat = lambda xs: torch.cat([xs[r][spans[r][0]: spans[r][1]] for r in live]).to(dtype).cuda()
        token_req = _i32([i for i, n in enumerate(lens) for _ in range(n)])
        positions = _i32([p for r in live for p in range(*spans[r])])
        tab = table[live].contiguous()
        ops.kv_cache_write(cat(k), cat(v), token_req, positions, tab, k_plane, v_plane, page)
        gates = torch.cat((cat(gate), torch.full((indptr[-1], 5), float("nan"), dtype=dtype, device="cuda")), -1)[:, :H]
        for use_mfma in ((False, True) if fits else (False,)):
            n = ops.LOCAL_ATTENTION_TILE_TOKENS
            tile_req = [i for i, m in enumerate(lens) for _ in range(-(-m // n))]
            tile_tok0 = [n * j for m in lens for j in range(-(-m // n))]
            tiles = (_i32(indptr), _i32([spans[r][0] for r in live]), _i32(tile_req), _i32(tile_tok0), len(tile_req)) if use_mfma else None
            out = torch.full((indptr[-1], H * vdim), float("nan"), dtype=dtype, device="cuda")
            ops.local_attention(cat(q), out, k_plane, v_plane, tab, token_req, positions, H, G, dim, vdim, page, scale, cap, tiles=tiles, gate=gates)
            for i, r in enumerate(live):
                outs[use_mfma][r][spans[r][0]: spans[r][1]] = out[indptr[i]: indptr[i + 1]].float().cpu()
    return outs, fits


def _plain_attention(q, k, v, gate, H, G, dim, vdim, scale, cap, dtype):
    n = q.shape[0]
    rounded = lambda t: t.to(dtype).double()
    qq, kk, vv, gg = rounded(q).view(n, H, dim), rounded(k).view(n, G, dim), rounded(v).view(n, G, vdim), torch.sigmoid(rounded(gate))
    mask = plain.mask_matrix(n, None)
    heads = []
    for h in range(H):
        s = plain.soft_cap(qq[:, h] @ kk[:, h // (H // G)].T * scale, cap or None)
        heads.append(torch.softmax(s + mask, -1) @ vv[:, h // (H // G)] * gg[:, h: h + 1])
    return torch.cat(heads, -1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, G, dim, vdim, page, cap", [(6, 2, 10, 14, 4, 2.0), (4, 2, 64, 80, 16, 3.0), (2, 1, 96, 48, 8, 0.0), (3, 3, 128, 112, 16, 20.0), (8, 2, 32, 160, 16, 1.5),
                                                          (1, 1, 4, 2, 8, 5.0)])
def test_causal_attention_with_a_cap_and_a_gate_per_head(dtype, H, G, dim, vdim, page, cap):
    g = torch.Generator().manual_seed(11)
    lengths, cuts = [83, 41], [[30, 32, 47, 48, 49, 50, 70], [2, 25, 26, 27]]
    q, k, v = ([torch.randn(n, h * m, generator=g) for n in lengths] for h, m in ((H, dim), (G, dim), (G, vdim)))
    gate = [torch.randn(n, H, generator=g) * 2 for n in lengths]
    scale = 3.0 * dim ** -0.5
    outs, fits = _attend(dtype, H, G, dim, vdim, page, lengths, cuts, g, q, k, v, gate, scale, cap)
    assert fits == (dtype == torch.bfloat16 and dim % 32 == 0)
    for r in range(2):
        want = _plain_attention(q[r], k[r], v[r], gate[r], H, G, dim, vdim, scale, cap, dtype)
        for use_mfma in ((False, True) if fits else (False,)):
            torch.testing.assert_close(outs[use_mfma][r].double(), want, **_tol(dtype, 2 if dtype == torch.float32 else 1.5))


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_key_carries_the_weight_up_to_the_cap(dtype):
    """One key of 900 stands out for the last query: with a high cap the output is its value times the gate; with a low cap the others, alike,
    keep the share the capped scores leave them.  In one prompt, in portions, and decoded alone; the key at a page's border."""
    g = torch.Generator().manual_seed(12)
    H = G = 1
    dim, vdim, n, at, page = 32, 48, 900, 48, 16
    q, k, v = torch.zeros(n, dim), torch.zeros(n, dim), torch.randn(n, vdim, generator=g).to(dtype).float()
    k[at, 0], q[:, 0] = 1.0, 30.0
    gate = torch.full((n, 1), 0.75)
    share = torch.sigmoid(torch.tensor(0.75, dtype=torch.float64))
    for cap, whole in ((100.0, True), (4.0, False)):
        top = float(plain.soft_cap(torch.tensor(30.0, dtype=torch.float64), cap))
        weight = torch.exp(torch.tensor(top, dtype=torch.float64))
        others = v.double().sum(0) - v[at].double()
        want = share * (weight * v[at].double() + others) / (weight + n - 1)
        for cuts in ([[]], [[n - 1]], [[500, n - 2]]):
            outs, fits = _attend(dtype, H, G, dim, vdim, page, [n], cuts, g, [q], [k], [v], [gate], 1.0, cap)
            for use_mfma in ((False, True) if fits else (False,)):
                got = outs[use_mfma][0][n - 1].double()
                torch.testing.assert_close(got, want, **_tol(dtype, 5 if dtype == torch.float32 else 1))
                assert (float((got - share * v[at].double()).abs().max()) < 0.03) == whole


# ------------------------------------------------------------------ the choice among the experts of the best groups

@pytest.mark.parametrize("E, count, keep, top", [(15, 5, 2, 4), (12, 2, 1, 5), (8, 8, 3, 2), (6, 1, 1, 2), (130, 13, 4, 8), (160, 5, 5, 6), (4096, 64, 3, 20), (512, 256, 5, 7)])
def test_choice_among_the_experts_of_the_best_groups(E, count, keep, top):
    from torchlet_amd.kernels import ops
    g = torch.Generator().manual_seed(13)
    T = 57
    logits = torch.randn(T, E, generator=g) * 2
    weights, offsets, slot_token, pair_slot = (t.cpu() for t in ops.route(logits.cuda(), top, "all", None, 1.7, groups=(count, keep)))
    s = torch.softmax(logits.double(), -1)
    owner = torch.repeat_interleave(torch.arange(E), (offsets[1:] - offsets[:-1]).long())
    chosen = owner[pair_slot.long()].view(T, top)
    want, want_w = plain.grouped_router(logits.double(), {"router": torch.eye(E, dtype=torch.float64)}, dict(experts=E, top=top, scale=1.7, groups=dict(count=count, keep=keep)))
    assert torch.equal(chosen, want)
    torch.testing.assert_close(weights.double(), want_w, atol=1e-6, rtol=2e-5)
    assert torch.equal(slot_token[pair_slot.long()].view(T, top), torch.arange(T, dtype=torch.int32)[:, None].expand(T, top))
    if keep < min(count, top):      # the groups change the choice for some tokens
        assert not torch.equal(chosen.sort(-1).values, torch.topk(s, top, -1).indices.sort(-1).values)


def test_choice_in_groups_ties_and_other_scores():
    """Equal logits: the lower group and the lower expert win.  The choice goes by what the scores and the correction say, in every kind of score; a
    group's best expert alone decides, not its sum."""
    from torchlet_amd.kernels import ops

    def chosen(logits, top, scores, groups, bias=None):
        weights, offsets, _, pair_slot = (t.cpu() for t in ops.route(logits.cuda(), top, scores, None if bias is None else bias.cuda(), groups=groups))
        owner = torch.repeat_interleave(torch.arange(logits.shape[1]), (offsets[1:] - offsets[:-1]).long())
        return owner[pair_slot.long()].view(logits.shape[0], top), weights

    for scores in ("all", "chosen", "sigmoid"):
        assert chosen(torch.zeros(2, 8), 3, scores, (4, 2))[0].tolist() == [[0, 1, 2]] * 2
    z = torch.tensor([[2.0, 2.0, 2.0, 5.0, -9.0, -9.0, 1.0, 0.5, 0.0]])          # the middle group has the best expert and the smallest sum
    for scores in ("all", "chosen", "sigmoid"):
        assert chosen(z, 2, scores, (3, 1))[0].tolist() == [[3, 4]]
    bias = torch.zeros(9)
    bias[6] = 4.0                                                                  # the correction lifts the last group above the others
    for scores in ("all", "sigmoid"):
        picks, weights = chosen(z, 2, scores, (3, 1), bias)
        assert picks.tolist() == [[6, 7]] and float(weights[0, 0]) < 1.0


# ------------------------------------------------------------------ the feed-forward gated by gelu

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T, hidden, inter", [(1, 72, 40), (7, 64, 96), (40, 128, 200), (300, 256, 320), (3, 50, 31), (70, 72, 40)])
def test_feed_forward_gated_by_gelu_fused_and_unfused(dtype, T, hidden, inter):
    from torchlet_amd.config import SwiGLUSpec
    from torchlet_amd.parts import FEED_FORWARDS
    g = torch.Generator().manual_seed(14)
    w = {"gate": torch.randn(inter, hidden, generator=g) * 2 * hidden ** -0.5, "up": torch.randn(inter, hidden, generator=g) * hidden ** -0.5,
         "down": torch.randn(hidden, inter, generator=g) * inter ** -0.5}
    w = {k: v.to(torch.bfloat16) for k, v in w.items()}
    ff = FEED_FORWARDS.build(SwiGLUSpec(hidden=hidden, intermediate=inter, activation="gelu_tanh", gate_name="gate", up_name="up", down_name="down"), dtype, torch.device("cuda"))
    ff.load_weights(w)
    h = torch.randn(T, hidden, generator=g).to(dtype)
    y = ff.forward(h.cuda(), None)
    y = y.sum(0) if y.dim() == 3 else y
    want = plain.gated_ff(h.double(), {k: v.double() for k, v in w.items()}, "", plain.gelu_tanh)
    torch.testing.assert_close(y.cpu().double(), want, **_tol(dtype))


def test_operands_that_do_not_fit_are_refused():
    from torchlet_amd.kernels import ops
    z = lambda *s, dt=torch.float32: torch.zeros(*s, dtype=dt, device="cuda")
    i = lambda *v: _i32(list(v))
    with pytest.raises(ops.KernelError):         # two kept groups of two experts hold no five choices
        ops.route(z(3, 8), 5, "all", groups=(4, 2))
    with pytest.raises(ops.KernelError):         # eight experts are no three equal groups
        ops.route(z(3, 8), 2, "all", groups=(3, 2))
    with pytest.raises(ops.KernelError):         # a norm with and without weights
        ops.head_norm_rotate(z(2, 8), 1, 1, 4, z(4), z(4), 1e-5, i(0, 1), None, 0, False, unit=True)
    with pytest.raises(ops.KernelError):         # a temperature without positions
        ops.head_norm_rotate(z(2, 8), 1, 1, 4, None, None, 1e-5, None, None, 0, False, heat=(0.1, 4))
    with pytest.raises(ops.KernelError):         # a gate of another size
        ops.heads_linear(z(2, 8), 4, z(2, 3, 4), z(2, 6), 3, gate=z(2, 5))
    with pytest.raises(ops.KernelError):
        ops.local_attention(z(1, 8), z(1, 8), z(2, 1, 4, 4), z(2, 1, 4, 4), i(1).view(1, 1), i(0), i(0), 2, 1, 4, 4, 4, 1.0, gate=z(1, 3))
    with pytest.raises(ops.KernelError):         # rows that do not hold the queries
        ops.latent_prepare(z(2, 20), 0, 4, 2, 2, None, z(4), 1e-5, i(0, 1), z(1), None, kv_off=8, queries=(z(2, 11), 2, 4, 2))
    with pytest.raises(ops.KernelError):
        ops.linear_swiglu(z(2, 8, dt=torch.bfloat16), z(64, 8, dt=torch.bfloat16), z(2, 32, dt=torch.bfloat16), "gelu")
