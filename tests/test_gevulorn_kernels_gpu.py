"""Each mechanism of the Gevulorn design alone: the kernel (or the part) against the plain function of tests/plain_gevulorn.py."""

import numpy as np
import pytest
import torch

import plain_gevulorn as plain

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]


def kernels():
    from mini_llm_amd.ops import kernels

    return kernels


def gpu(array, dtype=torch.float32):
    return torch.tensor(np.asarray(array), dtype=torch.float32).to(dtype).cuda().contiguous()


def ints(values):
    return torch.tensor(np.asarray(values), dtype=torch.int32).cuda()


def rounded(array, dtype):
    return torch.tensor(np.asarray(array), dtype=torch.float32).to(dtype).to(torch.float32).numpy().astype(np.float64)


def tol(dtype):
    return dict(atol=3e-5, rtol=3e-5) if dtype == torch.float32 else dict(atol=2e-2, rtol=2e-2)


# -- the sum of two branches and the norms behind it -----------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 7, 70])
@pytest.mark.parametrize("width", [5, 64, 100, 270, 768, 1000, 2048, 2500, 4100])
def test_a_sum_of_branches_and_two_norms_of_it(dtype, rows, width):
    k = kernels()
    rng = np.random.default_rng(width + rows)
    stream, a, b = rng.normal(1, 2, (rows, width)), rng.normal(0, 1, (3, rows, width)), rng.normal(0, 1, (rows, width))
    bias, vector = rng.normal(0, 1, width), rng.normal(0, 1, width)
    norms = [k.RowNorm(gpu(rng.normal(1, 0.3, width)), gpu(rng.normal(0, 0.3, width)), 1e-3, centred=True) for _ in range(2)]
    branches = [k.BranchRows(gpu(a), gpu(bias)), gpu(b)]
    total, made = k.join_norms(gpu(stream), branches, vector=gpu(vector), norms=norms, out_dtype=dtype)
    want = stream + a.sum(axis=0) + bias + b + vector
    np.testing.assert_allclose(total.cpu().numpy(), want, atol=2e-5, rtol=2e-5)
    for norm, got in zip(norms, made):
        assert got.dtype == dtype
        np.testing.assert_allclose(got.float().cpu().numpy(), plain.layer_norm(want, norm.gain.cpu().numpy(), norm.offset.cpu().numpy(), 1e-3), **tol(dtype))
    # fewer operands: one branch, one norm; a vector alone; nothing to add (the stream is then not written again)
    total, made = k.join_norms(gpu(stream), [None, gpu(a[:2])], norms=norms[1:], out_dtype=dtype)
    np.testing.assert_allclose(total.cpu().numpy(), stream + a[:2].sum(axis=0), atol=2e-5, rtol=2e-5)
    np.testing.assert_allclose(made[0].float().cpu().numpy(), plain.layer_norm(stream + a[:2].sum(axis=0), norms[1].gain.cpu().numpy(), norms[1].offset.cpu().numpy(), 1e-3),
                               **tol(dtype))
    total, made = k.join_norms(gpu(stream), vector=gpu(vector))
    np.testing.assert_allclose(total.cpu().numpy(), stream + vector, atol=1e-6, rtol=1e-6)
    assert made == []
    kept = gpu(stream)
    total, made = k.join_norms(kept, norms=norms, out_dtype=dtype)
    assert total is kept and len(made) == 2
    np.testing.assert_allclose(made[1].float().cpu().numpy(), plain.layer_norm(stream, norms[1].gain.cpu().numpy(), norms[1].offset.cpu().numpy(), 1e-3), **tol(dtype))
    # RMS norms, gains stored around zero
    rms = [k.RowNorm(norm.offset, None, 1e-2, centred=False, one_plus=True) for norm in norms]
    total, made = k.join_norms(gpu(stream), [gpu(b)], norms=rms, out_dtype=dtype)
    for norm, got in zip(rms, made):
        np.testing.assert_allclose(got.float().cpu().numpy(), plain.rms_norm(stream + b, 1e-2, 1.0 + norm.gain.cpu().numpy()), **tol(dtype))


def test_norms_of_two_kinds_are_not_joined():
    k = kernels()
    one = torch.ones(8).cuda()
    norms = [k.RowNorm(one, one, 1e-5, centred=True), k.RowNorm(one, one, 1e-6, centred=True), k.RowNorm(one, None, 1e-5, centred=False), None]
    assert k.shared_row_norms(norms[:1]) and not k.shared_row_norms(norms[:2]) and not k.shared_row_norms([norms[0], norms[2]])
    assert not k.shared_row_norms([norms[0], norms[3]]) and not k.shared_row_norms([])
    with pytest.raises(k.OperandError, match="one kind"):
        k.join_norms(torch.zeros(3, 8).cuda(), norms=norms[:2], out_dtype=torch.float32)
    with pytest.raises(k.OperandError, match="shape"):
        k.join_norms(torch.zeros(3, 8).cuda(), [torch.zeros(3, 9).cuda()])


def test_a_layer_norm_centres_before_it_squares():
    # rows far from zero: a variance taken as E[x^2] - E[x]^2 would have lost it all in 32 bits
    k = kernels()
    rng = np.random.default_rng(0)
    x = rounded(5000.0 + rng.normal(0, 0.5, (4, 768)), torch.float32)
    norm = k.RowNorm(torch.ones(768).cuda(), torch.zeros(768).cuda(), 1e-6, centred=True)
    _, made = k.join_norms(gpu(x), norms=[norm], out_dtype=torch.float32)
    np.testing.assert_allclose(made[0].cpu().numpy(), plain.layer_norm(x, 1.0, 0.0, 1e-6), atol=2e-3)


def test_capped_logits():
    k = kernels()
    x = np.random.default_rng(1).normal(0, 30, (5, 333))
    np.testing.assert_allclose(k.soft_cap(gpu(x), 12.5).cpu().numpy(), plain.soft_cap(x, 12.5), atol=2e-6, rtol=2e-6)
    t = gpu(x)
    assert k.soft_cap(t, 3.0, out=t) is t
    np.testing.assert_allclose(t.cpu().numpy(), plain.soft_cap(x, 3.0), atol=1e-6)


# -- normed and rotated rows -------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("unit", [True, False])
@pytest.mark.parametrize("lead", [3, 4])   # columns in front of the queries: with 4 the heads start on 16 bytes, and whole fours take the kernel for them
@pytest.mark.parametrize("dim,vdim,heads,kv_heads,rot_dims", [(16, 16, 4, 2, 16), (24, 8, 3, 3, 8), (8, 40, 2, 1, 0), (64, 64, 6, 2, 32), (10, 6, 3, 1, 4), (48, 80, 6, 1, 48),
                                                              (128, 128, 2, 1, 128), (192, 20, 1, 1, 64), (4, 4, 1, 1, 0)])
def test_rows_are_normed_and_rotated(dtype, unit, lead, dim, vdim, heads, kv_heads, rot_dims):
    k = kernels()
    rng = np.random.default_rng(dim + rot_dims)
    rows, page_size, n_pages, eps, base = 9, 16, 3, 1e-3, 700.0
    head_size = -(-max(dim, vdim) // 16) * 16
    positions, slots = [0, 1, 5, 63, 64, 5000, 2, 100000, 7], [4, 0, -1, 33, 20, 47, 19, 1, 2]
    q_width, k_width, v_width = heads * dim, kv_heads * dim, kv_heads * vdim
    width = lead + -(-(q_width + k_width + v_width) // 4) * 4 + (4 - lead % 4) % 4
    fused = rng.normal(0, 2, (rows, width))
    fused[6, lead : lead + dim] = 1e-3   # a query about as small as eps
    q_gain, k_gain = (1.0, 1.0) if unit else (rng.normal(1, 0.3, dim), rng.normal(1, 0.3, dim))
    frequencies = torch.tensor(plain.pair_frequencies(rot_dims, base) if rot_dims else [0.0], dtype=torch.float64).cuda()
    k_pages = torch.full((n_pages, kv_heads, page_size, head_size), 7.0, dtype=dtype).cuda()
    v_pages = torch.full_like(k_pages, 8.0)
    got = k.map_rows(gpu(fused), lead, lead + q_width, lead + q_width + k_width, None if unit else gpu(q_gain), None if unit else gpu(k_gain), eps, frequencies, rot_dims,
                     ints(positions), ints(slots), k_pages, v_pages, heads, kv_heads, 1, dim, vdim, unit=unit)
    split = lambda at, n, size: rounded(fused, torch.float32)[:, at : at + n * size].reshape(rows, n, size)
    made = lambda x, gain: plain.rotate_halves(plain.rms_norm(x, eps, gain), positions, rot_dims, base)
    want_q, want_k = made(split(lead, heads, dim), q_gain), made(split(lead + q_width, kv_heads, dim), k_gain)
    want_v = split(lead + q_width + k_width, kv_heads, vdim)
    got = got.float().cpu().numpy().reshape(rows, heads, head_size)
    np.testing.assert_allclose(got[:, :, :dim], want_q, **tol(dtype))
    assert (got[:, :, dim:] == 0).all()
    for pages, want, size, fill in ((k_pages, want_k, dim, 7.0), (v_pages, want_v, vdim, 8.0)):
        kept = pages.float().cpu().numpy().transpose(0, 2, 1, 3).reshape(n_pages * page_size, kv_heads, head_size)
        for row, slot in enumerate(slots):
            if slot >= 0:
                np.testing.assert_allclose(kept[slot, :, :size], want[row], **tol(dtype))
                assert (kept[slot, :, size:] == 0).all()
        assert (np.delete(kept, [s for s in slots if s >= 0], axis=0) == fill).all()


# -- windows that keep a sequence's first keys --------------------------------------------------------------------------------
def paged(keys, values, page_size, head_size, dtype, order):
    """Keys and values [T, G, d] of one request in pages taken in ``order``; one more page, the last, holds no numbers."""
    T, G, _ = keys.shape
    n_blocks = -(-T // page_size)
    k_pages = torch.zeros((max(order) + 2, G, page_size, head_size), dtype=dtype).cuda()
    v_pages = torch.zeros_like(k_pages)
    k_pages[-1], v_pages[-1] = float("nan"), float("nan")
    for b in range(n_blocks):
        rows = slice(b * page_size, min(T, (b + 1) * page_size))
        n = rows.stop - rows.start
        k_pages[order[b], :, :n, : keys.shape[2]] = gpu(keys[rows], dtype).transpose(0, 1)
        v_pages[order[b], :, :n, : values.shape[2]] = gpu(values[rows], dtype).transpose(0, 1)
    return k_pages, v_pages, [int(page) for page in order[:n_blocks]]


def without_the_gap(table, first_position, window, keep, page_size, spare):
    """The table as it stands when a step starts at ``first_position``: pages that hold neither kept keys nor keys of the window have been
    given back, and whatever another request has put there (no numbers, here) may not be looked at."""
    return [page if b * page_size < keep or b >= max(0, first_position - window + 1) // page_size else spare for b, page in enumerate(table)]


def every_way(k, q, k_pages, v_pages, table, common, want, dtype, page_size, portions=()):
    """The whole prompt at once, and portions of one and more rows over cached keys, each with the result in the pages' type and in 32-bit;
    and through the general kernel."""
    T = q.shape[0]
    rows, spare = gpu(q.reshape(T, -1), dtype), k_pages.shape[0] - 1
    for wide in (False, True):
        for at, n in ((0, T), *portions):
            tables = ints([without_the_gap(table, at, common["window"], common["keep_first"], page_size, spare)])
            batch = (ints(np.zeros(n)), ints(np.arange(at, at + n)), tables)
            got = k.paged_attention(rows[at : at + n], k_pages, v_pages, *batch, max_q_len=n, max_len=T, q_starts=ints([0, n]), context_lens=ints([at]), wide_out=wide, **common)
            np.testing.assert_allclose(got.float().cpu().numpy(), want[at : at + n], err_msg=f"rows {at}..{at + n - 1}", **tol(dtype))
            got = k.paged_attention(rows[at : at + n], k_pages, v_pages, *batch, wide_out=wide, **common)   # no queries' starts: a wave a (row, head)
            np.testing.assert_allclose(got.float().cpu().numpy(), want[at : at + n], err_msg=f"general, rows {at}..{at + n - 1}", **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("head_size,heads,kv_heads,window,keep,page_size", [
    (64, 4, 2, 40, 20, 16), (32, 2, 1, 16, 1, 32), (48, 3, 3, 70, 33, 16), (16, 2, 2, 5, 64, 16), (128, 2, 1, 64, 64, 64), (160, 1, 1, 33, 7, 16), (64, 2, 2, 1, 31, 32),
    (96, 2, 1, 249, 3, 16), (64, 8, 2, 1000, 100, 64), (64, 12, 4, 32, 32, 32), (128, 12, 3, 100, 130, 64), (32, 16, 4, 20, 299, 64)])
def test_a_window_that_keeps_the_first_keys(dtype, head_size, heads, kv_heads, window, keep, page_size):
    k = kernels()
    rng = np.random.default_rng(head_size + window)
    T = 300
    q = rounded(rng.normal(0, 1.5, (T, heads, head_size)), dtype)
    keys = rounded(rng.normal(0, 1.5, (T, kv_heads, head_size)), dtype)
    values = rounded(rng.normal(0, 1, (T, kv_heads, head_size)), dtype)
    sinks, scale = rng.normal(0, 2, heads), head_size ** -0.5 * 2.0
    want = plain.sink_attention(q, keys, values, scale, plain.window_mask(T, window, keep), sinks).reshape(T, -1)
    n_blocks = -(-T // page_size)
    k_pages, v_pages, table = paged(keys, values, page_size, head_size, dtype, list(rng.permutation(n_blocks + 2)))
    common = dict(n_heads=heads, n_kv_heads=kv_heads, head_size=head_size, scale=scale, window=window, keep_first=keep, sinks=gpu(sinks))
    portions = [(T - 1, 1), (T - 5, 5), (3, 1), (64, 2), (0, 1), (90, 210), (200, 70), (260, 9), (280, 20)]
    portions += [(e + d, 1) for e in (keep, window, keep + window) for d in (-1, 0, 1) if 0 <= e + d < T]
    every_way(k, q, k_pages, v_pages, table, common, want, dtype, page_size, portions)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep,at", [(40, 20, 19), (40, 20, 20), (64, 64, 63), (64, 64, 64), (100, 5, 0), (33, 1, 1), (16, 32, 31), (16, 32, 32), (7, 12, 200)])
def test_a_key_that_outscores_all_others_is_seen_where_it_should_be(dtype, window, keep, at):
    # among random keys a missing or an extra one hardly moves a softmax: one key is made ten times the others' size along the direction every
    # query looks in, with a value far from the others; kept, or the first that is not, or inside the window alone
    k = kernels()
    rng = np.random.default_rng(window + at)
    T, page_size, heads, head_size = 330, 16, 2, 64
    q, keys, values = rng.normal(0, 0.3, (T, heads, head_size)), rng.normal(0, 0.3, (T, 1, head_size)), rng.normal(0, 0.1, (T, 1, head_size))
    q[:, :, 5], keys[at, 0, 5], values[at, 0] = 4.0, 8.0, 50.0
    q, keys, values = rounded(q, dtype), rounded(keys, dtype), rounded(values, dtype)
    want = plain.sink_attention(q, keys, values, 1.0, plain.window_mask(T, window, keep), np.full(heads, -20.0)).reshape(T, -1)
    end = T if at < keep else at + window
    assert (want[at:end] > 49).all() and (end == T or np.abs(want[end:]).max() < 1) and (at == 0 or np.abs(want[:at]).max() < 1)
    k_pages, v_pages, table = paged(keys, values, page_size, head_size, dtype, list(rng.permutation(23)))
    common = dict(n_heads=heads, n_kv_heads=1, head_size=head_size, scale=1.0, window=window, keep_first=keep, sinks=gpu(np.full(heads, -20.0)))
    portions = [(at, 1), (min(end, T) - 1, 1), (max(0, at - 2), 5), (T - 100, 100)] + ([(end, 1), (end - 2, 4)] if end < T - 4 else [])
    every_way(k, q, k_pages, v_pages, table, common, want, dtype, page_size, portions)


@pytest.mark.parametrize("dtype", DTYPES)
def test_kept_keys_and_a_long_window_in_runs_of_keys(dtype):
    # one row over 300 kept keys and a window of 2,500 behind a gap of 2,700: the split-key kernel cuts what the row sees into runs
    k = kernels()
    rng = np.random.default_rng(1)
    T, page_size, heads, head_size, window, keep = 5500, 64, 2, 64, 2500, 300
    keys, values = rounded(rng.normal(0, 1, (T, 1, head_size)), dtype), rounded(rng.normal(0, 1, (T, 1, head_size)), dtype)
    q = rounded(rng.normal(0, 1, (1, heads, head_size)), dtype)
    keys[T - window - 1, 0], values[T - window - 1, 0] = 3.0 * q[0, 0], 40.0    # the last key before the window, and the first that is not kept:
    keys[keep, 0], values[keep, 0] = 3.0 * q[0, 1], 40.0                        # they would win if they were seen
    k_pages, v_pages, table = paged(keys, values, page_size, head_size, dtype, list(range(86)))
    seen = np.r_[0:keep, T - window : T]
    scores = np.einsum("hd,td->ht", q[0], keys[seen, 0]) * 0.2
    w = np.exp(scores - scores.max(axis=1, keepdims=True))
    want = (w @ values[seen, 0]) / w.sum(axis=1)[:, None]
    tables = ints([without_the_gap(table, T - 1, window, keep, page_size, k_pages.shape[0] - 1)])
    got = k.paged_attention(gpu(q.reshape(1, -1), dtype), k_pages, v_pages, ints([0]), ints([T - 1]), tables, heads, 1, head_size, 0.2, max_q_len=1, max_len=T,
                            q_starts=ints([0, 1]), context_lens=ints([T - 1]), window=window, keep_first=keep)
    np.testing.assert_allclose(got.float().cpu().numpy().reshape(heads, head_size), want, **(dict(atol=2e-5, rtol=2e-4) if dtype == torch.float32 else tol(dtype)))


@pytest.mark.parametrize("dtype", DTYPES)
def test_kept_keys_in_a_batch_of_unequal_portions(dtype):
    # many requests in one call (64 queries a block), at different depths, one of them shorter than what is kept
    k = kernels()
    rng = np.random.default_rng(2)
    page_size, heads, kv_heads, head_size, window, keep, scale = 32, 12, 4, 64, 50, 40, 0.3
    shapes = [(0, 300), (700, 129), (500, 1), (70, 65), (0, 20), (1000, 100), (0, 500)] * 3
    spare = sum(-(-(c + n) // page_size) for c, n in shapes)
    k_pages = torch.zeros((spare + 1, kv_heads, page_size, head_size), dtype=dtype).cuda()
    v_pages = torch.zeros_like(k_pages)
    k_pages[spare], v_pages[spare] = float("nan"), float("nan")
    order = rng.permutation(spare).tolist()
    tables = np.full((len(shapes), 40), spare, dtype=np.int32)
    qs, owner, positions, wants = [], [], [], []
    for r, (context, n) in enumerate(shapes):
        T = context + n
        q, keys, values = (rounded(rng.normal(0, 1.5, (T, h, head_size)), dtype) for h in (heads, kv_heads, kv_heads))
        wants.append(plain.sink_attention(q, keys, values, scale, plain.window_mask(T, window, keep), np.full(heads, -30.0))[context:].reshape(n, -1))
        for b in range(-(-T // page_size)):
            page = order.pop()
            chunk = slice(b * page_size, min(T, (b + 1) * page_size))
            k_pages[page, :, : chunk.stop - chunk.start] = gpu(keys[chunk], dtype).transpose(0, 1)
            v_pages[page, :, : chunk.stop - chunk.start] = gpu(values[chunk], dtype).transpose(0, 1)
            if b * page_size < keep or b >= max(0, context - window + 1) // page_size:
                tables[r, b] = page
        qs.append(q[context:].reshape(n, -1))
        owner += [r] * n
        positions += list(range(context, T))
    starts = np.cumsum([0] + [n for _, n in shapes])
    got = k.paged_attention(gpu(np.concatenate(qs), dtype), k_pages, v_pages, ints(owner), ints(positions), ints(tables), heads, kv_heads, head_size, scale, window=window,
                            keep_first=keep, max_q_len=500, max_len=1100, q_starts=ints(starts), context_lens=ints([c for c, _ in shapes]))
    np.testing.assert_allclose(got.float().cpu().numpy(), np.concatenate(wants), **tol(dtype))


# -- a memory whose channels fade at a pace of their own -----------------------------------------------------------------------
def memory_operands(rng, rows, heads, dim, vdim, rank, lead=3, z_scale=2.0, z_mean=1.0):
    q, k = rng.normal(0, 1, (rows, heads * dim)), rng.normal(0, 1, (rows, heads * dim))
    v, g, low = rng.normal(0, 1, (rows, heads * vdim)), rng.normal(0, 1, (rows, heads * vdim)), rng.normal(0, 1, (rows, rank))
    up, bias = rng.normal(0, z_scale * rank ** -0.5, (rank, heads * dim)), rng.normal(z_mean, 1.0, heads * dim)
    at = {}
    width = lead
    for name, part in (("q", q), ("k", k), ("v", v), ("g", g), ("low", low)):
        at[name] = width
        width += part.shape[1]
    fused = np.zeros((rows, width + 2))
    for name, part in (("q", q), ("k", k), ("v", v), ("g", g), ("low", low)):
        fused[:, at[name] : at[name] + part.shape[1]] = part
    return rounded(fused, torch.float32), at, rounded(up, torch.float32), rounded(bias, torch.float32)


def plain_memory(fused, at, up, bias, heads, dim, vdim, tau, q_scale, gain, eps, state):
    T = fused.shape[0]
    cut = lambda name, size: fused[:, at[name] : at[name] + heads * size].reshape(T, heads, size)
    alpha = plain.decays((fused[:, at["low"] : at["low"] + up.shape[0]] @ up + bias).reshape(T, heads, dim), tau)
    o, last = plain.decayed_memory(cut("q", dim) * q_scale, cut("k", dim), cut("v", vdim), alpha, state)
    return (plain.rms_norm(o, eps, gain) * plain.silu(cut("g", vdim))).reshape(T, -1), last


# (heads, dim, vdim, rank, tau): sizes off every multiple; heads whose values a block holds and ones it does not; chunks of 64 and of 32 rows;
# decays from all but none (tau 50) to ones that leave nothing of a row a few rows on (tau 0.05: pairs of rows one by one)
MEMORIES = [(2, 16, 24, 6, 8.0), (3, 7, 13, 5, 3.0), (1, 1, 1, 1, 1.0), (2, 96, 128, 16, 16.0), (4, 48, 64, 33, 2.0), (1, 200, 40, 16, 0.5), (2, 40, 200, 16, 30.0),
            (2, 64, 64, 64, 50.0), (2, 33, 17, 8, 0.05), (1, 128, 256, 16, 1.0), (1, 256, 100, 4, 6.0), (1, 100, 300, 8, 2.0), (1, 300, 60, 8, 2.0), (5, 32, 128, 20, 0.3)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,vdim,rank,tau", MEMORIES)
def test_memory_over_portions_slots_and_padding(dtype, heads, dim, vdim, rank, tau):
    # requests in portions of changing size beside single rows, in slots nobody's neighbours touch, with a padding request in every batch
    k = kernels()
    rng = np.random.default_rng(dim * 7 + vdim)
    eps, q_scale, n_slots = 1e-4, dim ** -0.5, 5
    gain = rng.normal(1, 0.2, vdim)
    slots_of = {"a": 3, "b": 0, "c": 2}
    state = torch.full((n_slots, heads * dim * vdim + 3), 9.0).cuda()
    for slot in slots_of.values():
        state[slot] = 0.0
    up = bias = None
    kept = {name: None for name in slots_of}
    bound = dict(atol=2e-4, rtol=2e-4) if dtype == torch.float32 else tol(dtype)
    for step in ([("a", 5), ("b", 1)], [("b", 2), ("a", 1), ("c", 150)], [("a", 70), ("b", 9), ("c", 1)], [("c", 64), ("a", 33), ("b", 16)], [("a", 1), ("b", 1), ("c", 1)],
                 [("b", 17), ("c", 129)], [("a", 8), ("c", 3)]):
        n = sum(size for _, size in step)
        fused, at, new_up, new_bias = memory_operands(rng, n + 2, heads, dim, vdim, rank)
        up, bias = (new_up, new_bias) if up is None else (up, bias)
        starts = np.concatenate([[0], np.cumsum([size for _, size in step]), [n + 2]])   # two padding rows of a request without a slot
        slots = [slots_of[name] for name, _ in step] + [-1]
        out = k.channel_memory(gpu(fused), at["q"], at["k"], at["v"], at["g"], at["low"], gpu(up), gpu(bias), state, ints(starts), ints(slots), heads, dim, vdim, tau=tau,
                               q_scale=q_scale, gain=gpu(gain), eps=eps, out_dtype=dtype, max_q_len=max(size for _, size in step)).float().cpu().numpy()
        for i, (name, size) in enumerate(step):
            rows = slice(starts[i], starts[i] + size)
            want, kept[name] = plain_memory(fused[rows], at, up, bias, heads, dim, vdim, tau, q_scale, gain, eps, kept[name])
            np.testing.assert_allclose(out[rows], want, err_msg=f"{step} {name}", **bound)
            got = state[slots_of[name], : heads * dim * vdim].cpu().numpy().reshape(heads, dim, vdim)
            np.testing.assert_allclose(got, kept[name], atol=1e-4, rtol=1e-4, err_msg=f"{step} {name}: state")
        assert (state[[1, 4]] == 9.0).all() and (state[:, heads * dim * vdim :][[0, 2, 3]] == 0.0).all()


@pytest.mark.parametrize("tau", [1.0, 20.0])
def test_a_row_is_remembered_as_long_as_its_channels_last(tau):
    # one row writes a value far above all others; half of the channels hardly fade (their gates all but open), the others are gone in a few
    # rows. 700 rows on, through chunks and row by row, the result is what the lasting channels hold.
    k = kernels()
    rng = np.random.default_rng(3)
    heads, dim, vdim, rank, T = 1, 32, 16, 4, 700
    fused, at, up, bias = memory_operands(rng, T, heads, dim, vdim, rank)
    up[:] = 0.0
    bias[: dim // 2], bias[dim // 2 :] = 14.0, -4.0 * tau
    fused[:, at["v"] : at["v"] + vdim] *= 0.01
    fused[5, at["v"] : at["v"] + vdim] = 40.0
    gain = np.ones(vdim)
    want, last = plain_memory(fused, at, up, bias, heads, dim, vdim, tau, 1.0, gain, 1e-6, None)
    forgotten, _ = plain_memory(np.delete(fused, 5, axis=0), at, up, bias, heads, dim, vdim, tau, 1.0, gain, 1e-6, None)
    assert np.abs(want[-1] - forgotten[-1]).max() > 0.3
    for sizes in ((700,), (1,) * 20 + (680,), (640, 60), (699, 1), (8,) * 87 + (4,), (100,) * 7):
        state = torch.zeros((1, dim * vdim)).cuda()
        made, lo = [], 0
        for n in sizes:
            made.append(k.channel_memory(gpu(fused[lo : lo + n]), at["q"], at["k"], at["v"], at["g"], at["low"], gpu(up), gpu(bias), state, ints([0, n]), ints([0]), heads, dim, vdim,
                                         tau=tau, q_scale=1.0, gain=gpu(gain), eps=1e-6, out_dtype=torch.float32, max_q_len=n).cpu().numpy())
            lo += n
        np.testing.assert_allclose(np.concatenate(made), want, atol=3e-4, rtol=3e-4, err_msg=str(sizes[:3]))
        np.testing.assert_allclose(state.cpu().numpy().reshape(last.shape), last, atol=1e-3, rtol=1e-4)


def test_gated_norm_with_silu_and_one_gain_for_all_groups():
    k = kernels()
    rng = np.random.default_rng(4)
    for groups, size in ((3, 20), (2, 300), (1, 5000)):
        x, gate, gain = rng.normal(0, 1, (6, groups * size)), rng.normal(0, 2, (6, groups * size)), rng.normal(1, 0.2, size)
        out = torch.empty((6, groups * size)).cuda()
        k.gated_norm(gpu(x), gpu(gain), gpu(gate), 1e-4, out, group=size, silu=True)
        want = (plain.rms_norm(x.reshape(6, groups, size), 1e-4, gain)).reshape(6, -1) * plain.silu(gate)
        np.testing.assert_allclose(out.cpu().numpy(), want, atol=3e-5, rtol=3e-5)


# -- feed-forwards -------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 40, 65, 300])
@pytest.mark.parametrize("width,ff", [(64, 96), (100, 50), (256, 1024), (51, 18)])
def test_the_square_of_relu_in_a_dense_feed_forward(dtype, rows, width, ff):
    from mini_llm_amd.parts import make_part
    from mini_llm_amd.precision import Precision
    from mini_llm_amd.weights.loader import place

    k = kernels()
    rng = np.random.default_rng(width + rows)
    part = make_part("feed_forward", "plain_mlp", width=width, inner=ff, activation="squared_relu")
    tensors = {name: rounded(rng.normal(0, 1.5 * spec.shape[1] ** -0.5, spec.shape), dtype) for name, spec in part.tensor_specs().items()}
    precision = Precision.from_name("float32" if dtype == torch.float32 else "bfloat16")
    part.bind({name: place(torch.tensor(t, dtype=torch.float32), part.tensor_specs()[name], precision, "cuda:0") for name, t in tensors.items()})
    x, residual = rounded(rng.normal(0, 1, (rows, width)), dtype), rng.normal(0, 1, (rows, width))
    want = plain.dense_feed_forward(x, tensors, "")
    bound = dict(atol=2e-4, rtol=2e-4) if dtype == torch.float32 else dict(atol=6e-2, rtol=2e-2)
    np.testing.assert_allclose(k.settle(part.forward(gpu(x, dtype), gpu(residual))).cpu().numpy(), want + residual, **bound)
    part.sums_later = True
    branch = part.forward(gpu(x, dtype), None).rows
    np.testing.assert_allclose((branch.sum(dim=0) if branch.dim() == 3 else branch).cpu().numpy(), want, **bound)


def test_the_router_weighs_by_the_picked_sums_alone():
    k = kernels()
    rng = np.random.default_rng(5)
    for experts, top, always in ((6, 2, 0), (6, 6, 1), (1, 1, 2), (70, 4, 3), (64, 8, 1)):
        z = rng.normal(0, 3, (40, experts))
        z[3] -= 500.0   # scores are the same whatever all sums have in common
        if experts > 2:
            z[4], z[4, 2] = np.linspace(-300.0, -200.0, experts), 90.0   # all but one vanish beside the largest: the order stays that of the sums
        picks = k.route(gpu(z), experts, top, picks=True, always=always)
        want = plain.route(rounded(z, torch.float32), top)
        ids, weights = picks.experts.cpu().numpy(), picks.weights.cpu().numpy()
        assert ids.shape == (40, top + always) and (ids[:, top:] == experts + np.arange(always)).all() and (weights[:, top:] == 1.0).all()
        for t in range(40):
            order = np.argsort(-rounded(z, torch.float32)[t], kind="stable")[:top]
            assert ids[t, :top].tolist() == order.tolist()
            np.testing.assert_allclose(weights[t, :top], want[t, order], atol=2e-6, rtol=2e-5)
        np.testing.assert_allclose(k.route(gpu(z), experts, top).cpu().numpy(), want, atol=2e-6, rtol=2e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 16, 40, 65, 300])
@pytest.mark.parametrize("width,experts,ff,top,shared", [(64, 6, 40, 2, 56), (128, 8, 64, 1, 200), (192, 70, 96, 4, 96), (64, 3, 130, 3, 20), (100, 5, 24, 2, 33), (51, 1, 70, 1, 141),
                                                         (256, 12, 200, 4, None)])
def test_routed_experts_with_a_shared_one(dtype, rows, width, experts, ff, top, shared):
    from mini_llm_amd.parts import make_part

    part = make_part("feed_forward", "routed_experts", width=width, n_experts=experts, ff=ff, top=top, correction=False, unit="clamped_gate", limit=None, shared_ff=shared)
    rng = np.random.default_rng(rows + ff)
    tensors = {name: rounded(rng.normal(0, (2.0 if name.endswith(("gate", "router")) else 1.0) * spec.shape[1] ** -0.5, spec.shape), dtype)
               for name, spec in part.tensor_specs().items()}
    part.bind({name: gpu(t, dtype) for name, t in tensors.items()})
    x = rounded(rng.normal(0, 1, (rows, width)), dtype)
    mlp = {"expert": {"ff": ff}, "router": {"experts": experts, "top": top}, "shared": None if shared is None else {"ff": shared}}
    want = plain.routed_feed_forward(x, mlp, tensors, "")
    out = part.forward(gpu(x, dtype), None)
    bound = dict(atol=2e-4, rtol=2e-4) if dtype == torch.float32 else dict(atol=4e-2, rtol=2e-2)
    np.testing.assert_allclose((out.sum(dim=0) if out.dim() == 3 else out).cpu().numpy(), want, **bound)
    if shared:   # the shared expert is a part of the sum that shows
        assert np.abs(want - plain.routed_feed_forward(x, {**mlp, "shared": None}, tensors, "")).max() > 0.2
