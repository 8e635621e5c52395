"""Each mechanism of the Goletar design alone: the kernel (or the part) against the plain function of tests/plain_goletar.py."""

import numpy as np
import pytest
import torch

import plain_goletar as plain

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


# -- embedding ----------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mul_prev,mul_cur,buckets", [(31, 7, 50), (2**31 - 1, 2**31 - 1, 97), (0, 1, 1), (1, 0, 13)])
def test_token_pairs_across_portions_slots_and_tokens_on_the_device(dtype, mul_prev, mul_cur, buckets):
    k = kernels()
    rng = np.random.default_rng(buckets)
    vocab, width = 60000, 72
    table, pair_table = rounded(rng.normal(0, 1, (vocab, width)), dtype), rounded(rng.normal(0, 1, (buckets + 1, width)), dtype)
    wte, wpairs = gpu(table, dtype), gpu(pair_table, dtype)
    config = {"embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}}
    slots_of = {"a": 3, "b": 0, "c": 2}
    previous = ints([-7, 123, 456, 59999])   # a slot keeps what its last owner left: a sequence's first token must not look at it
    token_slots = ints([11, 12, 13, 14])
    fed = {name: [] for name in slots_of}
    steps = [[("a", 5), ("b", 1)], [("b", 2), ("a", 1), ("c", 300)], [("a", 2), ("b", 1), ("c", 1)], [("c", 7), ("a", 40)], [("a", 1), ("b", 1), ("c", 1)]]
    for number, step in enumerate(steps):
        from_device = number == len(steps) - 1   # the last step's tokens lie in the last-token slots
        tokens, positions, owner, starts, slots, sources = [], [], [], [0], [], []
        for at, (name, n) in enumerate(step):
            new = rng.integers(0, vocab, n).tolist()
            if from_device:
                new = [int(token_slots[slots_of[name]])]
            positions += list(range(len(fed[name]), len(fed[name]) + n))
            fed[name] += new
            tokens += [0] if from_device else new
            sources += [slots_of[name] if from_device else -1] * n
            owner += [at] * n
            starts.append(starts[-1] + n)
            slots.append(slots_of[name])
        # a padding row of no request behind the others, as a captured step has
        tokens, positions, owner, sources = tokens + [-1], positions + [0], owner + [-1], sources + [-1]
        pairs = k.TokenPairs(wpairs, mul_prev, mul_cur, ints(owner), ints(starts + [starts[-1]]), ints(slots + [-1]), previous)
        got = k.embed(ints(tokens), ints(positions), wte, None, token_sources=ints(sources) if from_device else None,
                      token_slots=token_slots if from_device else None, pairs=pairs).cpu().numpy()
        for at, (name, n) in enumerate(step):
            want = plain.embedding(fed[name], config, {"embed": table, "bigram": pair_table})[-n:]
            np.testing.assert_allclose(got[starts[at] : starts[at] + n], want, atol=1e-6, rtol=1e-6, err_msg=f"step {number} request {name}")
        assert (got[-1] == 0).all()
        assert previous.cpu().tolist()[1] == 123   # nobody's slot
        for name, n in step:
            assert int(previous[slots_of[name]]) == fed[name][-1]


# -- latent attention ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,rot,rot_dims,rank", [(3, 16, 8, 8, 40), (1, 5, 6, 4, 21), (2, 64, 32, 32, 64), (4, 8, 0, 0, 16)])
def test_latent_rows_of_neighbouring_pairs(dtype, heads, dim, rot, rot_dims, rank):
    k = kernels()
    rng = np.random.default_rng(rank)
    rows, page_size, n_pages, eps, base = 7, 16, 3, 1e-5, 700.0
    row_size = -(-(rank + rot + 5) // 8) * 8
    positions, slots = [0, 1, 5, 63, 64, 5000, 2], [4, 0, -1, 33, 20, 47, 19]
    q, dkv = rounded(rng.normal(0, 1, (rows, heads * (dim + rot))), dtype), rounded(rng.normal(0, 1, (rows, rank + rot)), dtype)
    gain = rng.normal(1, 0.2, rank)
    frequencies = torch.tensor(plain.pair_frequencies(rot_dims, base) if rot_dims else [0.0], dtype=torch.float64).cuda()
    pages = torch.full((n_pages, 1, page_size, row_size), 7.0, dtype=dtype).cuda()
    q_full = k.latent_rows(gpu(q, dtype), gpu(dkv, dtype), gpu(gain), eps, frequencies, 1.0, rot_dims, ints(positions), ints(slots), pages, heads, dim, rot, rank,
                           pairing="neighbours").cpu().numpy()
    want_q = plain.rotate_neighbours(q.reshape(rows, heads, dim + rot)[:, :, dim:], positions, rot_dims, base)
    np.testing.assert_allclose(q_full[:, :, rank : rank + rot], want_q, atol=2e-6, rtol=2e-6)
    assert (q_full[:, :, rank + rot :] == 0).all()
    kept = pages.float().cpu().numpy().reshape(n_pages * page_size, row_size)
    want_c, want_r = plain.rms_norm(dkv[:, :rank], gain, eps), plain.rotate_neighbours(dkv[:, rank:], positions, rot_dims, base)
    for row, slot in enumerate(slots):
        if slot >= 0:
            np.testing.assert_allclose(kept[slot, :rank], want_c[row], **tol(dtype))
            np.testing.assert_allclose(kept[slot, rank : rank + rot], want_r[row], **(tol(dtype) if dtype == torch.bfloat16 else dict(atol=2e-6, rtol=2e-6)))
            assert (kept[slot, rank + rot :] == 0).all()
    assert (np.delete(kept, [s for s in slots if s >= 0], axis=0) == 7).all()


@pytest.mark.parametrize("sink", [True, False])
@pytest.mark.parametrize("heads,rank,rot,page_size", [(3, 24, 8, 16), (6, 64, 32, 64), (2, 100, 20, 32), (17, 160, 32, 64), (5, 256, 32, 64), (1, 61, 3, 8)])
def test_latent_attention_on_the_matrix_cores(heads, rank, rot, page_size, sink):
    # A batch of portions at any depth, single tokens among them, and rows of no request behind; every row's query makes one key stand out:
    # its sequence's first, the last it sees, or one beside the borders of pages and of the 32 and 128 keys a wave and a block take at a
    # time. One key further on, which the row must not see, would stand out still more.
    k = kernels()
    rng = np.random.default_rng(rank)
    contexts, portions = [0, 130, 1000, 31, 700, 127], [150, 2, 1, 97, 33, 129]
    row_size, pad = k.latent_row_size(rank + rot), 5
    assert k.library().mllm_latent_attention_mfma_supported(rank, row_size, 1)
    lengths = [c + n for c, n in zip(contexts, portions)]
    n_blocks = [-(-n // page_size) for n in lengths]
    order = rng.permutation(sum(n_blocks) + 2)
    pages = torch.zeros((len(order), 1, page_size, row_size), dtype=torch.bfloat16)
    tables, cached, at = np.full((len(lengths) + 1, max(n_blocks) + 1), -1, dtype=np.int32), [], 0
    for r, n in enumerate(lengths):
        rows = rounded(rng.normal(0, 1, (n, row_size)), torch.bfloat16)
        rows[:, rank + rot :] = 0
        cached.append(rows)
        for b in range(n_blocks[r]):
            tables[r, b] = order[at]
            chunk = rows[b * page_size : (b + 1) * page_size]
            pages[order[at], 0, : len(chunk)] = torch.tensor(chunk).to(torch.bfloat16)
            at += 1
    total = sum(portions)
    starts = np.concatenate([[0], np.cumsum(portions), [total + pad]])
    owner, positions = np.full(total + pad, -1), np.zeros(total + pad, dtype=int)
    q = rng.normal(0, 0.1, (total + pad, heads, row_size))
    borders = (0, 31, 32, 63, 64, 127, 128, 255, 256, 999)
    for r, (c, n) in enumerate(zip(contexts, portions)):
        for i in range(n):
            row, position = starts[r] + i, c + i
            owner[row], positions[row] = r, position
            seen = [b for b in borders if b <= position] + [position]
            hot = seen[int(rng.integers(len(seen)))] if i % 3 else position
            q[row] += cached[r][hot] * 20.0 / np.linalg.norm(cached[r][hot])
            if position + 1 < lengths[r]:
                q[row] += cached[r][position + 1] * 40.0 / np.linalg.norm(cached[r][position + 1])
    q[:, :, rank + rot :] = 0
    q = rounded(q, torch.bfloat16)
    sinks, scale = rng.normal(0, 1, heads), 0.5
    for max_len, longest in ((max(lengths), max(portions)), (8 * max(lengths), total)):   # bounds as they are, and as a captured step gives them
        got = k.latent_attention(gpu(q), pages.cuda(), gpu(sinks) if sink else None, ints(owner), ints(positions), ints(tables), rank, scale, max_len=max_len,
                                 q_starts=ints(starts), context_lens=ints(contexts + [-1]), max_q_len=longest).cpu().numpy()
        assert (got[total:] == 0).all()
        for row in range(total):
            keys = cached[owner[row]][: positions[row] + 1]
            scores = q[row] @ keys.T * scale
            weights = np.exp(scores - scores.max(axis=1, keepdims=True))
            bottom = weights.sum(axis=1, keepdims=True) + (np.exp(sinks[:, None] - scores.max(axis=1, keepdims=True)) if sink else 0.0)
            np.testing.assert_allclose(got[row], weights @ keys[:, :rank] / bottom, atol=4e-2, rtol=3e-2, err_msg=f"row {row} position {positions[row]}")


@pytest.mark.parametrize("sink", [True, False])
def test_latent_attention_of_few_rows_with_many_keys(sink):
    # runs of keys by different blocks, put together behind them; rows of no request between and behind
    k = kernels()
    rng = np.random.default_rng(7)
    heads, rank, rot, page_size, length, row_size = 4, 64, 32, 64, 3000, 96
    cached = rounded(rng.normal(0, 1, (length, row_size)), torch.bfloat16)
    blocks = -(-length // page_size)
    pages = torch.zeros((blocks, 1, page_size, row_size), dtype=torch.bfloat16)
    pages.view(-1, row_size)[:length] = torch.tensor(cached).to(torch.bfloat16)
    tables = np.stack([np.arange(blocks)] * 3)
    sinks = rng.normal(0, 1, heads)
    for hot in (0, 127, 128, 1535, 1536, 2998, 2999):
        positions = [2999, 0, 2998]
        q = np.tile(cached[hot] * 30.0 / np.linalg.norm(cached[hot]), (3, heads, 1)) + rng.normal(0, 0.1, (3, heads, row_size))
        q = rounded(q, torch.bfloat16)
        got = k.latent_attention(gpu(q), pages.cuda(), gpu(sinks) if sink else None, ints([0, -1, 2]), ints(positions), ints(tables), rank, 1.0, max_len=length,
                                 q_starts=ints([0, 1, 2, 3]), context_lens=ints([2999, -1, 2998]), max_q_len=1).cpu().numpy()
        assert (got[1] == 0).all()
        for row in (0, 2):
            keys = cached[: positions[row] + 1]
            scores = q[row] @ keys.T
            top = np.maximum(scores.max(axis=1, keepdims=True), sinks[:, None] if sink else -np.inf)
            weights = np.exp(scores - top)
            want = weights @ keys[:, :rank] / (weights.sum(axis=1, keepdims=True) + (np.exp(sinks[:, None] - top) if sink else 0.0))
            np.testing.assert_allclose(got[row], want, atol=4e-2, rtol=3e-2, err_msg=f"hot key {hot} row {row}")


@pytest.mark.parametrize("w_dtype", DTYPES)
@pytest.mark.parametrize("rows,heads,n,k_size", [(1, 3, 40, 16), (17, 2, 24, 64), (33, 5, 48, 21), (5, 6, 7, 512), (70, 3, 130, 32)])
def test_heads_linear_with_a_gate_a_head(w_dtype, rows, heads, n, k_size):
    k = kernels()
    rng = np.random.default_rng(rows)
    x, w, gate = rng.normal(0, 1, (rows, heads, k_size)), rounded(rng.normal(0, 1, (heads, n, k_size)), w_dtype), rng.normal(0, 2, (rows, heads + 3))
    out = torch.empty((rows, heads, n), dtype=torch.float32).cuda()
    k.heads_linear(gpu(x), gpu(w, w_dtype), out, n_heads=heads, k=k_size, x_head_stride=k_size, gate=gpu(gate)[:, 1 : 1 + heads])
    want = np.einsum("thk,hnk->thn", x, w) * plain.sigmoid(gate[:, 1 : 1 + heads])[:, :, None]
    np.testing.assert_allclose(out.cpu().numpy(), want, **(dict(atol=1e-4, rtol=1e-4) if w_dtype == torch.float32 else dict(atol=0.02 * k_size**0.5, rtol=2e-2)))


# -- gated recurrence ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("lengths", [[1, 1, 1], [3, 16, 1], [17, 2], [64, 65, 1, 63], [200, 1, 129, 2, 128], [700, 5]])
@pytest.mark.parametrize("width", [1, 40, 64, 300])
def test_gated_scan(dtype, lengths, width):
    k = kernels()
    rng = np.random.default_rng(width + len(lengths))
    total, pad = sum(lengths), 3
    rows = rng.normal(0, 2, (total + pad, 3 * width + 5))
    rows[:, 2 : 2 + width] -= 2.0            # update gates that mostly keep the state
    rows[5 % total, 2 : 2 + width] = 60.0    # one that takes the candidate alone, and one that keeps the state as it is
    rows[total - 1, 2 : 2 + width] = -60.0
    rows[0, 2 + width : 2 + 2 * width] = 0.0     # the candidate's border
    state = rng.normal(0, 1, (len(lengths) + 2, width + 7))
    slots = [len(lengths) + 1 - i for i in range(len(lengths))]
    starts = np.concatenate([[0], np.cumsum(lengths)])
    device_state, device_rows = gpu(state), gpu(rows)
    # behind the requests one of padding, which spans the rows nobody owns
    got = k.gated_scan(device_rows, 2, 2 + width, 4 + 2 * width, width, device_state, ints(list(starts) + [total + pad]), ints(slots + [-1]), dtype,
                       shift=plain.CANDIDATE_SHIFT, max_q_len=max(lengths)).float().cpu().numpy()
    rows = device_rows.cpu().numpy().astype(np.float64)
    want_state = device_state.cpu().numpy().astype(np.float64)
    for at, slot in enumerate(slots):
        r = rows[starts[at] : starts[at + 1]]
        states, last = plain.gated_scan(plain.sigmoid(r[:, 2 : 2 + width]), plain.recurrence_candidate(r[:, 2 + width : 2 + 2 * width]),
                                        state[slot, :width].astype(np.float32).astype(np.float64))
        want = states * plain.silu(r[:, 4 + 2 * width : 4 + 3 * width])
        np.testing.assert_allclose(got[starts[at] : starts[at + 1]], want, **(dict(atol=1e-5, rtol=2e-5) if dtype == torch.float32 else tol(dtype)))
        np.testing.assert_allclose(want_state[slot, :width], last, atol=1e-5, rtol=2e-5)
    untouched = np.delete(want_state, slots, axis=0)
    np.testing.assert_array_equal(untouched, np.delete(state, slots, axis=0).astype(np.float32))
    np.testing.assert_array_equal(want_state[:, width:], state[:, width:].astype(np.float32))


def test_a_scan_of_one_portion_and_of_many_small_ones_agree():
    k = kernels()
    rng = np.random.default_rng(4)
    width, total = 130, 333
    rows = gpu(rng.normal(0, 1.5, (total, 3 * width)))
    whole_state = torch.zeros((1, width)).cuda()
    whole = k.gated_scan(rows, 0, width, 2 * width, width, whole_state, ints([0, total]), ints([0]), torch.float32, shift=0.5)
    state, at, parts = torch.zeros((1, width)).cuda(), 0, []
    for n in (2, 70, 1, 16, 17, 64, 65, 2, 96):
        parts.append(k.gated_scan(rows[at : at + n], 0, width, 2 * width, width, state, ints([0, n]), ints([0]), torch.float32, shift=0.5, max_q_len=n))
        at += n
    assert at == total
    torch.testing.assert_close(torch.cat(parts), whole, atol=2e-6, rtol=1e-5)
    torch.testing.assert_close(state, whole_state, atol=2e-6, rtol=1e-5)


# -- experts ------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,experts,top", [(1, 64, 8, 1), (5, 40, 8, 2), (130, 72, 3, 3), (33, 256, 64, 7), (9, 128, 1, 1), (70, 512, 13, 4)])
def test_router_with_its_product_and_without(dtype, rows, width, experts, top):
    k = kernels()
    rng = np.random.default_rng(rows)
    x, router = rounded(rng.normal(0, 1, (rows, width)), dtype), rounded(rng.normal(0, 2 * width**-0.5, (experts, width)), dtype)
    want = plain.route(x @ router.T, top)
    assert k.route_rows_supported(experts, width, dtype)
    how = dict(score="sigmoid", renormalise=False)
    dense = k.route_rows(gpu(x, dtype), gpu(router, dtype), top, **how)
    picks = k.route_rows(gpu(x, dtype), gpu(router, dtype), top, picks=True, **how)
    logits = gpu(x @ router.T)
    again = k.route(logits, experts, top, picks=True, **how)
    np.testing.assert_allclose(dense.cpu().numpy(), want, atol=2e-6, rtol=2e-6)
    np.testing.assert_allclose(k.route(logits, experts, top, **how).cpu().numpy(), want, atol=2e-6, rtol=2e-6)
    for some in (picks, again):
        ids, weights = some.experts.cpu().numpy(), some.weights.cpu().numpy()
        scattered = np.zeros((rows, experts))
        scattered[np.arange(rows)[:, None], ids] = weights
        np.testing.assert_allclose(scattered, want, atol=2e-6, rtol=2e-6)
        assert (np.diff(weights, axis=1) <= 0).all()   # in the order of their scores
    # the softmax form, renormalised over the picks
    s = np.exp(x @ router.T)
    s /= s.sum(axis=1, keepdims=True)
    chosen = np.argsort(-s, axis=1, kind="stable")[:, :top]
    soft = np.zeros_like(s)
    np.put_along_axis(soft, chosen, np.take_along_axis(s, chosen, 1) / np.take_along_axis(s, chosen, 1).sum(1, keepdims=True), 1)
    np.testing.assert_allclose(k.route_rows(gpu(x, dtype), gpu(router, dtype), top).cpu().numpy(), soft, atol=1e-5, rtol=1e-4)


def test_router_leaves_no_pick_where_the_sums_are_no_numbers():
    k = kernels()
    logits = gpu(np.array([[0.5, np.nan, 0.1], [1.0, 2.0, 3.0]]))
    logits[0, :] = float("nan")
    picks = k.route(logits, 3, 2, score="sigmoid", renormalise=False, picks=True)
    assert picks.experts.cpu().tolist() == [[-1, -1], [2, 1]]
    assert k.route(logits, 3, 2, score="sigmoid", renormalise=False).cpu()[0].tolist() == [0.0, 0.0, 0.0]


def experts_part(width, experts, ff, top, dtype, seed, limit=1.0, weigh="input"):
    from mini_llm_amd.parts import make_part

    part = make_part("feed_forward", "routed_experts", width=width, n_experts=experts, ff=ff, top=top, correction=False, score="sigmoid", renormalise=False,
                     unit="clamped_gate", limit=limit, alpha=plain.QUICK_SIGMOID, shift=plain.UP_SHIFT, weigh=weigh)
    rng = np.random.default_rng(seed)
    tensors = {}
    for name, spec in part.tensor_specs().items():
        scale = 2.0 if name.endswith(("gate", "up")) or name == "router" else 1.0
        tensors[name] = rounded(rng.normal(0, scale * spec.shape[1] ** -0.5, spec.shape), dtype)
    part.bind({name: gpu(t, dtype) for name, t in tensors.items()})
    return part, tensors


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 7, 16, 17, 32, 40, 64, 65, 130, 500])
@pytest.mark.parametrize("width,experts,ff,top", [(64, 6, 40, 2), (128, 8, 64, 1), (192, 70, 96, 4), (64, 3, 130, 3), (1088, 4, 1100, 2), (100, 5, 24, 2), (72, 9, 200, 3), (51, 4, 70, 2)])
def test_routed_experts_part(dtype, rows, width, experts, ff, top):
    # few rows (up to 64) in the products that find their rows themselves, more in the grouped ones: bfloat16 with a width of whole 64s in
    # the streaming kernel, else in the tiled one, and a width that is not even whole pieces of 16 bytes there from the first row on
    part, tensors = experts_part(width, experts, ff, top, dtype, seed=rows + ff)
    rng = np.random.default_rng(rows)
    x = rounded(rng.normal(0, 1, (rows, width)), dtype)
    if rows > 16:
        x[3 : rows // 2] = x[2]   # many rows of one expert, so that its tiles fill and others stay empty
    mlp = {"expert": {"ff": ff, "limit": 1.0}, "router": {"experts": experts, "top": top}}
    want = plain.routed_feed_forward(x, mlp, tensors, "")
    out = part.forward(gpu(x, dtype), None)
    got = (out.sum(dim=0) if out.dim() == 3 else out).cpu().numpy()
    bound = dict(atol=2e-4, rtol=2e-4) if dtype == torch.float32 else dict(atol=3e-2, rtol=2e-2)
    np.testing.assert_allclose(got, want, **bound)
    residual = rng.normal(0, 1, (rows, width))
    added = part.forward(gpu(x, dtype), gpu(residual))
    np.testing.assert_allclose(kernels().settle(added).cpu().numpy(), want + residual, **bound)


def test_an_expert_row_does_not_depend_on_its_batch():
    # a row's result from the products of few rows, alone and among others, and from the grouped products of many
    part, _ = experts_part(128, 6, 96, 2, torch.bfloat16, seed=5)
    x = gpu(np.random.default_rng(5).normal(0, 1, (300, 128)), torch.bfloat16)
    many = part.forward(x, None).sum(dim=0)
    few = part.forward(x[:64].contiguous(), None).sum(dim=0)
    alone = torch.cat([part.forward(x[i : i + 1].contiguous(), None).sum(dim=0) for i in range(0, 64, 7)])
    torch.testing.assert_close(few, many[:64], atol=1e-2, rtol=1e-2)
    torch.testing.assert_close(alone, few[::7], atol=1e-2, rtol=1e-2)


def test_experts_that_weigh_their_output():
    part, tensors = experts_part(64, 5, 40, 2, torch.bfloat16, seed=9, weigh="output", limit=None)
    x = rounded(np.random.default_rng(9).normal(0, 1, (90, 64)), torch.bfloat16)
    weights = plain.route(x @ tensors["router"].T, 2)
    want = np.zeros_like(x)
    for e in range(5):
        want += weights[:, e, None] * plain.expert(x, tensors[f"e{e}.gate"], tensors[f"e{e}.up"], tensors[f"e{e}.down"], np.inf)
    for rows in (90, 20):
        np.testing.assert_allclose(part.forward(gpu(x[:rows], torch.bfloat16), None).sum(dim=0).cpu().numpy(), want[:rows], atol=5e-2, rtol=2e-2)


# -- norm with one number -----------------------------------------------------------------------------------------------
def test_norm_with_one_gain():
    from mini_llm_amd.parts import make_part

    part = make_part("norm", "rmsnorm", width=70, eps=1e-3, one_gain=True, tensor_name="")
    assert part.tensor_specs()[""].shape == ()
    part.bind({"": torch.tensor(0.37).cuda()})
    rng = np.random.default_rng(8)
    x, stream = rng.normal(0, 0.05, (9, 70)), rng.normal(0, 1, (9, 70))
    np.testing.assert_allclose(part.forward(gpu(x), torch.float32).cpu().numpy(), plain.rms_norm(x, 0.37, 1e-3), atol=1e-6, rtol=1e-5)
    np.testing.assert_allclose(part.forward_added(gpu(stream), gpu(x)).cpu().numpy(), stream + plain.rms_norm(x, 0.37, 1e-3), atol=1e-6, rtol=1e-5)
