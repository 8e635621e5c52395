"""The Gevulorn configuration, its registry entry, the tensors, cache groups, state and schedule its model declares, the pages its cache
keeps and gives back, and the plain implementation's own mechanisms against each other (no GPU)."""

import copy

import numpy as np
import pytest

import plain_gevulorn as plain
from gevulorn_cases import CASES, chunked, dense, gla, model, moe, window
from mini_llm_amd.cache import CacheManager, NO_PAGE, first_needed_block
from mini_llm_amd.config import ConfigError, GevulornConfig, config_from_dict
from mini_llm_amd.engine.loading import build_model
from mini_llm_amd.models.base import CacheGroupSpec
from mini_llm_amd.parts import KVNeed


@pytest.mark.parametrize("name", list(CASES))
def test_round_trip_tensor_names_schedule_cache_and_state(name):
    raw = CASES[name]
    config = config_from_dict(raw)
    assert isinstance(config, GevulornConfig) and config_from_dict(config.to_dict()) == config
    built = build_model(config, "float32")
    assert {n: tuple(s.shape) for n, s in built.named_tensor_specs().items()} == plain.tensor_shapes(raw, decay_rank=16)
    runs = plain.layer_runs(raw)
    assert [(call.block, call.step) for call in built.schedule] == runs and [call.cache for call in built.schedule] == list(range(len(runs)))
    kinds = [raw["layers"][block]["type"] for block, _ in runs]
    groups = built.cache_groups()
    assert sorted(i for group in groups for i in group.layers) == [i for i, kind in enumerate(kinds) if kind != "gla"]
    for group in groups:
        for i in group.layers:
            mixer = raw["layers"][runs[i][0]]["mixer"]
            mask = mixer.get("mask") or {}
            windowed = kinds[i] == "attention"
            assert group.n_kv_heads == mixer["kv_heads"] and group.head_size >= max(mixer["dim"], mixer["vdim"])
            assert group.window == (mask.get("size") if windowed else None) and group.chunk == (None if windowed else mask.get("size"))
            assert group.keep_first == (mask.get("keep_first", 0) if windowed else 0)
    state = built.state_needs()
    assert set(state) == {i for i, kind in enumerate(kinds) if kind == "gla"}
    for i, need in state.items():
        mixer = raw["layers"][runs[i][0]]["mixer"]
        assert need.shape == (mixer["heads"] * mixer["dim"] * mixer["vdim"],)
    assert built.all_graph_safe() and built.max_positions() is None


def test_what_the_configuration_refuses():
    def broken(change, match):
        bad = copy.deepcopy(CASES["mixed"])
        change(bad)
        with pytest.raises(ConfigError, match=match):
            config_from_dict(bad)

    broken(lambda c: c["layers"][0].update(type="convolution"), "unknown type")
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "rot.dims")
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "rot.dims|even")
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(scaling={"factor": 2.0, "low": 1.0, "high": 4.0, "original": 64}), "stretches")
    broken(lambda c: c["layers"][0]["mixer"].pop("scale"), "scale")
    broken(lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "divide")
    broken(lambda c: c["layers"][0]["mixer"].update(vdim=257), "wider")
    broken(lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size")
    broken(lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=-1), "keep_first")
    broken(lambda c: c["layers"][1]["mixer"].update(tau=0.0), "tau")
    broken(lambda c: c["layers"][1]["mixer"].update(dim=5000), "larger")
    broken(lambda c: c["layers"][2]["mixer"].update(softcap=-1.0), "softcap")
    broken(lambda c: c["layers"][2]["mlp"].update(kind="sparse"), "mlp.kind")
    broken(lambda c: c["layers"][2]["mlp"]["router"].update(top=6), "picked")
    broken(lambda c: c["layers"][2]["mlp"]["router"].update(experts=1024), "router kernel")
    broken(lambda c: c["layers"][2]["mlp"]["shared"].update(ff=0), "ff")
    broken(lambda c: c["loop"].update(stop=9), "loop")
    broken(lambda c: c["loop"].update(start=3), "loop")
    broken(lambda c: c["loop"].update(times=0), "times")
    broken(lambda c: c.update(logit_softcap=0.0), "logit_softcap")
    broken(lambda c: c["norm"].update(eps=0.0), "eps")
    broken(lambda c: c.update(layers=[]), "layers")


def test_what_config_json_leaves_out_is_off():
    raw = model([window(size=None), chunked(size=None, softcap=None, scaling=None)], softcap=None)
    del raw["embedding"]
    config = config_from_dict(raw)
    assert config.embedding_scale == 1.0 and config.loop is None and config.logit_softcap is None
    assert config.layers[0].mixer.window is None and config.layers[1].mixer.chunk is None and config.layers[1].mixer.softcap is None
    built = build_model(config, "float32")
    names = set(built.named_tensor_specs())
    assert "loop.step" not in names and "l0.norm2" not in names and "l0.mlp.up" not in names
    # a second norm that nobody reads may stand in a file; one that a layer needs may not be passed over
    assert built.canonical_tensor_name("l0.norm2") is None and built.canonical_tensor_name("l1.norm2.b") is None
    assert build_model(config_from_dict(model([gla(mlp=dense())])), "float32").canonical_tensor_name("l0.norm2") == "l0.norm2"


def test_the_decay_matrices_rank_comes_with_the_tensors():
    from mini_llm_amd.weights.loader import WeightsError, check_names

    built = build_model(config_from_dict(model([gla(), gla(dim=8)])), "float32")
    specs = built.named_tensor_specs()

    def found(**changes):
        shapes = {name: tuple(int(n) for n in spec.shape) for name, spec in specs.items()}
        shapes.update(changes)
        return {name: (shape, True) for name, shape in shapes.items()}

    same = lambda n: n
    check_names("a file", specs, found(**{"l0.mix.a1": (3, 64), "l0.mix.a2": (32, 3)}), same)       # each layer its own rank
    check_names("a file", specs, found(**{"l1.mix.a1": (99, 64), "l1.mix.a2": (16, 99)}), same)
    for bad in ({"l0.mix.a1": (3, 64)}, {"l0.mix.a1": (3, 64), "l0.mix.a2": (32, 4)}, {"l0.mix.a1": (0, 64), "l0.mix.a2": (32, 0)}, {"l0.mix.a1": (16, 63)}):
        with pytest.raises(WeightsError, match="a1|a2"):
            check_names("a file", specs, found(**bad), same)


# -- pages ----------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("keep_first,win,page_size", [(5, 10, 4), (4, 1, 4), (8, 7, 4), (9, 20, 8), (100, 3, 4), (0, 6, 4)])
def test_pages_between_the_kept_first_keys_and_the_window_come_back(keep_first, win, page_size):
    group = CacheGroupSpec("g", (0,), 1, 16, win, keep_first=keep_first)
    cache = CacheManager([group], {}, num_pages=60, page_size=page_size, max_requests=2)
    cache.open("a")
    length = 0
    for n in (1, 3, 12, 1, 1, 7, 30, 1, 2, 20):
        cache.reserve("a", n)
        cache.commit("a", n)
        cache.check_invariants()
        length += n
        table = cache.block_table("a", 0)
        # exactly the pages are held that hold a key the next query (or a later one) can see
        needed = {p // page_size for p in range(length) if p < keep_first or p >= length - win + 1}
        assert {b for b, page in enumerate(table) if page != NO_PAGE} == needed | {b for b in range(len(table)) if b >= max(0, length - win + 1) // page_size}
    cache.close("a")
    assert cache.free_pages() == [60]


@pytest.mark.parametrize("chunk,page_size", [(10, 4), (4, 4), (1, 4), (33, 8), (64, 16)])
def test_pages_of_earlier_chunks_come_back(chunk, page_size):
    cache = CacheManager([CacheGroupSpec("g", (0,), 1, 16, None, chunk=chunk)], {}, num_pages=60, page_size=page_size, max_requests=2)
    cache.open("a")
    length = 0
    for n in (1, 3, 12, 1, 1, 7, 30, 1, 2, 20):
        cache.reserve("a", n)
        cache.commit("a", n)
        cache.check_invariants()
        length += n
        first = length // chunk * chunk // page_size      # the next query's chunk
        assert [b for b, page in enumerate(cache.block_table("a", 0)) if page != NO_PAGE] == list(range(first, -(-length // page_size)))
        assert first == first_needed_block(length, None, page_size, chunk)


def test_keys_bounded_in_two_ways_are_refused():
    for bad in (dict(window=4, chunk=4), dict(chunk=0), dict(keep_first=3), dict(window=4, keep_first=-1)):
        with pytest.raises(ValueError, match="bounded|kept"):
            KVNeed(1, 16, **bad)


# -- the plain implementation against itself --------------------------------------------------------------------------------
def test_plain_memory_in_portions_and_unrolled():
    rng = np.random.default_rng(0)
    T, H, dim, vdim = 20, 2, 5, 3
    q, k, v = rng.normal(size=(T, H, dim)), rng.normal(size=(T, H, dim)), rng.normal(size=(T, H, vdim))
    alpha = plain.decays(rng.normal(0, 3, (T, H, dim)), 4.0)
    out, last = plain.decayed_memory(q, k, v, alpha)
    state, pieces = None, []
    for lo, hi in ((0, 1), (1, 4), (4, 20)):
        o, state = plain.decayed_memory(q[lo:hi], k[lo:hi], v[lo:hi], alpha[lo:hi], state)
        pieces.append(o)
    np.testing.assert_allclose(np.concatenate(pieces), out, atol=1e-12)
    np.testing.assert_allclose(state, last, atol=1e-12)
    for t in (0, 7, 19):   # as attention whose weights fade channel by channel
        want = np.zeros((H, vdim))
        for s in range(t + 1):
            fade = np.prod(alpha[s + 1 : t + 1], axis=0)
            want += np.einsum("hi,hi,hi->h", q[t], k[s], fade)[:, None] * v[s]
        np.testing.assert_allclose(out[t], want, atol=1e-10)


def test_plain_decays():
    z = np.array([-50.0, -1.0, 0.0, 3.0, 60.0])
    np.testing.assert_allclose(plain.decays(z, 1.0), 1 / (1 + np.exp(-z)), rtol=1e-12)
    np.testing.assert_allclose(plain.decays(z, 16.0), (1 / (1 + np.exp(-z))) ** (1 / 16.0), rtol=1e-12)


def test_plain_masks():
    seen = plain.window_mask(12, 3, 2)
    assert [j for j in range(12) if seen[9, j]] == [0, 1, 7, 8, 9] and [j for j in range(12) if seen[1, j]] == [0, 1] and [j for j in range(12) if seen[3, j]] == [0, 1, 2, 3]
    assert plain.window_mask(12, 3, 0)[9].sum() == 3 and plain.window_mask(12, 1, 0)[9].sum() == 1 and plain.window_mask(12, None)[9].sum() == 10
    inside = plain.chunk_mask(12, 5)
    assert [j for j in range(12) if inside[9, j]] == [5, 6, 7, 8, 9] and [j for j in range(12) if inside[10, j]] == [10]


def test_plain_rotation_keeps_sizes_and_goes_by_distance():
    rng = np.random.default_rng(1)
    q, k = rng.normal(size=(1, 1, 10)), rng.normal(size=(1, 1, 10))
    turn = lambda x, p: plain.rotate_halves(x, [p], 8, 100.0, {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 32})
    scores = [float((turn(q, p + 5) * turn(k, p)).sum()) for p in (0, 7, 1000)]
    np.testing.assert_allclose(scores, scores[0], atol=1e-9)
    # dividing by the root mean square before or after a rotation is the same thing
    np.testing.assert_allclose(turn(plain.rms_norm(q, 1e-3), 9), plain.rms_norm(turn(q, 9), 1e-3), atol=1e-12)
    assert (turn(q, 3)[..., 8:] == q[..., 8:]).all() and not np.allclose(turn(q, 3)[..., 0], q[..., 0])


def test_plain_frequencies_by_their_wavelength():
    from mini_llm_amd.parts import RotaryEncoding

    for scaling in ({"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64}, {"factor": 3.0, "low": 2.0, "high": 16.0, "original": 4096}):
        want = plain.pair_frequencies(32, 5000.0, scaling)
        np.testing.assert_allclose(RotaryEncoding(32, 5000.0, {"kind": "wavelength", **scaling}, pairing="half").values, want, rtol=1e-13)
        plain_f = plain.pair_frequencies(32, 5000.0)
        assert want[0] == plain_f[0] and np.isclose(want[-1], plain_f[-1] / scaling["factor"]) and (want <= plain_f + 1e-18).all()


def test_plain_sink_and_cap():
    q, k, v = np.zeros((2, 1, 4)), np.zeros((2, 1, 4)), np.array([[[3.0]], [[6.0]]])
    mask = plain.window_mask(2, None)
    np.testing.assert_allclose(plain.sink_attention(q, k, v, 1.0, mask, np.array([0.0]))[:, 0, 0], [1.5, 3.0])   # a sink as large as one score
    hot = np.full((1, 1, 4), 100.0)
    one = plain.sink_attention(hot, hot, np.ones((1, 1, 1)), 1.0, plain.window_mask(1, None), np.array([0.0]), cap=2.0)
    np.testing.assert_allclose(one, 1.0 / (1.0 + np.exp(-2.0)), atol=1e-9)   # the score capped at 2, the sink not


def test_plain_experts_and_their_router():
    rng = np.random.default_rng(2)
    mlp = moe(experts=4, top=2, ff=8, shared=5)
    tensors = {"router": rng.normal(size=(4, 6)), "shared.gate": rng.normal(size=(5, 6)), "shared.up": rng.normal(size=(5, 6)), "shared.down": rng.normal(size=(6, 5))}
    for e in range(4):
        tensors.update({f"e{e}.gate": rng.normal(size=(8, 6)), f"e{e}.up": rng.normal(size=(8, 6)), f"e{e}.down": rng.normal(size=(6, 8))})
    h = rng.normal(size=(5, 6))
    weights = plain.route(h @ tensors["router"].T, 2)
    np.testing.assert_allclose(weights.sum(axis=1), 1.0)
    assert ((weights > 0).sum(axis=1) == 2).all()
    silu = lambda z: z / (1 + np.exp(-z))
    want = (silu(h @ tensors["shared.gate"].T) * (h @ tensors["shared.up"].T)) @ tensors["shared.down"].T
    for e in range(4):
        want += weights[:, e, None] * ((silu(h @ tensors[f"e{e}.gate"].T) * (h @ tensors[f"e{e}.up"].T)) @ tensors[f"e{e}.down"].T)
    np.testing.assert_allclose(plain.routed_feed_forward(h, mlp, tensors, ""), want, atol=1e-12)


def test_plain_layer_runs_of_a_loop():
    layers = [gla()] * 4
    assert plain.layer_runs(model(layers, loop=(1, 3, 2))) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert plain.layer_runs(model(layers, loop=(0, 4, 1))) == [(0, 0), (1, None), (2, None), (3, None)]
    assert plain.layer_runs(model(layers)) == [(i, None) for i in range(4)]
