"""The Goletar configuration, its registry entry, the tensors, cache groups and state its model declares, and the plain implementation's
own mechanisms against each other (no GPU)."""

import copy

import numpy as np
import pytest

import plain_goletar as plain
from goletar_cases import CASES, latent, mingru, model
from mini_llm_amd.config import ConfigError, GoletarConfig, config_from_dict
from mini_llm_amd.engine.loading import build_model
from mini_llm_amd.models.base import EMBEDDING_STATE


@pytest.mark.parametrize("name", list(CASES))
def test_round_trip_tensor_names_cache_and_state(name):
    raw = CASES[name]
    config = config_from_dict(raw)
    assert isinstance(config, GoletarConfig) and config_from_dict(config.to_dict()) == config
    built = build_model(config, "float32")
    assert {n: tuple(s.shape) for n, s in built.named_tensor_specs().items()} == plain.tensor_shapes(raw)
    # one row of pages a token for every latent layer, a state vector for every recurrent one, and the embedding's previous token
    kinds = [entry["type"] for entry in raw["layers"]]
    groups = built.cache_groups()
    assert sorted(i for group in groups for i in group.layers) == [i for i, kind in enumerate(kinds) if kind == "latent_attention"]
    for group in groups:
        assert (group.planes, group.n_kv_heads, group.window) == (1, 1, None)
        for i in group.layers:
            assert group.head_size >= raw["layers"][i]["mixer"]["kv_rank"] + raw["layers"][i]["mixer"]["rot_dim"]
    state = built.state_needs()
    assert set(state) == {i for i, kind in enumerate(kinds) if kind == "mingru"} | {EMBEDDING_STATE}
    assert all(state[i].shape == (raw["layers"][i]["mixer"]["width"],) for i in state if i != EMBEDDING_STATE) and state[EMBEDDING_STATE].shape == ()
    assert built.all_graph_safe() and built.max_positions() is None
    assert all(a._following is b.norm_1 for a, b in zip(built.blocks, built.blocks[1:])) and built.blocks[-1]._following is None


def test_what_the_configuration_refuses():
    def broken(change, match):
        bad = copy.deepcopy(CASES["mixed"])
        change(bad)
        with pytest.raises(ConfigError, match=match):
            config_from_dict(bad)

    broken(lambda c: c["layers"][0].update(type="convolution"), "unknown type")
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10), "rot.dims")
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "rot.dims")
    broken(lambda c: c["layers"][0]["mixer"].pop("scale"), "scale")
    broken(lambda c: c["layers"][0]["mixer"].update(kv_rank=513), "latent")
    broken(lambda c: c["layers"][1]["mixer"].update(width=0), "width")
    broken(lambda c: c["layers"][1]["mlp"].update(kind="dense"), "mlp.kind")
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=6), "picked")
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(experts=1025, top=1), "router kernel")
    broken(lambda c: c["layers"][1]["mlp"]["expert"].update(limit=0.0), "limit")
    broken(lambda c: c["embedding"]["bigram"].pop("buckets"), "buckets")
    broken(lambda c: c["embedding"]["bigram"].update(mul_prev=-1), "mul_prev")
    broken(lambda c: c["embedding"]["bigram"].update(mul_cur=2**31), "bigram")
    broken(lambda c: c["embedding"].pop("bigram"), "bigram")
    broken(lambda c: c["norm"].update(eps=0.0), "eps")
    broken(lambda c: c.update(layers=[]), "layers")


def test_a_layer_without_a_feed_forward_has_no_second_pair_of_norms():
    names = set(build_model(config_from_dict(model([mingru(mlp=None), latent()])), "float32").named_tensor_specs())
    assert "l0.norm2" not in names and "l0.norm2b" not in names and "l0.norm1b" in names and "l1.norm2b" in names


# -- the plain implementation against itself -----------------------------------------------------------------------------
def test_plain_scan_in_portions_and_its_candidate():
    rng = np.random.default_rng(0)
    z, c = rng.uniform(0, 1, (30, 5)), rng.uniform(0, 2, (30, 5))
    whole, last = plain.gated_scan(z, c, np.zeros(5))
    state, pieces = np.zeros(5), []
    for lo, hi in ((0, 1), (1, 3), (3, 17), (17, 30)):
        out, state = plain.gated_scan(z[lo:hi], c[lo:hi], state)
        pieces.append(out)
    np.testing.assert_allclose(np.concatenate(pieces), whole, atol=1e-15)
    np.testing.assert_allclose(state, last)
    u = np.array([-3.0, -1e-9, 0.0, 1e-9, 2.0])
    np.testing.assert_allclose(plain.recurrence_candidate(u), [1 / (1 + np.exp(3.0)), 0.5, 0.5, 0.5, 2.5], atol=1e-8)


def test_plain_rotation_depends_on_the_distance_alone():
    rng = np.random.default_rng(1)
    q, k = rng.normal(size=(1, 8)), rng.normal(size=(1, 8))
    scores = [float((plain.rotate_neighbours(q, [p + 5], 8, 100.0) * plain.rotate_neighbours(k, [p], 8, 100.0)).sum()) for p in (0, 7, 1000)]
    np.testing.assert_allclose(scores, scores[0], atol=1e-9)


def test_plain_pairs_rows_and_the_sink():
    table = {"buckets": 10, "mul_prev": 3, "mul_cur": 7}
    assert plain.bigram_rows([4, 5, 6], table).tolist() == [10, (12 + 35) % 10, (15 + 42) % 10]
    assert plain.bigram_rows([6], table, previous=5).tolist() == [(15 + 42) % 10]
    # a sink as large as the one score there is takes half of the first row's weight
    out = plain.sink_softmax_sum(np.zeros((2, 2)), 0.0, np.array([[3.0], [6.0]]))
    np.testing.assert_allclose(out, [[1.5], [3.0]])


def test_plain_experts_weigh_their_input():
    rng = np.random.default_rng(2)
    mlp = {"kind": "moe", "expert": {"ff": 8, "limit": 0.5}, "router": {"experts": 4, "top": 2}}
    tensors = {"router": rng.normal(size=(4, 6))}
    for e in range(4):
        tensors.update({f"e{e}.gate": rng.normal(size=(8, 6)), f"e{e}.up": rng.normal(size=(8, 6)), f"e{e}.down": rng.normal(size=(6, 8))})
    h = rng.normal(size=(5, 6))
    weights = plain.route(h @ tensors["router"].T, 2)
    assert ((weights > 0).sum(axis=1) == 2).all()
    want = np.zeros_like(h)
    for t in range(5):
        for e in range(4):
            if weights[t, e]:
                row = weights[t, e] * h[t]
                g, u = np.minimum(tensors[f"e{e}.gate"] @ row, 0.5), np.clip(tensors[f"e{e}.up"] @ row, -0.5, 0.5)
                want[t] += tensors[f"e{e}.down"] @ (g / (1 + np.exp(-1.702 * g)) * (u + 1))
    np.testing.assert_allclose(plain.routed_feed_forward(h, mlp, tensors, ""), want, atol=1e-12)
