"""The Gevulorn design through the framework: replayed traces (whole prompts, decoding, portions, mixed batches with pages and slots used
again) against the plain implementation, generation through the entry point and the scheduler, and weights made so that a far key, a key
at a window's, a chunk's or a page's edge, a sink, a lost state or a pass's vector shows in the logits."""

import copy
import json
import subprocess
import sys

import numpy as np
import pytest

import plain_gevulorn as plain
import plain_gpt2
import replay
from conftest import random_tokens
from gevulorn_cases import CASES, chunked, dense, gla, model, moe, window

pytestmark = pytest.mark.gpu


def settle_routers(config, weights, seed=1):
    """Routers without a close call, for bfloat16 runs: every token has a level of its own in as many columns of the stream as there are experts
    at most, evenly spaced and in a random order, which nothing else writes to and no norm weighs; router output e reads column e. The picks
    and their weights then differ from token to token, but no rounding of the router's input changes one."""
    most = max((entry["mlp"]["router"]["experts"] for entry in config["layers"] if entry["mlp"] and entry["mlp"]["kind"] == "moe"), default=0)
    rng = np.random.default_rng(seed)
    levels = np.linspace(-2.5, 2.5, most) if most > 1 else np.full(most, 0.5)
    if most:
        weights["embed"][:, :most] = np.stack([rng.permutation(levels) for _ in range(config["vocab"])]) / config["embedding"]["scale"]
    if "loop.step" in weights:
        weights["loop.step"][:, :most] = 0.0
    for name, value in weights.items():
        if name.endswith((".mix.o", ".mix.o.b", ".down")):
            value[:most] = 0.0
        elif name.endswith(".norm2"):
            value[:most] = 1.0
        elif name.endswith(".norm2.b"):
            value[:most] = 0.0
        elif name.endswith(".router"):
            value[:] = 0.0
            value[np.arange(value.shape[0]), np.arange(value.shape[0])] = 2.0
    return {name: plain_gpt2.round_to_bf16(np.asarray(value, dtype=np.float32)) for name, value in weights.items()}


@pytest.fixture(scope="module")
def gevulorn_dirs(tmp_path_factory):
    out = {}
    for seed, (name, config) in enumerate(CASES.items()):
        rank = (6, 1, 19, 16, 33, 4)[seed % 6]
        weights = plain.random_weights(config, 80 + seed, decay_rank=rank)
        folder = plain.write_model_dir(tmp_path_factory.mktemp(f"gevulorn_{name}"), config, weights)
        out[name] = (folder, copy.deepcopy(config), weights)
        weights = settle_routers(config, plain.random_weights(config, 80 + seed, decay_rank=rank))
        folder = plain.write_model_dir(tmp_path_factory.mktemp(f"gevulorn_{name}_settled"), config, weights)
        out[name, "bfloat16"] = (folder, copy.deepcopy(config), weights)
    return out


def requests_for(config, lengths, seed=700):
    return {f"r{i}": random_tokens(seed + i, n, config["vocab"]) for i, n in enumerate(lengths)}


_remembered = {}   # (weights object, request's tokens, rounded) -> logits; the fixture's weights are never changed


def plain_logits(config, weights, requests, bf16, keep=False):
    w, out = plain.as_float64(weights), {}
    for name, tokens in requests.items():
        key = (id(weights), tuple(tokens), bf16)
        if not keep or key not in _remembered:
            rows = plain.forward(config, w, tokens, round_to=plain_gpt2.stored_as_bf16 if bf16 else None)
            if not keep:
                out[name] = rows
                continue
            _remembered[key] = rows
        out[name] = _remembered[key]
    return out


LENGTHS = {"mixed": [5, 130, 64, 65, 1, 200, 33], "odd": [67, 2, 130, 31], "wide": [3, 150, 64, 17, 129, 330], "recurrent": [150, 1, 70, 3, 97], "large": [3, 140, 66],
           "attending": [66, 2, 140, 20]}
MODES = {"whole": replay.whole, "tail": replay.prefill_then_decode, "chunked": replay.chunked, "mixed": replay.mixed}
TOLERANCE = {"float32": dict(atol=3e-4, rtol=2e-4)}   # sums in another order than numpy's


def check(got, config, weights, requests, dtype, keep=False):
    """32-bit: every logit of every position within the tolerance (one position in a hundred may be up to five times off: a router whose
    two candidates lie within rounding of each other picks the other one). bfloat16 (weights of ``settle_routers``): the engine rounds at
    other places than the plain implementation does when it rounds what a bfloat16 run stores, so the two are not compared with each other
    but each with exact arithmetic, position by position (root mean square over a position's logits): the engine's distance may be three
    times the plain bfloat16 run's at 98 positions in a hundred, and one and a half times in the median and over all positions together. A
    wrong key, page or slot moves the logits of every position behind it by tens of times the noise."""
    exact = plain_logits(config, weights, requests, False, keep)
    if dtype == "float32":
        atol, rtol = TOLERANCE[dtype]["atol"], TOLERANCE[dtype]["rtol"]
        for name, rows in exact.items():
            assert set(got[name]) == set(range(len(rows))), name
            share = np.array([(np.abs(got[name][p].astype(np.float64) - rows[p]) / (atol + rtol * np.abs(rows[p]))).max() for p in range(len(rows))])
            assert share.max() <= 5.0 and (share > 1.0).sum() <= max(1, len(rows) // 100), f"request {name!r}: position {int(share.argmax())} is {share.max():.2f} times the tolerance off, {(share > 1.0).sum()} positions beyond it"
        return
    rounded = plain_logits(config, weights, requests, True, keep)
    noise, error = [], []
    for name, rows in exact.items():
        assert set(got[name]) == set(range(len(rows))), name
        noise.append(np.sqrt(((rounded[name] - rows) ** 2).mean(axis=1)))
        error.append(np.sqrt(((np.stack([got[name][p] for p in range(len(rows))]).astype(np.float64) - rows) ** 2).mean(axis=1)))
    noise, error = np.concatenate(noise), np.concatenate(error)
    ratio = error / (noise + 0.05 * np.median(noise) + 1e-3)
    assert np.quantile(ratio, 0.98) <= 3.0 and np.median(ratio) <= 1.5, (np.quantile(ratio, 0.98), np.median(ratio), ratio.max(), int(ratio.argmax()))
    assert np.sqrt((error**2).mean()) <= 1.5 * np.sqrt((noise**2).mean()) + 1e-3, "rms error against rms noise"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("mode", list(MODES))
@pytest.mark.parametrize("name", list(CASES))
def test_replay_matches_plain(gevulorn_dirs, tmp_path, name, mode, dtype):
    folder, config, weights = gevulorn_dirs[name if dtype == "float32" else (name, dtype)]
    requests = requests_for(config, LENGTHS[name])
    collector = MODES[mode](requests)
    for page_size in ((None, 16) if mode == "mixed" and dtype == "float32" else (None,)):
        # exactly the pages that are needed: they are used again (16: many pages a request, borders everywhere), and so are the slots
        outputs = replay.run_trace(folder, dtype, collector.steps, tmp_path / f"out{page_size}", replay.peak_tokens(collector, page_size or 64), page_size=page_size)
        check(collector.gather(outputs), config, weights, requests, dtype, keep=True)


def test_the_runner_in_a_process_of_its_own(gevulorn_dirs, tmp_path):
    folder, config, weights = gevulorn_dirs["mixed"]
    requests = requests_for(config, [70, 3])
    collector = replay.mixed(requests)
    check(collector.gather(replay.run_trace(folder, "float32", collector.steps, tmp_path / "out", 192, own_process=True)), config, weights, requests, "float32")


def test_portions_of_every_small_size(gevulorn_dirs, tmp_path):
    # portions of 1 to 20 tokens, and around the lengths at which kernels change (8 / 9 rows, chunks of 64, tiles of 128)
    folder, config, weights = gevulorn_dirs["mixed"]
    requests = requests_for(config, [330], seed=50)
    collector = replay.chunked(requests, sizes=tuple(range(2, 21)) + (63, 1, 64, 65))
    check(collector.gather(replay.run_trace(folder, "float32", collector.steps, tmp_path / "out", 384)), config, weights, requests, "float32", keep=True)
    for first in (2, 127, 128, 129, 200):
        requests = requests_for(config, [300], seed=51)
        collector = replay.chunked(requests, sizes=(first, 300))
        check(collector.gather(replay.run_trace(folder, "float32", collector.steps, tmp_path / f"out{first}", 320)), config, weights, requests, "float32", keep=True)


def test_replay_hands_out_the_stream_after_every_layer_run(gevulorn_dirs, tmp_path):
    # a looped layer counts each time, and what joins the stream ahead of the next pass is not part of what a layer leaves
    for name in ("mixed", "odd"):
        folder, config, weights = gevulorn_dirs[name]
        requests = requests_for(config, [40, 9])
        collector = replay.chunked(requests, sizes=(7, 2, 16))
        replay.run_trace(folder, "float32", collector.steps, tmp_path / f"out_{name}", replay.peak_tokens(collector), hidden_out=tmp_path / f"hidden_{name}")
        layers = {request: [] for request in requests}
        for request, tokens in requests.items():
            plain.forward(config, plain.as_float64(weights), tokens, streams=layers[request])
        fed = {}
        for step in collector.steps:
            for e in step["entries"]:   # one request a step
                start, n = fed.get(e["id"], 0), len(e["tokens"])
                for index in range(len(plain.layer_runs(config))):
                    rows = np.fromfile(tmp_path / f"hidden_{name}" / f"{step['step']}.{index}.f32", dtype="<f4").reshape(n, config["width"])
                    np.testing.assert_allclose(rows, layers[e["id"]][index][start : start + n], atol=3e-4, rtol=3e-4, err_msg=f"step {step['step']} run {index}")
                fed[e["id"]] = start + n


HOT = 7   # the token every query looks for


def hot_key_model(kind, size, keep_first=0):
    """One layer of attention in which every query looks for HOT's key, which outscores all others by far. Column 0 of the stream is the same
    for every token and column 1 is large for HOT alone; element 12 of every head (behind the turned ones) reads column 0 in the queries and
    column 1 in the keys."""
    layer = (window(heads=2, kv_heads=1, dim=16, vdim=16, dims=4, scale=0.9, size=size, keep_first=keep_first) if kind == "window" else
             chunked(heads=2, kv_heads=1, dim=16, vdim=16, dims=4, scale=0.9, size=size, softcap=20.0))
    config = model([layer], width=64, vocab=50, scale=2.0, softcap=None)
    weights = plain.random_weights(config, 33)
    weights["embed"][:, 0], weights["embed"][:, 1] = 1.5, 0.0
    weights["embed"][HOT, 1] = 3.0
    for name in ("norm1.b", "mix.q.b", "mix.k.b", "mix.v.b"):
        if "l0." + name in weights:
            weights["l0." + name][:] = 0.0
    weights["l0.norm1"][:2] = 1.0
    weights["l0.mix.sink"][:] = -2.0
    for head in range(2):
        weights["l0.mix.q"][head * 16 + 12] = 0.0
        weights["l0.mix.q"][head * 16 + 12, 0] = 6.0
    weights["l0.mix.k"][12] = 0.0
    weights["l0.mix.k"][12, 1] = 6.0
    return config, {name: plain_gpt2.round_to_bf16(np.asarray(value, dtype=np.float32)) for name, value in weights.items()}


HOT_PLACES = {"window": [((30, 9), [(0, 70), (8, 120), (9, 80), (63, 140), (64, 130), (40, 71), (5, 420), (2, 3)]), ((64, 64), [(63, 300), (64, 200), (1, 66)]), ((1, 1), [(0, 9), (1, 9)]),
                         ((200, 0), [(0, 250), (64, 300)])],
              "chunk": [((40, 0), [(0, 70), (39, 90), (40, 90), (79, 130), (119, 121), (2, 3)]), ((64, 0), [(63, 140), (64, 140), (127, 140)]), ((5, 0), [(4, 12), (5, 12)]),
                        ((200, 0), [(199, 260), (200, 420), (20, 190)])]}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind,case", [(kind, case) for kind in HOT_PLACES for case in range(4)])
def test_a_key_at_the_edges_of_windows_chunks_kept_keys_and_pages(tmp_path, kind, case, dtype):
    # HOT appears once; with another token in its place the logits change at exactly the places that see it, by far more than the tolerance. The
    # logits are checked in whole prompts, in token-by-token decoding past the edges, in portions and in mixed batches.
    (size, keep), places = HOT_PLACES[kind][case]
    config, weights = hot_key_model(kind, size, keep)
    folder = plain.write_model_dir(tmp_path / "model", config, weights)
    rng = np.random.default_rng(3)
    requests = {}
    for at, length in places:
        tokens = rng.integers(10, 50, size=length).tolist()
        tokens[at] = HOT
        requests[f"hot{at}"] = tokens
    for mode in MODES:
        collector = replay.prefill_then_decode(requests, tail=60) if mode == "tail" else MODES[mode](requests)
        outputs = replay.run_trace(folder, dtype, collector.steps, tmp_path / mode, replay.peak_tokens(collector))
        check(collector.gather(outputs), config, weights, requests, dtype)
    if dtype == "bfloat16":
        return
    w = plain.as_float64(weights)
    for at, length in places:
        tokens = requests[f"hot{at}"]
        without = list(tokens)
        without[at] = 11
        moved = np.abs(plain.forward(config, w, without) - plain.forward(config, w, tokens)).max(axis=1)
        mask = plain.window_mask(length, size, keep) if kind == "window" else plain.chunk_mask(length, size)
        assert (moved[mask[:, at]] > 100 * TOLERANCE["float32"]["atol"]).all() and moved[~mask[:, at]].max(initial=0.0) < 1e-9, (at, length)


def test_the_sinks_show(tmp_path):
    config = model([window(), chunked()], width=64, vocab=50)
    weights = plain.random_weights(config, 4)
    for index in range(2):
        weights[f"l{index}.mix.sink"][:] = [6.0, -2.0, 3.0, 0.0]
    requests = requests_for(config, [60, 1], seed=4)
    folder = plain.write_model_dir(tmp_path / "model", config, weights)
    collector = replay.chunked(requests)
    check(collector.gather(replay.run_trace(folder, "float32", collector.steps, tmp_path / "out", 128)), config, weights, requests, "float32")
    base = plain.forward(config, plain.as_float64(weights), requests["r0"])
    for index in range(2):
        changed = {**weights, f"l{index}.mix.sink": np.full(4, -30.0)}
        assert np.median(np.abs(plain.forward(config, plain.as_float64(changed), requests["r0"]) - base).max(axis=1)) > 5e-2


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_state_that_hardly_fades(tmp_path, dtype):
    # Decays that all but keep everything, and one token whose row is far larger than the others': what it wrote is still most of the state
    # hundreds of tokens on, over chunks, portions, decoded tokens and the other requests' use of neighbouring slots, in each pass of a loop
    config = model([gla(heads=2, dim=16, vdim=24, tau=16.0)], width=64, vocab=50, loop=(0, 1, 2))
    weights = plain.random_weights(config, 12)
    weights["l0.mix.a2"][:] *= 0.1
    weights["l0.mix.a2.b"][:] = 9.0
    weights["embed"][HOT] *= 4.0
    weights["l0.norm1"][:] *= 0.2   # (all rows' norms alike: HOT's own row differs by its direction)
    weights["l0.norm1"][1], weights["embed"][:, 1] = 4.0, 0.0
    weights["embed"][HOT, 1] = 3.0
    weights = {name: plain_gpt2.round_to_bf16(np.asarray(value, dtype=np.float32)) for name, value in weights.items()}
    folder = plain.write_model_dir(tmp_path / "model", config, weights)
    rng = np.random.default_rng(6)
    requests = {}
    for at, length in ((0, 300), (63, 140), (64, 129), (1, 2), (15, 40), (130, 200)):
        tokens = rng.integers(10, 50, size=length).tolist()
        tokens[at] = HOT
        requests[f"hot{at}"] = tokens
    for mode in MODES:
        collector = MODES[mode](requests)
        outputs = replay.run_trace(folder, dtype, collector.steps, tmp_path / mode, replay.peak_tokens(collector))
        check(collector.gather(outputs), config, weights, requests, dtype)
    w = plain.as_float64(weights)
    tokens = requests["hot0"]
    moved = np.abs(plain.forward(config, w, [11] + tokens[1:]) - plain.forward(config, w, tokens)).max(axis=1)
    assert moved[-1] > 1e-2, moved[-1]


def test_every_constant_of_the_design_shows(tmp_path):
    # each number config.json gives moves the logits, and the framework follows
    base_config = CASES["mixed"]
    base = plain.random_weights(base_config, 5)
    requests = requests_for(base_config, [90, 3])
    mixer = lambda c, i: c["layers"][i]["mixer"]
    changes = {
        "base": lambda c: None,
        "eps": lambda c: c["norm"].update(eps=0.3),
        "embedding": lambda c: c["embedding"].update(scale=1.0),
        "softcap": lambda c: c.update(logit_softcap=2.0),
        "loop times": lambda c: c["loop"].update(times=1),
        "loop start": lambda c: c["loop"].update(start=0),
        "loop stop": lambda c: c["loop"].update(stop=2),
        "no loop": lambda c: c.pop("loop"),
        "tau": lambda c: mixer(c, 1).update(tau=1.0),
        "scale": lambda c: mixer(c, 0).update(scale=1.5),
        "rotation": lambda c: mixer(c, 0)["rot"].update(base=3.0),
        "rotated": lambda c: mixer(c, 0)["rot"].update(dims=8),
        "window": lambda c: mixer(c, 0)["mask"].update(size=25),
        "kept": lambda c: mixer(c, 0)["mask"].update(keep_first=6),
        "chunk": lambda c: mixer(c, 2)["mask"].update(size=34),
        "capped scores": lambda c: mixer(c, 2).update(softcap=1.0),
        "factor": lambda c: mixer(c, 2)["rot"]["scaling"].update(factor=2.0),
        "low": lambda c: mixer(c, 2)["rot"]["scaling"].update(low=0.2),
        "high": lambda c: mixer(c, 2)["rot"]["scaling"].update(high=9.0),
        "original": lambda c: mixer(c, 2)["rot"]["scaling"].update(original=20),
        "top": lambda c: c["layers"][1]["mlp"]["router"].update(top=5),
    }
    logits = {}
    for name, change in changes.items():
        changed = copy.deepcopy(base_config)
        change(changed)
        weights = dict(base)
        if "loop" not in changed:
            del weights["loop.step"]
        else:
            weights["loop.step"] = weights["loop.step"][: changed["loop"]["times"]]
        folder = plain.write_model_dir(tmp_path / name, changed, weights)
        collector = replay.whole(requests)
        got = collector.gather(replay.run_trace(folder, "float32", collector.steps, tmp_path / f"out_{name}", 128))
        check(got, changed, weights, requests, "float32")
        logits[name] = got
    for name in changes:
        assert name == "base" or np.abs(logits[name]["r0"][89] - logits["base"]["r0"][89]).max() > 1e-2, name


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "recurrent"])
def test_generation_through_the_engine_and_its_scheduler(gevulorn_dirs, name, dtype):
    from mini_llm_amd.engine.engine import Engine, EngineOptions

    folder, config, weights = gevulorn_dirs[name if dtype == "float32" else (name, dtype)]
    prompts = [random_tokens(9, 5, config["vocab"]), random_tokens(10, 70, config["vocab"]), [3], random_tokens(11, 31, config["vocab"]), random_tokens(13, 66, config["vocab"])]
    # few pages: the requests do not all fit at once, so pages and slots are given back and used again
    with Engine(folder, EngineOptions(dtype=dtype, max_sessions=4, max_length=256, max_tokens=256)) as engine:
        generated = engine.generate(prompts, max_new_tokens=24)
        with engine.open_session() as session:
            first = session.prefill(prompts[1])
    w = plain.as_float64(weights)
    rnd = plain_gpt2.stored_as_bf16 if dtype == "bfloat16" else None
    for prompt, new in zip(prompts, generated):
        assert len(new) == 24
        logits = plain.forward(config, w, list(prompt) + list(new), round_to=rnd)
        for k, token in enumerate(new):   # greedy: the plain implementation's own choice, unless the two lie within rounding
            row = logits[len(prompt) - 1 + k]
            assert row[token] >= row.max() - (2e-4 if dtype == "float32" else 0.5), (prompt[:3], k, token, int(row.argmax()))
    want = plain.forward(config, w, prompts[1])[-1]
    if dtype == "float32":
        np.testing.assert_allclose(first, want, **TOLERANCE["float32"])
    else:
        assert want[int(np.argmax(first))] >= want.max() - 1.0


def test_the_command_line_completes_greedily(gevulorn_dirs):
    folder, config, weights = gevulorn_dirs["odd"]
    prompt = random_tokens(12, 9, config["vocab"])
    done = subprocess.run([sys.executable, str(replay.ROOT / "bin" / "complete"), "--model", str(folder), "--dtype", "float32", "--temperature", "0",
                           "--max-new-tokens", "12", "--max-length", "128", "--tokens", ",".join(map(str, prompt))], capture_output=True, text=True, timeout=300)
    assert done.returncode == 0, done.stderr[-2000:]
    new = [int(t) for t in done.stdout.strip().split(",")]
    logits = plain.forward(config, plain.as_float64(weights), prompt + new)
    assert len(new) == 12
    for k, token in enumerate(new):
        row = logits[len(prompt) - 1 + k]
        assert row[token] >= row.max() - 2e-4, (k, token, int(row.argmax()))


def test_long_decoding_from_captured_steps(gevulorn_dirs):
    # 400 decoded tokens, one by one, from captured steps whose tokens never leave the device: past six pages, windows and chunks that give
    # their pages back on the way, and states moved on 400 times
    from mini_llm_amd.engine.engine import Engine, EngineOptions

    folder, config, weights = gevulorn_dirs["wide"]
    prompt = random_tokens(4, 3, config["vocab"])
    with Engine(folder, EngineOptions(dtype="float32", max_sessions=2, max_length=512, max_tokens=1024)) as engine:
        new = engine.generate([prompt], max_new_tokens=400)[0]
    assert len(new) == 400
    logits = plain.forward(config, plain.as_float64(weights), prompt + new)
    wrong = [k for k, token in enumerate(new) if logits[len(prompt) - 1 + k][token] < logits[len(prompt) - 1 + k].max() - 5e-4]
    assert not wrong, wrong[:5]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_captured_steps_match_eager_ones_over_many_replays(gevulorn_dirs, dtype):
    # the same batches, decode steps and steps with portions, from captured graphs (replayed with eager steps between them) and run eagerly
    from mini_llm_amd.engine import StepEntry
    from mini_llm_amd.engine.engine import Engine, EngineOptions

    folder, config, _ = gevulorn_dirs["mixed" if dtype == "float32" else ("mixed", dtype)]
    rng = np.random.default_rng(1)
    logits = {}
    plan = []
    for turn in range(14):
        plan.append([(name, rng.integers(0, config["vocab"], n).tolist()) for name, n in (("a", 1), ("b", 3 if turn % 2 else 1), ("c", 20 if turn % 2 else 1))])
    for graphs in (True, False):
        with Engine(folder, EngineOptions(dtype=dtype, max_sessions=4, max_length=512, max_tokens=2048)) as engine:
            if not graphs:
                engine.runner.use_graphs = False
            handles = {name: engine.try_take_cache() for name in "abc"}
            rows = []
            for step in plan:
                out = engine.runner.step([StepEntry(handles[name], tokens, [len(tokens) - 1]) for name, tokens in step])
                rows.append(out.float().cpu().numpy().copy())
            logits[graphs] = np.stack(rows)
            if graphs:
                assert engine.runner.graph_steps > 4 and engine.runner.portion_graph_steps > 2
    bound = dict(atol=2e-5, rtol=1e-5) if dtype == "float32" else dict(atol=0.25, rtol=0.05)
    np.testing.assert_allclose(logits[True], logits[False], **bound)


def test_config_json_round_trip_and_random_weights(tmp_path):
    from mini_llm_amd.config import config_from_dict
    from mini_llm_amd.engine.engine import Engine, EngineOptions
    from mini_llm_amd.weights import write_model_dir

    config = config_from_dict(CASES["mixed"])
    folder = write_model_dir(config, 3, tmp_path / "random")
    plain_config = json.loads((folder / "config.json").read_text())
    assert plain_config["layers"][1]["mlp"]["router"] == {"experts": 6, "top": 2} and plain_config["loop"] == {"start": 1, "stop": 3, "times": 2}
    weights = plain_gpt2.read_safetensors(folder / "model.safetensors")
    assert {name: value.shape for name, value in weights.items()} == plain.tensor_shapes(plain_config, decay_rank=16)
    with Engine(folder, EngineOptions(dtype="float32", max_sessions=2, max_length=64)) as engine:
        got = engine.forward_last([1, 2, 3, 4, 5])
    np.testing.assert_allclose(got, plain.forward(plain_config, plain.as_float64(weights), [1, 2, 3, 4, 5])[-1], atol=3e-4, rtol=3e-4)


def test_a_step_takes_the_kernels_it_is_meant_to(gevulorn_dirs):
    # a decode step of a looped model: one join behind every layer run (it adds the pass's vector and runs both norms of the next run), one
    # more for the embedding's rows, no separate norms but the last
    from mini_llm_amd.engine import StepEntry
    from mini_llm_amd.engine.engine import Engine, EngineOptions
    from mini_llm_amd.ops import kernels

    folder, config, _ = gevulorn_dirs["wide"]
    with Engine(folder, EngineOptions(dtype="bfloat16", max_sessions=2, max_length=256, max_tokens=512)) as engine:
        engine.runner.use_graphs = False
        handle = engine.try_take_cache()
        engine.runner.step([StepEntry(handle, [1, 2, 3], [2])])
        before = kernels.launch_counts()
        engine.runner.step([StepEntry(handle, [4], [0])])
        seen = kernels.launches_since(before)
    runs = [config["layers"][i] for i, _ in plain.layer_runs(config)]
    routed = [layer for layer in runs if layer["mlp"]["kind"] == "moe"]
    attention = [layer for layer in runs if layer["type"] != "gla"]
    assert seen["join_norms"] == len(runs) + 1 and seen["layernorm"] == 1 and "pending_layernorm" not in seen
    assert seen["map_rows"] == len(attention) == seen["attention_decode"] and seen["channel_memory"] == len(runs) - len(attention)
    assert seen["route"] == len(routed) and seen["experts_few"] == 2 * len(routed) and seen["soft_cap"] == 1
    assert "expert_unit" not in seen and "gate_unit" not in seen and "gated_norm" not in seen
