"""The Goletar design through the framework: replayed traces (whole prompts, decoding, portions, mixed batches with pages and slots used
again) against the plain implementation, generation through the entry point and the scheduler, and weights made so that a far key, a key
at a page's border, a sink, a lost state or a wrong previous token shows in the logits."""

import copy
import json
import subprocess
import sys

import numpy as np
import pytest

import plain_goletar as plain
import plain_gpt2
import replay
from conftest import random_tokens
from goletar_cases import CASES, latent, mingru, model, moe

pytestmark = pytest.mark.gpu


def sharpen(config, weights, factor=3.0):
    """Random projections give nearly uniform softmaxes, under which a wrong key or page hardly moves a logit: the query matrices are
    scaled up, so that attention weights differ by orders of magnitude."""
    for index, entry in enumerate(config["layers"]):
        if entry["type"] == "latent_attention":
            weights[f"l{index}.mix.q"] = plain_gpt2.round_to_bf16(weights[f"l{index}.mix.q"] * factor)
    return weights


def settle_routers(config, weights, seed=1):
    """Routers without a close call, for bfloat16 runs: every token has a level of its own in as many columns of the stream as there are experts
    at most, evenly spaced and in a random order, which nothing else writes to; router output e reads column e. The picks and their
    weights then differ from token to token, but no rounding of the router's input changes one."""
    most = max(entry["mlp"]["router"]["experts"] for entry in config["layers"] if entry["mlp"] is not None)
    rng = np.random.default_rng(seed)
    levels = np.linspace(-2.0, 2.0, most) if most > 1 else np.array([0.5])
    weights["embed"][:, :most] = np.stack([rng.permutation(levels) for _ in range(config["vocab"])])
    weights["bigram"][:, :most] = 0.0
    for index, entry in enumerate(config["layers"]):
        weights[f"l{index}.mix.o"][:most] = 0.0
        if entry["mlp"] is not None:
            router = weights[f"l{index}.mlp.router"]
            router[:] = 0.0
            for e in range(router.shape[0]):
                router[e, e] = 1.5
                weights[f"l{index}.mlp.e{e}.down"][:most] = 0.0
    return {name: plain_gpt2.round_to_bf16(np.asarray(value, dtype=np.float32)) for name, value in weights.items()}


@pytest.fixture(scope="module")
def goletar_dirs(tmp_path_factory):
    out = {}
    for seed, (name, config) in enumerate(CASES.items()):
        weights = sharpen(config, plain.random_weights(config, 60 + seed))
        folder = plain.write_model_dir(tmp_path_factory.mktemp(f"goletar_{name}"), config, weights)
        out[name] = (folder, copy.deepcopy(config), weights)
        weights = settle_routers(config, sharpen(config, plain.random_weights(config, 60 + seed)))
        folder = plain.write_model_dir(tmp_path_factory.mktemp(f"goletar_{name}_settled"), config, weights)
        out[name, "bfloat16"] = (folder, copy.deepcopy(config), weights)
    return out


def requests_for(config, lengths, seed=700):
    return {f"r{i}": random_tokens(seed + i, n, config["vocab"]) for i, n in enumerate(lengths)}


def plain_logits(config, weights, requests, bf16):
    w = plain.as_float64(weights)
    return {name: plain.forward(config, w, tokens, round_to=plain_gpt2.stored_as_bf16 if bf16 else None) for name, tokens in requests.items()}


LENGTHS = {"mixed": [5, 130, 64, 65, 1, 200, 33], "odd": [67, 2, 130, 31], "wide": [3, 150, 64, 17, 129, 260], "recurrent": [150, 1, 70, 3, 97],
           "large": [3, 140, 66],
           "attending": [66, 2, 140, 20]}
MODES = {"whole": replay.whole, "tail": replay.prefill_then_decode, "chunked": replay.chunked, "mixed": replay.mixed}
TOLERANCE = {"float32": dict(atol=3e-4, rtol=2e-4)}   # sums in another order than numpy's


def check(got, config, weights, requests, dtype):
    """32-bit: every logit of every position within the tolerance (one position in a hundred may be up to five times off: a router whose
    two candidates lie within rounding of each other picks the other one). bfloat16 (weights of ``settle_routers``): the engine rounds at
    other places than the plain implementation does when it rounds what a bfloat16 run stores, so the two are not compared with each other
    but each with exact arithmetic, position by position (root mean square over a position's logits): the engine's distance may be three
    times the plain bfloat16 run's at 98 positions in a hundred, and one and a half times in the median and over all positions together. A
    wrong key, page or slot moves the logits of every position behind it by tens of times the noise."""
    exact = plain_logits(config, weights, requests, False)
    if dtype == "float32":
        atol, rtol = TOLERANCE[dtype]["atol"], TOLERANCE[dtype]["rtol"]
        for name, rows in exact.items():
            assert set(got[name]) == set(range(len(rows))), name
            share = np.array([(np.abs(got[name][p].astype(np.float64) - rows[p]) / (atol + rtol * np.abs(rows[p]))).max() for p in range(len(rows))])
            assert share.max() <= 5.0 and (share > 1.0).sum() <= max(1, len(rows) // 100), f"request {name!r}: position {int(share.argmax())} is {share.max():.2f} times the tolerance off, {(share > 1.0).sum()} positions beyond it"
        return
    rounded = plain_logits(config, weights, requests, True)
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
def test_replay_matches_plain(goletar_dirs, tmp_path, name, mode, dtype):
    folder, config, weights = goletar_dirs[name if dtype == "float32" else (name, dtype)]
    requests = requests_for(config, LENGTHS[name])
    collector = MODES[mode](requests)
    for page_size in ((None, 16) if mode == "mixed" and dtype == "float32" else (None,)):
        # exactly the pages that are needed: they are used again (16: many pages a request, borders everywhere), and so are the slots
        outputs = replay.run_trace(folder, dtype, collector.steps, tmp_path / f"out{page_size}", replay.peak_tokens(collector, page_size or 64), page_size=page_size)
        check(collector.gather(outputs), config, weights, requests, dtype)


def test_portions_of_every_small_size(goletar_dirs, tmp_path):
    # portions of 1 to 20 tokens, and around the lengths at which kernels change (16 / 17 rows, chunks of 64, tiles of 128)
    folder, config, weights = goletar_dirs["mixed"]
    requests = requests_for(config, [330], seed=50)
    sizes = tuple(range(2, 21)) + (63, 1, 64, 65)
    collector = replay.chunked(requests, sizes=sizes)
    check(collector.gather(replay.run_trace(folder, "float32", collector.steps, tmp_path / "out", 384)), config, weights, requests, "float32")
    for first in (2, 127, 128, 129, 200):
        requests = requests_for(config, [300], seed=51)
        collector = replay.chunked(requests, sizes=(first, 300))
        check(collector.gather(replay.run_trace(folder, "float32", collector.steps, tmp_path / f"out{first}", 320)), config, weights, requests, "float32")


def test_replay_hands_out_the_stream_after_every_layer(goletar_dirs, tmp_path):
    folder, config, weights = goletar_dirs["mixed"]
    requests = requests_for(config, [40, 9])
    collector = replay.chunked(requests, sizes=(7, 2, 16))
    replay.run_trace(folder, "float32", collector.steps, tmp_path / "out", replay.peak_tokens(collector), hidden_out=tmp_path / "hidden")
    layers = {name: [] for name in requests}
    for name, tokens in requests.items():
        plain.forward(config, plain.as_float64(weights), tokens, streams=layers[name])
    fed = {}
    for step in collector.steps:
        for e in step["entries"]:   # one request a step
            start, n = fed.get(e["id"], 0), len(e["tokens"])
            for index in range(len(config["layers"])):
                rows = np.fromfile(tmp_path / "hidden" / f"{step['step']}.{index}.f32", dtype="<f4").reshape(n, config["width"])
                np.testing.assert_allclose(rows, layers[e["id"]][index][start : start + n], atol=2e-4, rtol=2e-4, err_msg=f"step {step['step']} layer {index}")
            fed[e["id"]] = start + n


HOT = 7   # the token every query looks for


def hot_key_model():
    config = model([latent(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=24, scale=1.0, mlp=None)], width=64, vocab=50)
    weights = plain.random_weights(config, 33)
    # Column 0 of the stream is the same for every token and column 1 is large for HOT alone; the pairs' table touches neither. Latent
    # element 0 reads column 1; one unrotated element of every head reads column 0 in the queries and latent element 0 in the keys, so the
    # key of HOT outscores every other key for every query that sees it.
    weights["embed"][:, 0], weights["embed"][:, 1] = 2.0, 0.0
    weights["embed"][HOT, 1] = 4.0
    weights["bigram"][:, :2] = 0.0
    weights["l0.mix.dkv"][0] = 0.0
    weights["l0.mix.dkv"][0, 1] = 4.0
    for head in range(2):
        weights["l0.mix.q"][head * 24 + 5] = 0.0
        weights["l0.mix.q"][head * 24 + 5, 0] = 4.0
        weights["l0.mix.uk"][head * 16 + 5] = 0.0
        weights["l0.mix.uk"][head * 16 + 5, 0] = 3.0
    return config, weights


def test_a_far_key_and_keys_at_page_borders_in_prompts_and_in_decoding(tmp_path):
    # HOT appears once, at a sequence's first place, at a page's last and first place, and hundreds of tokens before the places that are
    # asked for; the logits are checked in whole prompts, in token-by-token decoding and in portions. Taking it away moves the logits of
    # every place behind it by far more than the tolerance, and those before it not at all.
    config, weights = hot_key_model()
    rng = np.random.default_rng(3)
    folder = plain.write_model_dir(tmp_path / "model", config, weights)
    requests = {}
    for at, length in ((0, 70), (63, 80), (64, 140), (127, 200), (128, 131), (5, 420), (2, 3)):
        tokens = rng.integers(10, 50, size=length).tolist()
        tokens[at] = HOT
        requests[f"hot{at}"] = tokens
    for dtype in ("float32", "bfloat16"):
        for mode in ("whole", "tail", "chunked"):
            collector = MODES[mode](requests)
            outputs = replay.run_trace(folder, dtype, collector.steps, tmp_path / f"{dtype}{mode}", replay.peak_tokens(collector))
            check(collector.gather(outputs), config, weights, requests, dtype)
    w = plain.as_float64(weights)
    for at in (0, 64, 5):
        tokens = requests[f"hot{at}"]
        without = list(tokens)
        without[at] = 11
        moved = np.abs(plain.forward(config, w, without) - plain.forward(config, w, tokens)).max(axis=1)
        assert moved[-1] > 100 * TOLERANCE["float32"]["atol"] and moved[at + 1 :].min() > 30 * TOLERANCE["float32"]["atol"], (at, moved[-1], moved[at + 1 :].min())
        assert at == 0 or moved[:at].max() < 1e-9, at


def test_the_sink_and_the_heads_gates_show(tmp_path):
    config, weights = hot_key_model()
    weights["l0.mix.sink"][:] = [6.0, -2.0]
    requests = requests_for(config, [30, 1], seed=4)
    folder = plain.write_model_dir(tmp_path / "model", config, weights)
    collector = replay.chunked(requests)
    check(collector.gather(replay.run_trace(folder, "float32", collector.steps, tmp_path / "out", 128)), config, weights, requests, "float32")
    base = plain.forward(config, plain.as_float64(weights), requests["r0"])
    for name, value in (("l0.mix.sink", -30.0), ("l0.mix.g", 0.0)):
        changed = dict(weights)
        changed[name] = np.full_like(weights[name], value)
        assert np.median(np.abs(plain.forward(config, plain.as_float64(changed), requests["r0"]) - base).max(axis=1)) > 2e-2, name


def test_a_state_that_hardly_fades(tmp_path):
    # Update gates that all but close unless column 1 of the stream is large, which it is for HOT alone: what HOT wrote is still most of the
    # state hundreds of tokens on, over chunks, portions, decoded tokens and the other requests' use of neighbouring slots.
    config = model([mingru(width=100, mlp=None)], width=64, vocab=50, buckets=50)
    weights = plain.random_weights(config, 12)
    weights["embed"][:, 1] = 0.0
    weights["embed"][HOT, 1] = 4.0
    weights["bigram"][:, 1] = 0.0
    weights["l0.mix.z"][:, :] *= 0.1
    weights["l0.mix.z"][:, 1] = 4.0
    weights["l0.mix.z.b"][:] = -9.0
    weights = {name: plain_gpt2.round_to_bf16(np.asarray(value, dtype=np.float32)) for name, value in weights.items()}
    folder = plain.write_model_dir(tmp_path / "model", config, weights)
    rng = np.random.default_rng(6)
    requests = {}
    for at, length in ((0, 300), (63, 140), (64, 129), (1, 2), (15, 40), (130, 200)):
        tokens = rng.integers(10, 50, size=length).tolist()
        tokens[at] = HOT
        requests[f"hot{at}"] = tokens
    for dtype in ("float32", "bfloat16"):
        for mode in MODES:
            collector = MODES[mode](requests)
            outputs = replay.run_trace(folder, dtype, collector.steps, tmp_path / f"{dtype}{mode}", replay.peak_tokens(collector))
            check(collector.gather(outputs), config, weights, requests, dtype)
    w = plain.as_float64(weights)
    tokens = requests["hot0"]
    moved = np.abs(plain.forward(config, w, [11] + tokens[1:]) - plain.forward(config, w, tokens)).max(axis=1)
    assert moved[-1] > 1e-2, moved[-1]


def test_the_previous_token_shows_at_every_cut(tmp_path):
    # The row a pair of tokens picks is most of the stream: a portion's first token that forgot the one before it, or took another
    # request's, is far off. Single tokens, pairs and long portions, requests left out of steps, slots used again.
    config = model([mingru(width=32, mlp=None), latent(heads=1, mlp=None)], width=64, vocab=40, buckets=1601, mul_prev=40, mul_cur=1)
    weights = plain.random_weights(config, 2)
    weights["bigram"] = plain_gpt2.round_to_bf16(weights["bigram"] * 6.0)
    folder = plain.write_model_dir(tmp_path / "model", config, weights)
    requests = requests_for(config, [1, 2, 40, 90, 3, 70, 20], seed=9)
    for dtype in ("float32", "bfloat16"):
        for mode in ("chunked", "mixed"):
            collector = MODES[mode](requests)
            outputs = replay.run_trace(folder, dtype, collector.steps, tmp_path / f"{dtype}{mode}", replay.peak_tokens(collector))
            check(collector.gather(outputs), config, weights, requests, dtype)


def test_every_constant_of_the_design_shows(tmp_path):
    # each number config.json gives moves the logits, and the framework follows
    base_config = CASES["mixed"]
    base = plain.random_weights(base_config, 5)
    requests = requests_for(base_config, [20, 3])
    changes = {
        "base": lambda c: None,
        "eps": lambda c: c["norm"].update(eps=0.3),
        "limit": lambda c: c["layers"][0]["mlp"]["expert"].update(limit=0.2),
        "top": lambda c: c["layers"][0]["mlp"]["router"].update(top=5),
        "scale": lambda c: c["layers"][0]["mixer"].update(scale=1.5),
        "rotation": lambda c: c["layers"][3]["mixer"]["rot"].update(base=3.0),
        "mul_prev": lambda c: c["embedding"]["bigram"].update(mul_prev=32),
        "mul_cur": lambda c: c["embedding"]["bigram"].update(mul_cur=11),
    }
    logits = {}
    for name, change in changes.items():
        changed = copy.deepcopy(base_config)
        change(changed)
        folder = plain.write_model_dir(tmp_path / name, changed, base)
        collector = replay.whole(requests)
        got = collector.gather(replay.run_trace(folder, "float32", collector.steps, tmp_path / f"out_{name}", 128))
        check(got, changed, base, requests, "float32")
        logits[name] = got
    for name in changes:
        assert name == "base" or np.abs(logits[name]["r0"][19] - logits["base"]["r0"][19]).max() > 1e-2, name


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "recurrent"])
def test_generation_through_the_engine_and_its_scheduler(goletar_dirs, name, dtype):
    from mini_llm_amd.engine.engine import Engine, EngineOptions

    folder, config, weights = goletar_dirs[name if dtype == "float32" else (name, dtype)]
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
        assert want[int(np.argmax(first))] >= want.max() - 3.0


def test_the_command_line_completes_greedily(goletar_dirs):
    folder, config, weights = goletar_dirs["odd"]
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


def test_long_decoding_from_captured_steps(goletar_dirs):
    # 400 decoded tokens, one by one, from captured steps whose tokens never leave the device: past six pages, every one of them the previous
    # token of the next, and a state moved on 400 times
    from mini_llm_amd.engine.engine import Engine, EngineOptions

    folder, config, weights = goletar_dirs["wide"]
    prompt = random_tokens(4, 3, config["vocab"])
    with Engine(folder, EngineOptions(dtype="float32", max_sessions=2, max_length=512, max_tokens=1024)) as engine:
        new = engine.generate([prompt], max_new_tokens=400)[0]
    assert len(new) == 400
    logits = plain.forward(config, plain.as_float64(weights), prompt + new)
    wrong = [k for k, token in enumerate(new) if logits[len(prompt) - 1 + k][token] < logits[len(prompt) - 1 + k].max() - 5e-4]
    assert not wrong, wrong[:5]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_captured_steps_match_eager_ones_over_many_replays(goletar_dirs, dtype):
    # the same batches, decode steps and steps with portions, from captured graphs (replayed with eager steps between them) and run eagerly
    from mini_llm_amd.engine import StepEntry
    from mini_llm_amd.engine.engine import Engine, EngineOptions

    folder, config, _ = goletar_dirs["mixed" if dtype == "float32" else ("mixed", dtype)]
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
    assert plain_config["layers"][1]["mlp"]["router"] == {"experts": 5, "top": 1} and plain_config["embedding"]["bigram"]["mul_prev"] == 31
    weights = plain_gpt2.read_safetensors(folder / "model.safetensors")
    assert {name: value.shape for name, value in weights.items()} == plain.tensor_shapes(plain_config)
    with Engine(folder, EngineOptions(dtype="float32", max_sessions=2, max_length=64)) as engine:
        got = engine.forward_last([1, 2, 3, 4, 5])
    np.testing.assert_allclose(got, plain.forward(plain_config, plain.as_float64(weights), [1, 2, 3, 4, 5])[-1], atol=3e-4, rtol=3e-4)
