"""A plain, slow implementation of the Goletar design: numpy, float64, whole sequences, no cache, no batching. One function per
mechanism; the framework's parts and kernels are compared with these.

A model is (config, tensors): ``config`` the dictionary that config.json holds, ``tensors`` name -> float64 array. The stream starts
as the token's row plus a row picked by the token and the one before it. A layer norms in front of each branch and behind it: x <- x +
n1b(mixer(n1(x))), x <- x + n2b(ff(n2(x))), every norm with one number as its gain. Logits = head . final_norm(x).

``round_to`` (optional, a function array -> array) is applied where a bfloat16 run stores something in bfloat16: the inputs of
matrix products and what lies in the cache. None: exact arithmetic."""

from __future__ import annotations

import numpy as np

QUICK_SIGMOID = 1.702   # the constant of the experts' activation g * sigmoid(1.702 g)
UP_SHIFT = 1.0          # what joins an expert's clamped up half
CANDIDATE_SHIFT = 0.5   # the candidate of a non-negative sum u is u + 1/2, that of a negative one sigmoid(u)


def _same(x):
    return x


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def product(x, w, rnd=_same, bias=None):
    """Rows of x times W^T (W stored [out, in]), plus a bias."""
    y = rnd(x) @ rnd(w).T
    return y if bias is None else y + bias


def rms_norm(x, gain, eps):
    """x / sqrt(mean(x^2) + eps) * gain; ``gain`` a vector or one number for all coordinates."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * gain


# -- embedding ----------------------------------------------------------------------------------------------------------
def bigram_rows(tokens, bigram: dict, previous: int | None = None):
    """The row of the second table that each token takes: (before * mul_prev + token * mul_cur) mod buckets, the extra last row
    where there is no token before (``previous``: the token in front of the first one given)."""
    out = []
    for token in tokens:
        if previous is None:
            out.append(int(bigram["buckets"]))
        else:
            out.append((int(previous) * int(bigram["mul_prev"]) + int(token) * int(bigram["mul_cur"])) % int(bigram["buckets"]))
        previous = token
    return np.asarray(out, dtype=np.int64)


def embedding(tokens, config: dict, tensors: dict, rnd=_same, previous: int | None = None):
    rows = bigram_rows(tokens, config["embedding"]["bigram"], previous)
    return rnd(tensors["embed"])[np.asarray(tokens, dtype=np.int64)] + rnd(tensors["bigram"])[rows]


# -- latent attention ---------------------------------------------------------------------------------------------------
def pair_frequencies(dims: int, base: float):
    return float(base) ** (-2.0 * np.arange(dims // 2) / max(dims, 1))


def rotate_neighbours(x, positions, dims: int, base: float):
    """x: [tokens, ..., size]. Of the first ``dims`` elements of the last axis, elements 2i and 2i + 1 make a pair (u, v) that becomes
    (u cos a - v sin a, v cos a + u sin a), a = position * base^(-2i/dims); the rest stays."""
    out = x.copy()
    if not dims:
        return out
    angles = np.asarray(positions, dtype=np.float64)[:, None] * pair_frequencies(dims, base)[None, :]
    shape = (x.shape[0],) + (1,) * (x.ndim - 2) + (dims // 2,)
    c, s = np.cos(angles).reshape(shape), np.sin(angles).reshape(shape)
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def latent_of(h, positions, mixer: dict, tensors: dict, prefix: str, eps: float, rnd=_same):
    """What a layer keeps of its input rows: the normed latent [T, kv_rank] and the rotated key part all heads share [T, rot_dim]."""
    rank = int(mixer["kv_rank"])
    both = product(h, tensors[prefix + "dkv"], rnd)
    c = rms_norm(both[:, :rank], tensors[prefix + "dkv.norm"], eps)
    rotated = rotate_neighbours(both[:, rank:], positions, int(mixer["rot"]["dims"]), float(mixer["rot"]["base"]))
    return rnd(c), rnd(rotated)


def sink_softmax_sum(scores, sink: float, values):
    """Row i of the result: sum_j e^(s_ij) v_j / (sum_j e^(s_ij) + e^sink) over the keys j <= i."""
    T = scores.shape[0]
    s = np.where(np.tril(np.ones((T, T), dtype=bool)), scores, -np.inf)
    top = np.maximum(s.max(axis=1, keepdims=True), sink)
    weights = np.exp(s - top)
    return weights @ values / (weights.sum(axis=1, keepdims=True) + np.exp(sink - top))


def latent_mixer(h, positions, mixer: dict, tensors: dict, prefix: str, eps: float, rnd=_same):
    """Every head's keys and values expanded from the shared latent, written out in full; one number per head and row gates the result."""
    H, dim, rot_dim, vdim = (int(mixer[key]) for key in ("heads", "dim", "rot_dim", "vdim"))
    T = h.shape[0]
    c, k_rot = latent_of(h, positions, mixer, tensors, prefix, eps, rnd)
    q = product(h, tensors[prefix + "q"], rnd).reshape(T, H, dim + rot_dim)
    q_rot = rotate_neighbours(q[:, :, dim:], positions, int(mixer["rot"]["dims"]), float(mixer["rot"]["base"]))
    k = product(c, tensors[prefix + "uk"], rnd).reshape(T, H, dim)
    v = product(c, tensors[prefix + "uv"], rnd).reshape(T, H, vdim)
    gates = sigmoid(product(h, tensors[prefix + "g"], rnd))
    out = np.zeros((T, H, vdim))
    for head in range(H):
        scores = (q[:, head, :dim] @ k[:, head].T + q_rot[:, head] @ k_rot.T) * float(mixer["scale"])
        out[:, head] = sink_softmax_sum(scores, float(tensors[prefix + "sink"][head]), v[:, head]) * gates[:, head : head + 1]
    return product(out.reshape(T, H * vdim), tensors[prefix + "o"], rnd)


# -- gated recurrence ---------------------------------------------------------------------------------------------------
def recurrence_candidate(u):
    """u + 1/2 for u >= 0, sigmoid(u) for u < 0: positive, increasing and continuous."""
    return np.where(u >= 0.0, u + CANDIDATE_SHIFT, sigmoid(np.minimum(u, 0.0)))


def gated_scan(update, candidate, state):
    """S_t = (1 - z_t) S_(t-1) + z_t c_t row by row from ``state`` -> (all S_t, the last one)."""
    out = np.zeros_like(update)
    for t in range(update.shape[0]):
        state = (1.0 - update[t]) * state + update[t] * candidate[t]
        out[t] = state
    return out, state


def mingru_mixer(h, mixer: dict, tensors: dict, prefix: str, rnd=_same, state=None):
    """Rows h [T, width] of one sequence -> (rows of the branch, the state behind the last one)."""
    z = sigmoid(product(h, tensors[prefix + "z"], rnd, tensors[prefix + "z.b"]))
    candidate = recurrence_candidate(product(h, tensors[prefix + "x"], rnd, tensors[prefix + "x.b"]))
    states, last = gated_scan(z, candidate, np.zeros(int(mixer["width"])) if state is None else state)
    return product(states * silu(product(h, tensors[prefix + "g"], rnd)), tensors[prefix + "o"], rnd), last


# -- experts ------------------------------------------------------------------------------------------------------------
def clamped_gate_unit(g, u, limit):
    """min(g, limit) * sigmoid(1.702 min(g, limit)) * (clamp(u, -limit, limit) + 1)."""
    g = np.minimum(g, limit)
    u = np.clip(u, -limit, limit)
    return g * sigmoid(QUICK_SIGMOID * g) * (u + UP_SHIFT)


def expert(h, gate, up, down, limit, rnd=_same):
    return product(clamped_gate_unit(product(h, gate, rnd), product(h, up, rnd), limit), down, rnd)


def route(z, top: int):
    """z: [T, E] router logits -> [T, E]: sigmoid(z) for the ``top`` largest of a row, 0 for the rest."""
    s = sigmoid(z)
    weights = np.zeros_like(s)
    for t in range(z.shape[0]):
        chosen = np.argsort(-s[t], kind="stable")[:top]
        weights[t, chosen] = s[t, chosen]
    return weights


def routed_feed_forward(h, mlp: dict, tensors: dict, prefix: str, rnd=_same):
    """The sum of the chosen experts, each on its own multiple of the row: expert(weight * h)."""
    router, limit = mlp["router"], float(mlp["expert"]["limit"])
    weights = route(product(h, tensors[prefix + "router"], rnd), int(router["top"]))
    out = np.zeros_like(h)
    for e in range(int(router["experts"])):
        rows = np.nonzero(weights[:, e])[0]
        if len(rows):
            p = f"{prefix}e{e}."
            out[rows] += expert(weights[rows, e, None] * h[rows], tensors[p + "gate"], tensors[p + "up"], tensors[p + "down"], limit, rnd)
    return out


# -- layer and model ----------------------------------------------------------------------------------------------------
def layer_forward(x, positions, config: dict, tensors: dict, index: int, rnd=_same):
    layer, eps, p = config["layers"][index], float(config["norm"]["eps"]), f"l{index}."
    h = rms_norm(x, tensors[p + "norm1"], eps)
    if layer["type"] == "latent_attention":
        branch = latent_mixer(h, positions, layer["mixer"], tensors, p + "mix.", eps, rnd)
    elif layer["type"] == "mingru":
        branch, _ = mingru_mixer(h, layer["mixer"], tensors, p + "mix.", rnd)
    else:
        raise ValueError(layer["type"])
    x = x + rms_norm(branch, tensors[p + "norm1b"], eps)
    if layer.get("mlp") is None:
        return x
    branch = routed_feed_forward(rms_norm(x, tensors[p + "norm2"], eps), layer["mlp"], tensors, p + "mlp.", rnd)
    return x + rms_norm(branch, tensors[p + "norm2b"], eps)


def forward(config: dict, tensors: dict, tokens, round_to=None, streams: list | None = None):
    """Logits [T, vocab] of one whole sequence; ``streams`` collects the stream after every layer."""
    rnd = round_to or _same
    tokens = np.asarray(tokens)
    positions = np.arange(len(tokens))
    x = embedding(tokens, config, tensors, rnd)
    for index in range(len(config["layers"])):
        x = layer_forward(x, positions, config, tensors, index, rnd)
        if streams is not None:
            streams.append(x.copy())
    return product(rms_norm(x, tensors["final.norm"], float(config["norm"]["eps"])), tensors["head"], rnd)


def tensor_shapes(config: dict) -> dict:
    """name -> shape of every tensor a model of this configuration has."""
    width, vocab = int(config["width"]), int(config["vocab"])
    shapes = {"embed": (vocab, width), "bigram": (int(config["embedding"]["bigram"]["buckets"]) + 1, width), "final.norm": (), "head": (vocab, width)}
    for index, layer in enumerate(config["layers"]):
        p, mixer, mlp = f"l{index}.", layer["mixer"], layer.get("mlp")
        m = p + "mix."
        shapes.update({p + "norm1": (), p + "norm1b": ()})
        if layer["type"] == "latent_attention":
            H, dim, rot_dim, vdim, rank = (int(mixer[key]) for key in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
            shapes.update({m + "q": (H * (dim + rot_dim), width), m + "dkv": (rank + rot_dim, width), m + "dkv.norm": (rank,), m + "uk": (H * dim, rank),
                           m + "uv": (H * vdim, rank), m + "sink": (H,), m + "g": (H, width), m + "o": (width, H * vdim)})
        else:
            S = int(mixer["width"])
            shapes.update({m + "z": (S, width), m + "z.b": (S,), m + "x": (S, width), m + "x.b": (S,), m + "g": (S, width), m + "o": (width, S)})
        if mlp is None:
            continue
        shapes.update({p + "norm2": (), p + "norm2b": (), p + "mlp.router": (int(mlp["router"]["experts"]), width)})
        ff = int(mlp["expert"]["ff"])
        for e in range(int(mlp["router"]["experts"])):
            shapes.update({p + f"mlp.e{e}.gate": (ff, width), p + f"mlp.e{e}.up": (ff, width), p + f"mlp.e{e}.down": (width, ff)})
    return shapes


def greedy(config: dict, tensors: dict, prompt, n_new: int, round_to=None) -> list:
    tokens = list(prompt)
    for _ in range(n_new):
        tokens.append(int(forward(config, tensors, tokens, round_to)[-1].argmax()))
    return tokens[len(prompt):]


# -- random models for the tests ------------------------------------------------------------------------------------------
def random_weights(config: dict, seed: int) -> dict:
    """Weights whose activations stay of order one and whose every mechanism moves the logits: matrices ~ N(0, 1/in) (the router's
    larger, so that its scores differ), gains around one (behind a branch around a half), update gates that mostly keep the state.
    float32 arrays holding bfloat16 values (as files hold them)."""
    import plain_gpt2

    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(config).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1b", "norm2b"):
            value = rng.normal(0.6, 0.1, shape)
        elif last in ("norm", "norm1", "norm2"):
            value = rng.normal(1.0, 0.15, shape)
        elif name.endswith(".z.b"):
            value = rng.normal(-2.0, 1.0, shape)
        elif last == "b":
            value = rng.normal(0.0, 0.4, shape)
        elif last == "sink":
            value = rng.normal(0.5, 1.0, shape)
        elif last in ("embed", "bigram"):
            value = rng.normal(0.0, 0.7, shape)
        elif last == "router":
            value = rng.normal(0.0, 2.0 * shape[1] ** -0.5, shape)
        elif last in ("gate", "up"):   # some units beyond the limit, though the row comes in times a weight below one
            value = rng.normal(0.0, 2.0 * shape[1] ** -0.5, shape)
        else:
            value = rng.normal(0.0, shape[1] ** -0.5, shape)
        out[name] = plain_gpt2.round_to_bf16(np.asarray(value, dtype=np.float32))
    return out


def as_float64(weights: dict) -> dict:
    return {name: np.asarray(value, dtype=np.float64) for name, value in weights.items()}


def write_model_dir(path, config: dict, weights: dict):
    import json
    from pathlib import Path

    import plain_gpt2

    path = Path(path)
    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(config, indent=1))
    plain_gpt2.write_safetensors(path / "model.safetensors", {k: np.asarray(v, dtype=np.float32) for k, v in weights.items()}, bf16=True)
    return path
