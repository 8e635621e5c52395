"""A plain, slow implementation of the Gevulorn design: numpy, float64, whole sequences, no cache, no batching. One function per
mechanism; the framework's parts and kernels are compared with these.

A model is (config, tensors): ``config`` the dictionary that config.json holds, ``tensors`` name -> float64 array. The stream starts
as a multiple of the token's row. A layer has two layer norms of the same stream, x <- x + mixer(n1(x)) + ff(n2(x)). A run of
neighbouring layers may be gone through several times; each time a vector of its own joins the stream first. Logits = cap
tanh(head . final_norm(x) / cap).

``round_to`` (optional, a function array -> array) is applied where a bfloat16 run stores something in bfloat16: the inputs of
matrix products and what lies in the cache. None: exact arithmetic."""

from __future__ import annotations

import numpy as np


def _same(x):
    return x


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def soft_cap(z, cap):
    """cap tanh(z / cap); None: z itself."""
    return z if cap is None else cap * np.tanh(z / cap)


def product(x, w, rnd=_same, bias=None):
    """Rows of x times W^T (W stored [out, in]), plus a bias."""
    y = rnd(x) @ rnd(w).T
    return y if bias is None else y + bias


# -- norms --------------------------------------------------------------------------------------------------------------
def layer_norm(x, gain, offset, eps):
    centred = x - x.mean(axis=-1, keepdims=True)
    return centred / np.sqrt((centred * centred).mean(axis=-1, keepdims=True) + eps) * gain + offset


def rms_norm(x, eps, gain=1.0):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * gain


# -- rotation -----------------------------------------------------------------------------------------------------------
def pair_frequencies(dims: int, base: float, scaling: dict | None = None):
    """base^(-2i/dims) for every pair i. ``scaling`` {factor, low, high, original} slows pairs by their wavelength: short ones keep their
    frequency, those longer than original / low are ``factor`` times slower, and between the two the frequency is blended."""
    f = float(base) ** (-2.0 * np.arange(dims // 2) / max(dims, 1))
    if not scaling:
        return f
    out = []
    factor, low, high, original = (float(scaling[key]) for key in ("factor", "low", "high", "original"))
    for one in f:
        turns = original * one / (2.0 * np.pi)   # how often the pair turns within the original length
        if turns > high:
            out.append(one)
        elif turns < low:
            out.append(one / factor)
        else:
            share = (turns - low) / (high - low)
            out.append((1.0 - share) * one / factor + share * one)
    return np.array(out)


def rotate_halves(x, positions, dims: int, base: float, scaling: dict | None = None):
    """x: [tokens, heads, size]. Of the first ``dims`` elements of a head, i and i + dims / 2 make a pair (u, v) that becomes (u cos a - v
    sin a, v cos a + u sin a), a = position * the pair's frequency; the rest stays."""
    out = x.copy()
    half = dims // 2
    if not half:
        return out
    angles = np.asarray(positions, dtype=np.float64)[:, None, None] * pair_frequencies(dims, base, scaling)[None, None, :]
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * np.cos(angles) - v * np.sin(angles)
    out[..., half:dims] = v * np.cos(angles) + u * np.sin(angles)
    return out


# -- attention ----------------------------------------------------------------------------------------------------------
def window_mask(n: int, size: int | None, keep_first: int = 0):
    """[n, n]: query i sees key j <= i that is at most size - 1 back or among the first ``keep_first``."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    seen = j <= i
    return seen if size is None else seen & ((i - j < size) | (j < keep_first))


def chunk_mask(n: int, size: int | None):
    """[n, n]: query i sees key j <= i of its own chunk of ``size`` positions."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    return (j <= i) if size is None else (j <= i) & (j // size == i // size)


def sink_attention(q, k, v, scale: float, mask, sinks, cap=None):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]; query head h reads key/value head h // (H / G). exp(sink_h) joins the
    denominator of head h, not scaled and not capped."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = np.where(mask, soft_cap(q[:, h] @ k[:, g].T * scale, cap), -np.inf)
        top = np.maximum(s.max(axis=1, keepdims=True), sinks[h])
        w = np.exp(s - top)
        out[:, h] = w @ v[:, g] / (w.sum(axis=1, keepdims=True) + np.exp(sinks[h] - top))
    return out


def _heads(h, mixer: dict, tensors: dict, prefix: str, rnd, biases: bool):
    T = h.shape[0]
    out = []
    for name, count, size in (("q", mixer["heads"], mixer["dim"]), ("k", mixer["kv_heads"], mixer["dim"]), ("v", mixer["kv_heads"], mixer["vdim"])):
        y = product(h, tensors[prefix + name], rnd, tensors[prefix + name + ".b"] if biases else None)
        out.append(y.reshape(T, int(count), int(size)))
    return out


def unit_attention(h, positions, mixer: dict, tensors: dict, prefix: str, eps: float, rnd=_same):
    """Rotated queries and keys divided by their root mean square, a window that keeps the first tokens, a sink."""
    q, k, v = _heads(h, mixer, tensors, prefix, rnd, biases=False)
    rot = mixer["rot"]
    q, k = (rms_norm(rotate_halves(x, positions, int(rot["dims"]), rot["base"]), eps) for x in (q, k))
    mask = mixer.get("mask") or {}
    seen = window_mask(len(positions), mask.get("size"), int(mask.get("keep_first", 0)))
    mixed = sink_attention(rnd(q), rnd(k), rnd(v), float(mixer["scale"]), seen, tensors[prefix + "sink"])
    return product(mixed.reshape(len(positions), -1), tensors[prefix + "o"], rnd)


def chunk_attention(h, positions, mixer: dict, tensors: dict, prefix: str, eps: float, rnd=_same):
    """Biases on all four projections, normed queries and keys with gains, stretched rotation, capped scores, chunks, a sink."""
    q, k, v = _heads(h, mixer, tensors, prefix, rnd, biases=True)
    rot = mixer["rot"]
    turn = lambda x: rotate_halves(x, positions, int(rot["dims"]), rot["base"], rot.get("scaling"))
    q, k = turn(rms_norm(q, eps, tensors[prefix + "q.norm"])), turn(rms_norm(k, eps, tensors[prefix + "k.norm"]))
    seen = chunk_mask(len(positions), (mixer.get("mask") or {}).get("size"))
    mixed = sink_attention(rnd(q), rnd(k), rnd(v), float(mixer["scale"]), seen, tensors[prefix + "sink"], mixer.get("softcap"))
    return product(mixed.reshape(len(positions), -1), tensors[prefix + "o"], rnd, tensors[prefix + "o.b"])


# -- gated linear attention ---------------------------------------------------------------------------------------------
def decays(z, tau: float):
    """sigmoid(z)^(1 / tau), through its logarithm."""
    return np.exp(log_sigmoid(z) / tau)


def decayed_memory(q, k, v, alpha, state=None):
    """Per head S_t = diag(alpha_t) S_(t-1) + k_t v_t^T and o_t = S_t^T q_t, row by row. q, k, alpha [T, H, dim], v [T, H, vdim] -> (o
    [T, H, vdim], the last S [H, dim, vdim])."""
    T, H, dim = q.shape
    S = np.zeros((H, dim, v.shape[2])) if state is None else state.copy()
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hij,hi->hj", S, q[t])
    return out, S


def gla_mixer(h, mixer: dict, tensors: dict, prefix: str, eps: float, rnd=_same, state=None):
    """Rows h [T, width] of one sequence -> (rows of the branch, the state behind the last one)."""
    T, H, dim, vdim = h.shape[0], int(mixer["heads"]), int(mixer["dim"]), int(mixer["vdim"])
    heads = lambda x, size: x.reshape(T, H, size)
    q = heads(product(h, tensors[prefix + "q"], rnd), dim) * dim ** -0.5
    k, v = heads(product(h, tensors[prefix + "k"], rnd), dim), heads(product(h, tensors[prefix + "v"], rnd), vdim)
    z = product(product(h, tensors[prefix + "a1"], rnd), tensors[prefix + "a2"], _same, tensors[prefix + "a2.b"])
    o, last = decayed_memory(q, k, v, heads(decays(z, float(mixer["tau"])), dim), state)
    mixed = rms_norm(o, eps, tensors[prefix + "norm"]).reshape(T, H * vdim) * silu(product(h, tensors[prefix + "g"], rnd))
    return product(mixed, tensors[prefix + "o"], rnd), last


# -- feed-forward -------------------------------------------------------------------------------------------------------
def squared_relu(z):
    return np.maximum(z, 0.0) ** 2


def dense_feed_forward(h, tensors: dict, prefix: str, rnd=_same):
    return product(squared_relu(product(h, tensors[prefix + "up"], rnd)), tensors[prefix + "down"], rnd)


def expert(h, tensors: dict, prefix: str, rnd=_same):
    return product(silu(product(h, tensors[prefix + "gate"], rnd)) * product(h, tensors[prefix + "up"], rnd), tensors[prefix + "down"], rnd)


def route(z, top: int):
    """z: [T, E] router logits -> [T, E]: the softmax over the ``top`` largest of a row alone, 0 for the rest."""
    weights = np.zeros_like(z)
    for t in range(z.shape[0]):
        chosen = np.argsort(-z[t], kind="stable")[:top]
        w = np.exp(z[t, chosen] - z[t, chosen].max())
        weights[t, chosen] = w / w.sum()
    return weights


def routed_feed_forward(h, mlp: dict, tensors: dict, prefix: str, rnd=_same):
    weights = route(product(h, tensors[prefix + "router"], rnd), int(mlp["router"]["top"]))
    out = np.zeros_like(h)
    for e in range(int(mlp["router"]["experts"])):
        rows = np.nonzero(weights[:, e])[0]
        if len(rows):
            out[rows] += weights[rows, e, None] * expert(h[rows], tensors, f"{prefix}e{e}.", rnd)
    return out + expert(h, tensors, prefix + "shared.", rnd) if mlp.get("shared") else out


# -- layer and model ----------------------------------------------------------------------------------------------------
def layer_forward(x, positions, config: dict, tensors: dict, index: int, rnd=_same):
    layer, eps, p = config["layers"][index], float(config["norm"]["eps"]), f"l{index}."
    h = layer_norm(x, tensors[p + "norm1"], tensors[p + "norm1.b"], eps)
    if layer["type"] == "gla":
        out, _ = gla_mixer(h, layer["mixer"], tensors, p + "mix.", eps, rnd)
    elif layer["type"] == "attention":
        out = unit_attention(h, positions, layer["mixer"], tensors, p + "mix.", eps, rnd)
    elif layer["type"] == "attention_2":
        out = chunk_attention(h, positions, layer["mixer"], tensors, p + "mix.", eps, rnd)
    else:
        raise ValueError(layer["type"])
    mlp = layer.get("mlp")
    if mlp is not None:
        h = layer_norm(x, tensors[p + "norm2"], tensors[p + "norm2.b"], eps)
        out = out + (dense_feed_forward(h, tensors, p + "mlp.", rnd) if mlp["kind"] == "dense" else routed_feed_forward(h, mlp, tensors, p + "mlp.", rnd))
    return x + out


def layer_runs(config: dict) -> list:
    """[(layer, the pass whose vector joins the stream right before it, or None)], in the order in which they run."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    start, stop = int(loop["start"]), int(loop["stop"])
    runs = [(i, None) for i in range(start)]
    for t in range(int(loop["times"])):
        runs += [(i, t if i == start else None) for i in range(start, stop)]
    return runs + [(i, None) for i in range(stop, n)]


def forward(config: dict, tensors: dict, tokens, round_to=None, streams: list | None = None):
    """Logits [T, vocab] of one whole sequence; ``streams`` collects the stream after every layer run."""
    rnd = round_to or _same
    positions = np.arange(len(tokens))
    x = rnd(tensors["embed"])[np.asarray(tokens)] * float(config["embedding"]["scale"])
    for index, step in layer_runs(config):
        if step is not None:
            x = x + tensors["loop.step"][step]
        x = layer_forward(x, positions, config, tensors, index, rnd)
        if streams is not None:
            streams.append(x.copy())
    h = layer_norm(x, tensors["final.norm"], tensors["final.norm.b"], float(config["norm"]["eps"]))
    return soft_cap(product(h, tensors["head"], rnd), config.get("logit_softcap"))


DECAY_RANK = 6   # the rank of the random models' decay matrices, unless a test asks for another (a model's tensors give it)


def tensor_shapes(config: dict, decay_rank: int = DECAY_RANK) -> dict:
    """name -> shape of every tensor a model of this configuration has."""
    width, vocab = int(config["width"]), int(config["vocab"])
    shapes = {"embed": (vocab, width), "final.norm": (width,), "final.norm.b": (width,), "head": (vocab, width)}
    if config.get("loop"):
        shapes["loop.step"] = (int(config["loop"]["times"]), width)
    for index, layer in enumerate(config["layers"]):
        p, mixer, mlp = f"l{index}.", layer["mixer"], layer.get("mlp")
        m = p + "mix."
        shapes.update({p + "norm1": (width,), p + "norm1.b": (width,)})
        H, dim, vdim = (int(mixer[key]) for key in ("heads", "dim", "vdim"))
        if layer["type"] == "gla":
            shapes.update({m + "q": (H * dim, width), m + "k": (H * dim, width), m + "v": (H * vdim, width), m + "g": (H * vdim, width), m + "o": (width, H * vdim),
                           m + "norm": (vdim,), m + "a1": (decay_rank, width), m + "a2": (H * dim, decay_rank), m + "a2.b": (H * dim,)})
        else:
            G = int(mixer["kv_heads"])
            shapes.update({m + "q": (H * dim, width), m + "k": (G * dim, width), m + "v": (G * vdim, width), m + "o": (width, H * vdim), m + "sink": (H,)})
            if layer["type"] == "attention_2":
                shapes.update({m + "q.b": (H * dim,), m + "k.b": (G * dim,), m + "v.b": (G * vdim,), m + "o.b": (width,), m + "q.norm": (dim,), m + "k.norm": (dim,)})
        if mlp is None:
            continue
        shapes.update({p + "norm2": (width,), p + "norm2.b": (width,)})
        if mlp["kind"] == "dense":
            shapes.update({p + "mlp.up": (int(mlp["ff"]), width), p + "mlp.down": (width, int(mlp["ff"]))})
            continue
        shapes[p + "mlp.router"] = (int(mlp["router"]["experts"]), width)
        parts = [(f"e{e}", int(mlp["expert"]["ff"])) for e in range(int(mlp["router"]["experts"]))]
        if mlp.get("shared"):
            parts.append(("shared", int(mlp["shared"]["ff"])))
        for name, ff in parts:
            shapes.update({f"{p}mlp.{name}.gate": (ff, width), f"{p}mlp.{name}.up": (ff, width), f"{p}mlp.{name}.down": (width, ff)})
    return shapes


def greedy(config: dict, tensors: dict, prompt, n_new: int, round_to=None) -> list:
    tokens = list(prompt)
    for _ in range(n_new):
        tokens.append(int(forward(config, tensors, tokens, round_to)[-1].argmax()))
    return tokens[len(prompt):]


# -- random models for the tests ------------------------------------------------------------------------------------------
def random_weights(config: dict, seed: int, decay_rank: int = DECAY_RANK) -> dict:
    """Weights whose activations stay of order one and whose every mechanism moves the logits: matrices ~ N(0, 1/in) (the router's
    larger, so that its scores differ), gains around one, decays from quick to all but none. float32 arrays holding bfloat16 values (as
    files hold them)."""
    import plain_gpt2

    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(config, decay_rank).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm", "norm1", "norm2"):
            value = rng.normal(1.0, 0.15, shape)
        elif name.endswith(".a2.b"):
            value = rng.normal(1.0, 2.0, shape)
        elif last == "b":
            value = rng.normal(0.0, 0.3, shape)
        elif last == "sink":
            value = rng.normal(0.5, 1.0, shape)
        elif last == "embed":
            value = rng.normal(0.0, 1.0 / float(config["embedding"]["scale"]), shape)
        elif last == "step":
            value = rng.normal(0.0, 0.6, shape)
        elif last == "router":
            value = rng.normal(0.0, 2.0 * shape[1] ** -0.5, shape)
        elif last == "head":
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
