"""The Gevulorn architecture as a recipe of parts: a scaled token embedding; layers with two layer norms of the same stream, x <- x +
mixer(norm1(x)) + ff(norm2(x)); per layer the mixer its configuration names (gated linear attention; attention with queries and keys of unit
size, a window that keeps the first tokens, and a sink; or attention with biases, normed queries and keys, stretched rotation, capped scores,
chunks and a sink); a dense feed-forward with the square of relu, routed experts with a shared one, or none; a run of layers that the schedule
goes through several times with the same weights, each pass with a cache or state of its own and a vector of its own that joins the stream in
front of it; a final layer norm, a head of its own and capped logits.

Tensor names: ``embed``, ``loop.step``, ``l<i>.norm{1,2}`` (+ ``.b``), ``l<i>.mix.<name>``, ``l<i>.mlp.{up,down}`` or
``l<i>.mlp.{router,e<j>.{gate,up,down},shared.{gate,up,down}}``, ``final.norm`` (+ ``.b``), ``head``."""

from __future__ import annotations

from ..config.gevulorn import ChunkAttentionConfig, DenseConfig, ExpertsConfig, GevulornConfig, GlaConfig, WindowAttentionConfig
from ..config.registry import register_architecture
from ..parts import LinearHead, TokenEmbedding, make_part
from .base import LayerCall, Model, StepVectors


def _rotary(rot):
    if rot is None or rot.dims == 0:
        return None
    scaling = None if rot.scaling is None else rot.scaling_dict()
    return make_part("position_encoding", "rotary", dims=rot.dims, base=rot.base, scaling=scaling, pairing="half")


def _mixer(config: GevulornConfig, mixer):
    width, eps = config.width, config.norm_eps
    if isinstance(mixer, GlaConfig):
        return make_part("mixer", "gated_linear_attention", width=width, n_heads=mixer.heads, dim=mixer.dim, vdim=mixer.vdim, tau=mixer.tau, eps=eps)
    common = dict(width=width, n_heads=mixer.heads, n_kv_heads=mixer.kv_heads, dim=mixer.dim, vdim=mixer.vdim, scale=mixer.scale,
                  rotary=_rotary(mixer.rot), eps=eps, sink=True)
    if isinstance(mixer, WindowAttentionConfig):
        return make_part("mixer", "rotary_attention", **common, biases=False, qk_norm="unit", window=mixer.window, keep_first=mixer.keep_first)
    if isinstance(mixer, ChunkAttentionConfig):
        return make_part("mixer", "rotary_attention", **common, biases=True, qk_norm="gains", softcap=mixer.softcap, chunk=mixer.chunk)
    raise TypeError(f"no mixer for {type(mixer).__name__}")


def _feed_forward(config: GevulornConfig, mlp):
    if mlp is None:
        return None
    if isinstance(mlp, DenseConfig):
        return make_part("feed_forward", "plain_mlp", width=config.width, inner=mlp.ff, activation="squared_relu")
    if isinstance(mlp, ExpertsConfig):   # the gate unit without a limit and without a shift is silu(gate) * up
        return make_part("feed_forward", "routed_experts", width=config.width, n_experts=mlp.experts, ff=mlp.ff, top=mlp.top, correction=False,
                         score="softmax", renormalise=True, unit="clamped_gate", limit=None, alpha=1.0, shift=0.0, shared_ff=mlp.shared_ff)
    raise TypeError(f"no feed-forward for {type(mlp).__name__}")


def _schedule(config: GevulornConfig) -> list:
    """The layers in their order, the looped ones `times` times; every call has a cache layer of its own."""
    n, loop = len(config.layers), config.loop
    if loop is None:
        runs = [(i, None) for i in range(n)]
    else:
        looped = [(i, t if i == loop.start else None) for t in range(loop.times) for i in range(loop.start, loop.stop)]
        runs = [(i, None) for i in range(loop.start)] + looped + [(i, None) for i in range(loop.stop, n)]
    return [LayerCall(block=i, cache=at, step=step) for at, (i, step) in enumerate(runs)]


class GevulornModel(Model):
    def canonical_tensor_name(self, name: str) -> str | None:
        """A layer without a feed-forward has no use for its second norm, should a file hold one."""
        head, dot, rest = name.partition(".")
        if head[:1] == "l" and head[1:].isdigit() and rest in ("norm2", "norm2.b"):
            index = int(head[1:])
            if index < len(self.config.layers) and self.config.layers[index].mlp is None:
                return None
        return name


def build_gevulorn(config: GevulornConfig, precision) -> Model:
    width, eps = config.width, config.norm_eps
    norm = lambda: make_part("norm", "layernorm", width=width, eps=eps, tensor_names=("", ".b"))
    blocks = [make_part("block", "parallel", norm_1=norm(), mixer=_mixer(config, layer.mixer), feed_forward=_feed_forward(config, layer.mlp),
                        norm_2=norm() if layer.mlp is not None else None, width=width, compute_dtype=precision.compute) for layer in config.layers]
    return GevulornModel(
        config, precision,
        embedding=TokenEmbedding(config.vocab, width, scale=config.embedding_scale, tensor_name="", std=1.0 / max(config.embedding_scale, 1e-6)),
        position_encoding=None, blocks=blocks, schedule=_schedule(config), final_norm=norm(),
        head=LinearHead(config.vocab, width, tensor_name="", softcap=config.logit_softcap),
        names={"embedding": "embed", "block": "l{i}.", "final_norm": "final.norm", "head": "head", "step_vectors": "loop.step"},
        step_vectors=None if config.loop is None else StepVectors(config.loop.times, width, tensor_name=""),
    )


register_architecture("Gevulorn", GevulornConfig, build_gevulorn)
