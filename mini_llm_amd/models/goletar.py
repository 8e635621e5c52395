"""The Goletar architecture as a recipe of parts: a token embedding plus a row picked by the token and the one before it, layers with a
norm in front of each branch and one on its output (x <- x + norm1b(mixer(norm1(x))), x <- x + norm2b(ff(norm2(x))), every norm with
one number as its gain), per layer the mixer its configuration names (attention over a shared latent with one gate a head, or a gated
recurrence whose gates read the current token alone), feed-forwards of routed experts whose weights multiply the experts' input, a
final norm and a head of its own.

Tensor names: ``embed``, ``bigram``, ``l<i>.norm{1,1b,2,2b}``, ``l<i>.mix.<name>``, ``l<i>.mlp.router``, ``l<i>.mlp.e<j>.{gate,up,down}``,
``final.norm``, ``head``."""

from __future__ import annotations

from ..config.goletar import GatedExpertsConfig, GoletarConfig, LatentAttentionConfig, MinGruConfig
from ..config.registry import register_architecture
from ..parts import LinearHead, PairEmbedding, make_part
from .base import LayerCall, Model

QUICK_SIGMOID = 1.702     # an expert's gate unit is g * sigmoid(1.702 g) * (u + 1)
UP_SHIFT = 1.0
CANDIDATE_SHIFT = 0.5     # what joins a non-negative sum in the recurrence's candidate


def _mixer(config: GoletarConfig, mixer):
    if isinstance(mixer, LatentAttentionConfig):
        rotary = make_part("position_encoding", "rotary", dims=mixer.rot.dims, base=mixer.rot.base, pairing="neighbours")
        return make_part("mixer", "latent_attention", width=config.width, n_heads=mixer.heads, dim=mixer.dim, rot_dim=mixer.rot_dim,
                         vdim=mixer.vdim, kv_rank=mixer.kv_rank, scale=mixer.scale, eps=config.norm_eps, rotary=rotary, gate="heads")
    if isinstance(mixer, MinGruConfig):
        return make_part("mixer", "mingru", width=config.width, state_width=mixer.width, candidate_shift=CANDIDATE_SHIFT)
    raise TypeError(f"no mixer for {type(mixer).__name__}")


def _feed_forward(config: GoletarConfig, mlp: GatedExpertsConfig | None):
    if mlp is None:
        return None
    return make_part("feed_forward", "routed_experts", width=config.width, n_experts=mlp.experts, ff=mlp.ff, top=mlp.top, correction=False,
                     score="sigmoid", renormalise=False, unit="clamped_gate", limit=mlp.limit, alpha=QUICK_SIGMOID, shift=UP_SHIFT,
                     weigh="input")


def build_goletar(config: GoletarConfig, precision) -> Model:
    width, eps = config.width, config.norm_eps
    norm = lambda: make_part("norm", "rmsnorm", width=width, eps=eps, one_gain=True, tensor_name="")
    blocks, schedule = [], []
    for index, layer in enumerate(config.layers):
        has_mlp = layer.mlp is not None
        blocks.append(make_part(
            "block", "sandwich_norm", norm_1=norm(), mixer=_mixer(config, layer.mixer), norm_1b=norm(), norm_2=norm() if has_mlp else None,
            feed_forward=_feed_forward(config, layer.mlp), norm_2b=norm() if has_mlp else None, compute_dtype=precision.compute,
        ))
        schedule.append(LayerCall(block=index, cache=index))
    for block, following in zip(blocks, blocks[1:]):   # the schedule runs the layers in their order: a layer's last kernel norms for the next
        block.hand_to(following.norm_1)
    return Model(
        config, precision,
        embedding=PairEmbedding(config.vocab, width, buckets=config.pairs.buckets, mul_previous=config.pairs.mul_prev, mul_current=config.pairs.mul_cur,
                                tensor_name="embed", pair_name="bigram", std=0.7),
        position_encoding=None,
        blocks=blocks, schedule=schedule,
        final_norm=norm(),
        head=LinearHead(config.vocab, width, tensor_name=""),
        names={"embedding": "", "block": "l{i}.", "final_norm": "final.norm", "head": "head"},
    )


register_architecture("Goletar", GoletarConfig, build_goletar)
