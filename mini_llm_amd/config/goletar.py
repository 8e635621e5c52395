"""Typed configuration of the Goletar architecture: an embedding of token pairs, a list of layers with a norm before and behind every
branch, each layer with its own kind of mixer and its own sizes, and feed-forwards of routed experts.

config.json keys: ``architecture`` ("Goletar"), ``vocab``, ``width``, ``embedding.bigram`` {buckets, mul_prev, mul_cur}, ``norm.eps`` and
``layers``, a list of {``type``, ``mixer``, ``mlp``}. By ``type``:

- "latent_attention": mixer = {heads, dim, rot_dim, vdim, kv_rank, scale, rot: {dims, base}}.
- "mingru": mixer = {width} (elements of the recurrent state).

``mlp`` is null or {kind: "moe", expert: {ff, limit}, router: {experts, top}}."""

from __future__ import annotations

from dataclasses import dataclass

from .base import ConfigError, ModelConfig, take_float, take_int
from .dizizen import MAX_ROUTER_OUTPUTS
from .gimozen import MAX_LATENT_RANK
from .ketolix import _section
from .perezen import HalfRotaryConfig

MAX_PAIR_FACTOR = 2**31 - 1   # the pair's number is formed in 64-bit integers: token ids and factors below 2^31 never wrap


@dataclass(frozen=True)
class PairTableConfig:
    buckets: int
    mul_prev: int
    mul_cur: int

    @classmethod
    def from_dict(cls, raw: dict) -> "PairTableConfig":
        out = cls(take_int(raw, "buckets"), take_int(raw, "mul_prev", minimum=0), take_int(raw, "mul_cur", minimum=0))
        if max(out.buckets, out.mul_prev, out.mul_cur) > MAX_PAIR_FACTOR:
            raise ConfigError(f"embedding.bigram: numbers up to {MAX_PAIR_FACTOR}")
        return out

    def to_dict(self) -> dict:
        return {"buckets": self.buckets, "mul_cur": self.mul_cur, "mul_prev": self.mul_prev}


@dataclass(frozen=True)
class LatentAttentionConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot: HalfRotaryConfig

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "LatentAttentionConfig":
        rot_dim, kv_rank = take_int(raw, "rot_dim", minimum=0), take_int(raw, "kv_rank")
        if kv_rank > MAX_LATENT_RANK:
            raise ConfigError(f"{where}a latent of {kv_rank} is wider than the latent attention kernel takes ({MAX_LATENT_RANK})")
        return cls(take_int(raw, "heads"), take_int(raw, "dim"), rot_dim, take_int(raw, "vdim"), kv_rank, take_float(raw, "scale"),
                   HalfRotaryConfig.from_dict(_section(raw, "rot", where), where, rot_dim))

    def to_dict(self) -> dict:
        return {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "rot": self.rot.to_dict(), "rot_dim": self.rot_dim,
                "scale": self.scale, "vdim": self.vdim}


@dataclass(frozen=True)
class MinGruConfig:
    width: int

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "MinGruConfig":
        return cls(take_int(raw, "width"))

    def to_dict(self) -> dict:
        return {"width": self.width}


MIXERS = {"latent_attention": LatentAttentionConfig, "mingru": MinGruConfig}


@dataclass(frozen=True)
class GatedExpertsConfig:
    experts: int
    top: int
    ff: int
    limit: float

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "GatedExpertsConfig":
        router, expert = _section(raw, "router", where), _section(raw, "expert", where)
        experts, top = take_int(router, "experts"), take_int(router, "top")
        if experts > MAX_ROUTER_OUTPUTS:
            raise ConfigError(f"{where}{experts} experts are more than the router kernel takes ({MAX_ROUTER_OUTPUTS})")
        if top > experts:
            raise ConfigError(f"{where}{top} experts cannot be picked among {experts}")
        limit = take_float(expert, "limit")
        if not limit > 0:
            raise ConfigError(f"{where}mlp.expert.limit must be positive, not {limit}")
        return cls(experts, top, take_int(expert, "ff"), limit)

    def to_dict(self) -> dict:
        return {"expert": {"ff": self.ff, "limit": self.limit}, "kind": "moe", "router": {"experts": self.experts, "top": self.top}}


@dataclass(frozen=True)
class LayerConfig:
    type: str
    mixer: object
    mlp: GatedExpertsConfig | None   # None: the layer has no feed-forward

    def to_dict(self) -> dict:
        return {"mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict(), "type": self.type}


@dataclass(frozen=True)
class GoletarConfig(ModelConfig):
    vocab: int
    width: int
    pairs: PairTableConfig
    norm_eps: float
    layers: tuple
    eos_token_id: int | None = None

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @classmethod
    def from_dict(cls, raw: dict) -> "GoletarConfig":
        layers_raw = raw.get("layers")
        if not isinstance(layers_raw, list) or not layers_raw:
            raise ConfigError("config.json has no list of 'layers'")
        layers = []
        for index, entry in enumerate(layers_raw):
            where = f"layer {index}: "
            if not isinstance(entry, dict):
                raise ConfigError(f"{where}must be an object")
            kind = entry.get("type")
            if kind not in MIXERS:
                raise ConfigError(f"{where}unknown type {kind!r}; known: {', '.join(sorted(MIXERS))}")
            mixer = MIXERS[kind].from_dict(_section(entry, "mixer", where), where)
            mlp_raw = _section(entry, "mlp", where, optional=True)
            mlp = None
            if mlp_raw is not None:
                if mlp_raw.get("kind", "moe") != "moe":
                    raise ConfigError(f"{where}unknown mlp.kind {mlp_raw.get('kind')!r}; known: moe")
                mlp = GatedExpertsConfig.from_dict(mlp_raw, where)
            layers.append(LayerConfig(kind, mixer, mlp))
        eps = take_float(_section(raw, "norm", ""), "eps")
        if not eps > 0:
            raise ConfigError(f"norm.eps must be positive, not {eps}")
        eos = raw.get("eos_token_id")
        if eos is not None and (isinstance(eos, bool) or not isinstance(eos, int)):
            raise ConfigError(f"'eos_token_id' must be an integer or null, not {eos!r}")
        return cls(architecture=raw.get("architecture") or "Goletar", vocab=take_int(raw, "vocab"), width=take_int(raw, "width"),
                   pairs=PairTableConfig.from_dict(_section(_section(raw, "embedding", ""), "bigram", "embedding.")), norm_eps=eps,
                   layers=tuple(layers), eos_token_id=eos)

    def to_dict(self) -> dict:
        out = {"architecture": self.architecture, "embedding": {"bigram": self.pairs.to_dict()}, "layers": [layer.to_dict() for layer in self.layers],
               "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width}
        if self.eos_token_id is not None:
            out["eos_token_id"] = self.eos_token_id
        return out
