"""Typed configuration of the Gevulorn architecture: layers whose mixer and feed-forward run side by side on norms of their own, each
layer with its own kind of mixer and its own sizes, and a run of layers that is gone through several times.

config.json keys: ``architecture`` ("Gevulorn"), ``vocab``, ``width``, ``embedding.scale`` (absent: 1), ``norm.eps``, ``logit_softcap`` (absent or
null: none), ``loop`` (absent or null: none) {start, stop, times} and ``layers``, a list of {``type``, ``mixer``, ``mlp``}. By ``type``:

- "gla": mixer = {heads, dim, vdim, tau}.
- "attention": mixer = {heads, kv_heads, dim, vdim, scale, rot: {dims, base}, mask: {size, keep_first | absent} | absent}.
- "attention_2": mixer = {heads, kv_heads, dim, vdim, scale, softcap | absent, rot: {dims, base, scaling: {factor, low, high, original} |
  absent}, mask: {size} | absent (chunks of so many positions)}.

``mlp`` is null, {kind: "dense", ff} or {kind: "moe", expert: {ff}, router: {experts, top}, shared: {ff} | absent}."""

from __future__ import annotations

from dataclasses import dataclass

from .base import ConfigError, ModelConfig, take_float, take_int
from .dizizen import MAX_ROUTER_OUTPUTS
from .ketolix import MAX_HEAD_SIZE, PairRotaryConfig, _grouped_heads, _rot, _section, recurrence_fits

EXPERT_UNITS = 64   # an expert's hidden units are laid out in multiples of this; a shared expert as so many experts of that size


def _optional(raw: dict, key: str, where: str):
    """A positive number, or None where the key is absent or null."""
    if raw.get(key) is None:
        return None
    value = take_float(raw, key)
    if not value > 0:
        raise ConfigError(f"{where}{key} must be positive, not {value}")
    return value


@dataclass(frozen=True)
class GlaConfig:
    heads: int
    dim: int
    vdim: int
    tau: float

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "GlaConfig":
        dim, vdim = take_int(raw, "dim"), take_int(raw, "vdim")
        if not recurrence_fits(dim, vdim):
            raise ConfigError(f"{where}heads of {dim} x {vdim} are larger than the recurrence kernel takes")
        tau = take_float(raw, "tau")
        if not tau > 0:
            raise ConfigError(f"{where}tau must be positive, not {tau}")
        return cls(take_int(raw, "heads"), dim, vdim, tau)

    def to_dict(self) -> dict:
        return {"dim": self.dim, "heads": self.heads, "tau": self.tau, "vdim": self.vdim}


@dataclass(frozen=True)
class HeadsConfig:
    """What both kinds of attention have."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: PairRotaryConfig | None

    @classmethod
    def _common(cls, raw: dict, where: str) -> tuple:
        heads, kv_heads = _grouped_heads(raw, where)
        dim, vdim = take_int(raw, "dim"), take_int(raw, "vdim")
        if max(dim, vdim) > MAX_HEAD_SIZE:
            raise ConfigError(f"{where}heads of {max(dim, vdim)} are wider than the attention kernels take ({MAX_HEAD_SIZE})")
        return heads, kv_heads, dim, vdim, take_float(raw, "scale"), _rot(raw, where, dim)

    def to_dict(self) -> dict:
        out = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.vdim}
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass(frozen=True)
class WindowAttentionConfig(HeadsConfig):
    window: int | None   # mask.size: a query sees so many keys, itself among them; None: all before it
    keep_first: int      # and the sequence's first so many

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "WindowAttentionConfig":
        common = cls._common(raw, where)
        if common[-1] is not None and common[-1].scaling is not None:
            raise ConfigError(f"{where}this kind of attention stretches no frequencies")
        mask = _section(raw, "mask", where, optional=True)
        if mask is None:
            return cls(*common, None, 0)
        return cls(*common, take_int(mask, "size"), take_int(mask, "keep_first", 0, minimum=0))

    def to_dict(self) -> dict:
        out = super().to_dict()
        if self.window is not None:
            out["mask"] = {"keep_first": self.keep_first, "size": self.window}
        return out


@dataclass(frozen=True)
class ChunkAttentionConfig(HeadsConfig):
    chunk: int | None    # mask.size: a query sees the keys of its own chunk of so many positions; None: all before it
    softcap: float | None

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "ChunkAttentionConfig":
        mask = _section(raw, "mask", where, optional=True)
        return cls(*cls._common(raw, where), None if mask is None else take_int(mask, "size"), _optional(raw, "softcap", where))

    def to_dict(self) -> dict:
        out = super().to_dict()
        if self.chunk is not None:
            out["mask"] = {"size": self.chunk}
        if self.softcap is not None:
            out["softcap"] = self.softcap
        return out


MIXERS = {"gla": GlaConfig, "attention": WindowAttentionConfig, "attention_2": ChunkAttentionConfig}


@dataclass(frozen=True)
class DenseConfig:
    ff: int

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "DenseConfig":
        return cls(take_int(raw, "ff"))

    def to_dict(self) -> dict:
        return {"ff": self.ff, "kind": "dense"}


@dataclass(frozen=True)
class ExpertsConfig:
    experts: int
    top: int
    ff: int
    shared_ff: int | None

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "ExpertsConfig":
        router, ff = _section(raw, "router", where), take_int(_section(raw, "expert", where), "ff")
        experts, top = take_int(router, "experts"), take_int(router, "top")
        if top > experts:
            raise ConfigError(f"{where}{top} experts cannot be picked among {experts}")
        shared = _section(raw, "shared", where, optional=True)
        shared_ff = None if shared is None else take_int(shared, "ff")
        units = -(-ff // EXPERT_UNITS) * EXPERT_UNITS
        laid_out = experts + (0 if shared_ff is None else -(-shared_ff // units))
        if laid_out > MAX_ROUTER_OUTPUTS:
            raise ConfigError(f"{where}{laid_out} experts (a shared one counted by its size) are more than the router kernel takes ({MAX_ROUTER_OUTPUTS})")
        return cls(experts, top, ff, shared_ff)

    def to_dict(self) -> dict:
        out = {"expert": {"ff": self.ff}, "kind": "moe", "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff is not None:
            out["shared"] = {"ff": self.shared_ff}
        return out


MLPS = {"dense": DenseConfig, "moe": ExpertsConfig}


@dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int    # layers start .. stop - 1 are gone through `times` times in a row
    times: int

    @classmethod
    def from_dict(cls, raw: dict, n_layers: int) -> "LoopConfig":
        out = cls(take_int(raw, "start", minimum=0), take_int(raw, "stop"), take_int(raw, "times"))
        if not out.start < out.stop <= n_layers:
            raise ConfigError(f"loop: layers {out.start} to {out.stop} are no run of the {n_layers} there are")
        return out

    def to_dict(self) -> dict:
        return {"start": self.start, "stop": self.stop, "times": self.times}


@dataclass(frozen=True)
class LayerConfig:
    type: str
    mixer: object
    mlp: object   # DenseConfig, ExpertsConfig or None: the layer has no feed-forward

    def to_dict(self) -> dict:
        return {"mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict(), "type": self.type}


@dataclass(frozen=True)
class GevulornConfig(ModelConfig):
    vocab: int
    width: int
    embedding_scale: float
    norm_eps: float
    logit_softcap: float | None
    loop: LoopConfig | None
    layers: tuple
    eos_token_id: int | None = None

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @classmethod
    def from_dict(cls, raw: dict) -> "GevulornConfig":
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
                mlp_kind = mlp_raw.get("kind", "dense")
                if mlp_kind not in MLPS:
                    raise ConfigError(f"{where}unknown mlp.kind {mlp_kind!r}; known: {', '.join(sorted(MLPS))}")
                mlp = MLPS[mlp_kind].from_dict(mlp_raw, where)
            layers.append(LayerConfig(kind, mixer, mlp))
        eps = take_float(_section(raw, "norm", ""), "eps")
        if not eps > 0:
            raise ConfigError(f"norm.eps must be positive, not {eps}")
        loop = _section(raw, "loop", "", optional=True)
        eos = raw.get("eos_token_id")
        if eos is not None and (isinstance(eos, bool) or not isinstance(eos, int)):
            raise ConfigError(f"'eos_token_id' must be an integer or null, not {eos!r}")
        return cls(architecture=raw.get("architecture") or "Gevulorn", vocab=take_int(raw, "vocab"), width=take_int(raw, "width"),
                   embedding_scale=take_float(_section(raw, "embedding", "", optional=True) or {}, "scale", 1.0), norm_eps=eps,
                   logit_softcap=_optional(raw, "logit_softcap", ""), loop=None if loop is None else LoopConfig.from_dict(loop, len(layers)),
                   layers=tuple(layers), eos_token_id=eos)

    def to_dict(self) -> dict:
        out = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale}, "layers": [layer.to_dict() for layer in self.layers],
               "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width}
        if self.logit_softcap is not None:
            out["logit_softcap"] = self.logit_softcap
        if self.loop is not None:
            out["loop"] = self.loop.to_dict()
        if self.eos_token_id is not None:
            out["eos_token_id"] = self.eos_token_id
        return out
