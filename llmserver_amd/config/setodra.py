"""Setodra configuration: a nested ``config.json`` that lists the layers one by one.

Top level: ``architecture`` ("Setodra"), ``vocab``, ``width``, ``norm.eps``, ``layers`` and, each optional,
``embedding.scale`` (what the embedding rows are multiplied by) and ``loop`` (``start``, ``stop``, ``times``: the layers
``start`` to ``stop - 1`` run ``times`` times in a row with the same weights).  A layer entry gives ``type`` (its mixer:
``latent_attention``, ``retention`` or ``mamba2``), ``mixer`` (the mixer's sizes and constants) and ``mlp`` (``kind`` ``moe``
with its experts, router and shared expert, or null).  Nothing here is a default of the design: what the file does not name is
not there (no loop, no shared expert, no identity experts, no scaling of a rotation, a scale of one).
"""
from __future__ import annotations

import dataclasses
from typing import Any, ClassVar, Mapping, Optional, Tuple, Union

from .barotar import _mapping, _positive
from .base import ConfigError, ModelConfig, UnsupportedModelError, field
from .kerudra import Loop, _optional_mapping
from .zepolix import _number

FEED_FORWARDS = ("moe",)
MOST_ROW = 256              # numbers a token of latent attention caches: what the attention kernels take
MOST_KEY_CHANNELS = 512     # ... and key channels of a head that carries a matrix: what the recurrence kernels take
MOST_CHOICES = 3072         # ... and router outputs


@dataclasses.dataclass(frozen=True)
class Yarn:
    factor: float
    original: float
    fast: float
    slow: float

    def to_dict(self) -> dict:
        return dataclasses.asdict(self)


@dataclasses.dataclass(frozen=True)
class Rotation:
    """Dimension i turns with dimension i + dims / 2; ``dims`` 0: nothing turns."""
    dims: int
    base: float
    scaling: Optional[Yarn]

    @classmethod
    def read(cls, where: str, raw: Mapping[str, Any], most: int) -> "Rotation":
        rot = _optional_mapping(where, raw, "rot")
        if rot is None:
            return cls(0, 1.0, None)
        where += ".rot"
        scaling = _optional_mapping(where, rot, "scaling")
        if scaling is not None:
            scaling = Yarn(*(_number(where + ".scaling", scaling, key, float) for key in ("factor", "original", "fast", "slow")))
            _positive(where + ".scaling", scaling, ("factor", "original", "fast", "slow"))
        out = cls(_number(where, rot, "dims"), _number(where, rot, "base", float), scaling)
        if out.dims < 0 or out.dims % 2 or out.dims > most or out.base <= 0 or (scaling is not None and out.base == 1.0):
            raise ConfigError(f"config.json: {where}: an even number of up to {most} dimensions turns, with a positive base; got {out.dims}, {out.base}")
        return out

    def to_dict(self) -> dict:
        if not self.dims:
            return {}
        return {"rot": {"dims": self.dims, "base": self.base, **({"scaling": self.scaling.to_dict()} if self.scaling is not None else {})}}


@dataclasses.dataclass(frozen=True)
class LatentSizes:
    """Attention over a shared low-rank latent with a rotated key part."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot: Rotation

    @classmethod
    def read(cls, where: str, raw: Mapping[str, Any]) -> "LatentSizes":
        rot_dim = _number(where, raw, "rot_dim")
        sizes = cls(_number(where, raw, "heads"), _number(where, raw, "dim"), rot_dim, _number(where, raw, "vdim"), _number(where, raw, "kv_rank"),
                    _number(where, raw, "scale", float), Rotation.read(where, raw, rot_dim))
        _positive(where, sizes, ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        if not sizes.rot.dims:
            raise ConfigError(f"config.json: {where} must give 'rot' for its rotated part")
        return sizes

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim, "kv_rank": self.kv_rank, "scale": self.scale,
                **self.rot.to_dict()}


@dataclasses.dataclass(frozen=True)
class RetentionSizes:
    """A matrix per head under a fixed decay."""
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    rot: Rotation

    @classmethod
    def read(cls, where: str, raw: Mapping[str, Any]) -> "RetentionSizes":
        dim, decay = _number(where, raw, "dim"), raw.get("decay")
        if not isinstance(decay, (list, tuple)) or not all(isinstance(d, (int, float)) and not isinstance(d, bool) and d > 0 for d in decay):
            raise ConfigError(f"config.json: {where}.decay must list a positive number for every head, got {decay!r}")
        sizes = cls(_number(where, raw, "heads"), dim, _number(where, raw, "vdim"), tuple(float(d) for d in decay), Rotation.read(where, raw, dim))
        _positive(where, sizes, ("heads", "dim", "vdim"))
        if len(sizes.decay) != sizes.heads:
            raise ConfigError(f"config.json: {where}.decay lists {len(sizes.decay)} decays for {sizes.heads} heads")
        return sizes

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay), **self.rot.to_dict()}


@dataclasses.dataclass(frozen=True)
class StateSpaceSizes:
    """A state-space mixer with one decay per head and token (Mamba-2)."""
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int

    @classmethod
    def read(cls, where: str, raw: Mapping[str, Any]) -> "StateSpaceSizes":
        names = ("heads", "vdim", "state", "groups", "conv", "norm_groups")
        sizes = cls(*(_number(where, raw, name) for name in names))
        _positive(where, sizes, names)
        if sizes.heads % sizes.groups:
            raise ConfigError(f"config.json: {where}: {sizes.heads} heads do not fall into {sizes.groups} equal groups")
        if (sizes.heads * sizes.vdim) % sizes.norm_groups:
            raise ConfigError(f"config.json: {where}: {sizes.heads * sizes.vdim} channels do not fall into {sizes.norm_groups} equal parts")
        return sizes

    def to_dict(self) -> dict:
        return dataclasses.asdict(self)


MIXER_SIZES = {"latent_attention": LatentSizes, "retention": RetentionSizes, "mamba2": StateSpaceSizes}
MIXERS = tuple(MIXER_SIZES)


@dataclasses.dataclass(frozen=True)
class ExpertsSizes:
    ff: int
    experts: int
    top: int
    scale: float
    identity: int
    shared_ff: int              # 0: no shared expert

    @classmethod
    def read(cls, where: str, raw: Mapping[str, Any]) -> "ExpertsSizes":
        router, expert = _mapping(where, raw, "router"), _mapping(where, raw, "expert")
        shared = _optional_mapping(where, raw, "shared")
        sizes = cls(_number(where + ".expert", expert, "ff"), _number(where + ".router", router, "experts"), _number(where + ".router", router, "top"),
                    _number(where + ".router", router, "scale", float) if "scale" in router else 1.0,
                    _number(where + ".router", router, "identity") if "identity" in router else 0,
                    _number(where + ".shared", shared, "ff") if shared is not None else 0)
        _positive(where, sizes, ("ff", "experts", "top"))
        if sizes.identity < 0 or sizes.top > sizes.experts + sizes.identity or (shared is not None and sizes.shared_ff <= 0):
            raise ConfigError(f"config.json: {where}: a token uses {sizes.top} of {sizes.experts} experts and {sizes.identity} identity experts, "
                              f"shared expert of {sizes.shared_ff}")
        return sizes

    def to_dict(self) -> dict:
        router = {"experts": self.experts, "top": self.top, "scale": self.scale, "identity": self.identity}
        return {"kind": "moe", "expert": {"ff": self.ff}, "router": router, **({"shared": {"ff": self.shared_ff}} if self.shared_ff else {})}


@dataclasses.dataclass(frozen=True)
class SetodraLayer:
    type: str
    mixer: Union[LatentSizes, RetentionSizes, StateSpaceSizes]
    mlp: Optional[ExpertsSizes]

    def to_dict(self) -> dict:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclasses.dataclass(frozen=True)
class SetodraConfig(ModelConfig):
    MODEL_TYPE: ClassVar[str] = "Setodra"

    vocab: int = field("vocab", int)
    width: int = field("width", int)
    norm: object = field("norm", object)
    layers_raw: object = field("layers", object)
    embedding: object = field("embedding", object, None)
    loop_raw: object = field("loop", object, None)
    layers: Tuple[SetodraLayer, ...] = ()
    loop: Optional[Loop] = None
    norm_eps: float = 0.0
    embedding_scale: float = 1.0

    def resolve(self, raw: Mapping[str, Any]) -> "SetodraConfig":
        if not isinstance(self.layers_raw, (list, tuple)) or not self.layers_raw:
            raise ConfigError("config.json: 'layers' must list at least one layer")
        layers = []
        for index, entry in enumerate(self.layers_raw):
            where = f"layers[{index}]"
            if not isinstance(entry, Mapping) or not isinstance(entry.get("type"), str):
                raise ConfigError(f"config.json: {where} must be an object with a 'type'")
            kind = entry["type"]
            if kind not in MIXERS:
                raise UnsupportedModelError(f"Model type {self.MODEL_TYPE!r}: {where} has the mixer {kind!r}; built: {', '.join(MIXERS)}")
            mixer = MIXER_SIZES[kind].read(where + ".mixer", _mapping(where, entry, "mixer"))
            mlp = entry.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, Mapping) or mlp.get("kind") not in FEED_FORWARDS:
                    named = mlp.get("kind") if isinstance(mlp, Mapping) else mlp
                    raise UnsupportedModelError(f"Model type {self.MODEL_TYPE!r}: {where} has the feed-forward {named!r}; built: {', '.join(FEED_FORWARDS)}")
                mlp = ExpertsSizes.read(where + ".mlp", mlp)
            layers.append(SetodraLayer(kind, mixer, mlp))
        loop = None
        if self.loop_raw is not None:
            loop = Loop(*(_number("loop", self.loop_raw, key) for key in ("start", "stop", "times")))
        scale = 1.0
        if self.embedding is not None:
            if not isinstance(self.embedding, Mapping):
                raise ConfigError("config.json: 'embedding' must be an object")
            if "scale" in self.embedding:
                scale = _number("embedding", self.embedding, "scale", float)
        return dataclasses.replace(self, layers=tuple(layers), loop=loop, norm_eps=_number("norm", self.norm, "eps", float),
                                   embedding_scale=scale)

    def validate(self, raw: Mapping[str, Any]) -> None:
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError(f"vocab and width must be positive: {self.vocab}, {self.width}")
        if self.norm_eps <= 0.0:
            raise ConfigError(f"norm.eps must be positive: {self.norm_eps}")
        if self.loop is not None and not (0 <= self.loop.start < self.loop.stop <= len(self.layers) and self.loop.times >= 1):
            raise ConfigError(f"loop: layers {self.loop.start} to {self.loop.stop - 1} of {len(self.layers)}, {self.loop.times} times")
        for index, layer in enumerate(self.layers):
            sizes = layer.mixer
            if isinstance(sizes, LatentSizes) and sizes.kv_rank + sizes.rot_dim > MOST_ROW:
                raise UnsupportedModelError(f"Model type {self.MODEL_TYPE!r}: layers[{index}] caches rows of {sizes.kv_rank} + {sizes.rot_dim}; "
                                            f"the attention kernels take rows of up to {MOST_ROW}")
            channels = sizes.dim if isinstance(sizes, RetentionSizes) else sizes.state if isinstance(sizes, StateSpaceSizes) else 0
            if channels > MOST_KEY_CHANNELS:
                raise UnsupportedModelError(f"Model type {self.MODEL_TYPE!r}: layers[{index}] has heads of {channels} key channels; "
                                            f"the recurrence kernels take up to {MOST_KEY_CHANNELS}")
            if layer.mlp is not None and layer.mlp.experts + layer.mlp.identity > MOST_CHOICES:
                raise UnsupportedModelError(f"Model type {self.MODEL_TYPE!r}: layers[{index}] routes among {layer.mlp.experts + layer.mlp.identity}; "
                                            f"the router kernel takes up to {MOST_CHOICES}")

    def layer_runs(self) -> Tuple[Tuple[int, Optional[int]], ...]:
        """The layers in the order they run, a looped layer once for every pass: (layer, number of the pass that begins right
        in front of it, or None)."""
        plain = tuple((index, None) for index in range(len(self.layers)))
        if self.loop is None:
            return plain
        start, stop = self.loop.start, self.loop.stop
        looped = tuple((index, number if index == start else None) for number in range(self.loop.times) for index in range(start, stop))
        return plain[:start] + looped + plain[stop:]

    # what the rest of the package asks of any configuration
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def to_dict(self) -> dict:
        out = {"architecture": self.MODEL_TYPE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "embedding": {"scale": self.embedding_scale}, "layers": [layer.to_dict() for layer in self.layers]}
        if self.loop is not None:
            out["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        return out
