"""Mefurax configuration: a nested ``config.json`` that lists the layers one by one.

Top level: ``architecture`` ("Mefurax"), ``vocab``, ``width``, ``norm.eps``, ``postln_alpha`` (what the stream is multiplied
by before a sublayer's result joins it) and ``layers``.  A layer entry gives ``type`` (its mixer: ``attention`` or
``attention_2``), ``mixer`` (the mixer's sizes and constants) and ``mlp`` (``kind`` ``dense`` with ``ff``, ``kind`` ``moe`` with
``expert.ff``, ``router.{experts, top}`` and possibly ``shared.ff``, or null).  Both mixers give ``heads``, ``kv_heads``,
``dim``, ``vdim``, ``scale``, possibly ``mask.size`` (``attention``: the keys of a window; ``attention_2``: the length of a chunk;
absent: every earlier key is seen) and ``v_mix`` (whether the layer's values are mixed with the first such layer's).
``attention`` also gives ``conv`` (the taps of its short convolutions); ``attention_2`` gives ``rot.{dims, base}`` and possibly
``softcap``.  Nothing here is a default of the design: what the file does not name is not there.
"""
from __future__ import annotations

import dataclasses
from typing import Any, ClassVar, Mapping, Optional, Tuple, Union

from .barotar import _mapping, _positive
from .base import ConfigError, ModelConfig, UnsupportedModelError, field
from .gogalix import DenseSizes, _grouped
from .kerudra import _optional_mapping, _rotation, _rotation_dict, _window
from .zepolix import _number

MIXERS = ("attention", "attention_2")
FEED_FORWARDS = ("dense", "moe")
MOST_HEAD = 256             # the widest head the attention kernels take
MOST_WIDTH, MOST_HEADS = 14336, 512         # a token's queries as the kernel in front of attention takes them (csrc/compose.hip)


def _flag(where: str, raw: Mapping[str, Any], key: str) -> bool:
    value = raw.get(key, False)
    if not isinstance(value, bool):
        raise ConfigError(f"config.json: {where}.{key} must be true or false, got {value!r}")
    return value


def _heads(where: str, raw: Mapping[str, Any]) -> dict:
    """What both mixers give."""
    heads = _number(where, raw, "heads")
    return {"heads": heads, "kv_heads": _number(where, raw, "kv_heads") if "kv_heads" in raw else heads, "dim": _number(where, raw, "dim"),
            "vdim": _number(where, raw, "vdim"), "scale": _number(where, raw, "scale", float), "v_mix": _flag(where, raw, "v_mix")}


def _check_heads(where: str, sizes) -> None:
    _positive(where, sizes, ("heads", "kv_heads", "dim", "vdim", "scale"))
    _grouped(where, sizes.heads, sizes.kv_heads)


def _heads_dict(sizes, size: Optional[int]) -> dict:
    out = {name: getattr(sizes, name) for name in ("heads", "kv_heads", "dim", "vdim", "scale", "v_mix")}
    if size is not None:
        out["mask"] = {"size": size}
    return out


@dataclasses.dataclass(frozen=True)
class SlopedAttentionSizes:
    """Convolved projections normed as a whole, scores that fall with the distance, a window."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    v_mix: bool
    taps: int
    window: Optional[int]

    @classmethod
    def read(cls, where: str, raw: Mapping[str, Any]) -> "SlopedAttentionSizes":
        sizes = cls(**_heads(where, raw), taps=_number(where, raw, "conv"), window=_window(where, raw))
        _check_heads(where, sizes)
        _positive(where, sizes, ("taps",))
        return sizes

    def to_dict(self) -> dict:
        return {**_heads_dict(self, self.window), "conv": self.taps}


@dataclasses.dataclass(frozen=True)
class ChunkedAttentionSizes:
    """Rotated heads of unit root mean square, capped scores, chunks, a gate a head."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    v_mix: bool
    rot_dims: int
    rot_base: float
    softcap: Optional[float]
    chunk: Optional[int]

    @classmethod
    def read(cls, where: str, raw: Mapping[str, Any]) -> "ChunkedAttentionSizes":
        heads = _heads(where, raw)
        dims, base = _rotation(where, raw, heads["dim"])
        softcap = _number(where, raw, "softcap", float) if raw.get("softcap") is not None else None
        sizes = cls(**heads, rot_dims=dims, rot_base=base, softcap=softcap, chunk=_window(where, raw))
        _check_heads(where, sizes)
        if softcap is not None:
            _positive(where, sizes, ("softcap",))
        return sizes

    def to_dict(self) -> dict:
        out = {**_heads_dict(self, self.chunk), **_rotation_dict(self.rot_dims, self.rot_base)}
        if self.softcap is not None:
            out["softcap"] = self.softcap
        return out


@dataclasses.dataclass(frozen=True)
class ExpertsSizes:
    ff: int
    experts: int
    top: int
    shared: Optional[int]       # the inner size of the expert that every token uses, or None: there is none

    @classmethod
    def read(cls, where: str, raw: Mapping[str, Any]) -> "ExpertsSizes":
        router, shared = _mapping(where, raw, "router"), _optional_mapping(where, raw, "shared")
        sizes = cls(_number(where + ".expert", _mapping(where, raw, "expert"), "ff"), _number(where + ".router", router, "experts"),
                    _number(where + ".router", router, "top"), _number(where + ".shared", shared, "ff") if shared is not None else None)
        _positive(where, sizes, ("ff", "experts", "top") + (("shared",) if shared is not None else ()))
        if sizes.top > sizes.experts:
            raise ConfigError(f"config.json: {where}: a token cannot use {sizes.top} of {sizes.experts} experts")
        return sizes

    def to_dict(self) -> dict:
        out = {"kind": "moe", "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top}}
        if self.shared is not None:
            out["shared"] = {"ff": self.shared}
        return out


@dataclasses.dataclass(frozen=True)
class MefuraxLayer:
    type: str
    mixer: Union[SlopedAttentionSizes, ChunkedAttentionSizes]
    mlp: Union[DenseSizes, ExpertsSizes, None]

    def to_dict(self) -> dict:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclasses.dataclass(frozen=True)
class MefuraxConfig(ModelConfig):
    MODEL_TYPE: ClassVar[str] = "Mefurax"

    vocab: int = field("vocab", int)
    width: int = field("width", int)
    norm: object = field("norm", object)
    layers_raw: object = field("layers", object)
    alpha: float = field("postln_alpha", float)
    layers: Tuple[MefuraxLayer, ...] = ()
    norm_eps: float = 0.0

    def resolve(self, raw: Mapping[str, Any]) -> "MefuraxConfig":
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
            sizes = _mapping(where, entry, "mixer")
            mixer = (SlopedAttentionSizes if kind == "attention" else ChunkedAttentionSizes).read(where + ".mixer", sizes)
            layers.append(MefuraxLayer(kind, mixer, self._feed_forward(where, entry.get("mlp"))))
        return dataclasses.replace(self, layers=tuple(layers), norm_eps=_number("norm", self.norm, "eps", float))

    def _feed_forward(self, where: str, mlp):
        if mlp is None:
            return None
        if not isinstance(mlp, Mapping) or mlp.get("kind") not in FEED_FORWARDS:
            named = mlp.get("kind") if isinstance(mlp, Mapping) else mlp
            raise UnsupportedModelError(f"Model type {self.MODEL_TYPE!r}: {where} has the feed-forward {named!r}; built: {', '.join(FEED_FORWARDS)}")
        if mlp["kind"] == "moe":
            return ExpertsSizes.read(where + ".mlp", mlp)
        sizes = DenseSizes(_number(where + ".mlp", mlp, "ff"))
        _positive(where + ".mlp", sizes, ("ff",))
        return sizes

    def validate(self, raw: Mapping[str, Any]) -> None:
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError(f"vocab and width must be positive: {self.vocab}, {self.width}")
        if self.norm_eps <= 0.0:
            raise ConfigError(f"norm.eps must be positive: {self.norm_eps}")
        mixed = None
        for index, layer in enumerate(self.layers):
            sizes = layer.mixer
            if max(sizes.dim, sizes.vdim) > MOST_HEAD:
                raise UnsupportedModelError(f"Model type {self.MODEL_TYPE!r}: layers[{index}] has heads of {sizes.dim} / {sizes.vdim}; "
                                            f"the attention kernels take heads of up to {MOST_HEAD}")
            if sizes.heads * sizes.dim > MOST_WIDTH or sizes.heads > MOST_HEADS:
                raise UnsupportedModelError(f"Model type {self.MODEL_TYPE!r}: layers[{index}] has {sizes.heads} heads of {sizes.dim}; the kernel in "
                                            f"front of attention takes {MOST_WIDTH} numbers in {MOST_HEADS} heads")
            if sizes.v_mix:
                mixed = mixed or sizes.kv_heads * sizes.vdim
                if sizes.kv_heads * sizes.vdim != mixed:
                    raise ConfigError(f"config.json: layers[{index}] mixes {sizes.kv_heads * sizes.vdim} values a token with the {mixed} of the "
                                      "first layer with v_mix")

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
        return {"architecture": self.MODEL_TYPE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "postln_alpha": self.alpha, "layers": [layer.to_dict() for layer in self.layers]}
