"""Typed configuration of the Tomopel decoder: pre-norm layers around several residual streams (hyper-connections) with
a scaled residual add, whose mixer is either two mixers side by side (grouped-query attention with a learned distance
bias beside Mamba-2) or a minGRU, with a dense gated feed-forward or a mixture of ungated experts.

config.json keys: ``architecture`` ("Tomopel"), ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``,
``residual_mult``, ``streams`` (absent, with no ``hc*`` tensors in the checkpoint: the plain residual sum) and
``layers``, a list with one object per layer: ``type`` ("parallel" or "mingru"), ``mixer`` with that mixer's sizes, and
``mlp`` (``{"kind": "dense", "ff": ...}``, ``{"kind": "moe", ...}`` or null).

``mixer`` of a parallel layer: ``left`` (``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``bias_max``, optional
``q_temp`` with ``coef`` and ``every``, and optionally ``buckets``, the rows of the bias table, which is otherwise what the
checkpoint's table has), ``right`` (``heads``, ``vdim``, ``state``, ``groups``, ``conv``, ``norm_groups``), ``left_scale``
and ``right_scale``.  ``mixer`` of a minGRU layer: ``width``.  ``mlp`` of kind moe: ``router`` (``experts``, ``top``),
``expert`` (``ff``) and optionally ``shared`` (``ff``).
"""

from __future__ import annotations

import dataclasses
from dataclasses import dataclass
from typing import Any, ClassVar

from .base import ConfigError, KeyReader, ModelConfig


def _need_sub(keys: KeyReader, key: str, where: str) -> KeyReader:
    sub = keys.sub(key)
    if sub is None:
        raise ConfigError(f"{where}: required key '{key}' is missing")
    return sub


@dataclass(frozen=True)
class TomopelAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: int
    temp_coef: float | None = None
    temp_every: int = 1
    buckets: int | None = None       # None: what the checkpoint's table has

    @classmethod
    def read(cls, keys: KeyReader, where: str) -> "TomopelAttention":
        heads, dim = keys.integer("heads", minimum=1), keys.integer("dim", minimum=1)
        temp = keys.sub("q_temp")
        out = cls(heads=heads, kv_heads=keys.integer("kv_heads", heads, minimum=1), dim=dim,
                  vdim=keys.integer("vdim", dim, minimum=1), scale=keys.number("scale", dim ** -0.5, positive=True),
                  bias_max=keys.integer("bias_max", minimum=2),
                  temp_coef=temp.number("coef") if temp is not None else None,
                  temp_every=temp.integer("every", minimum=1) if temp is not None else 1,
                  buckets=keys.optional_integer("buckets", minimum=2))
        out.check(where)
        return out

    def check(self, where: str) -> None:
        if self.heads % self.kv_heads:
            raise ConfigError(f"{where}: 'heads' ({self.heads}) must be a multiple of 'kv_heads' ({self.kv_heads})")
        if self.buckets is not None and self.bias_max <= self.buckets // 2:
            raise ConfigError(f"{where}: 'bias_max' ({self.bias_max}) must lie beyond half of the {self.buckets} buckets")

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim,
                               "scale": self.scale, "bias_max": self.bias_max}
        if self.temp_coef is not None:
            out["q_temp"] = {"coef": self.temp_coef, "every": self.temp_every}
        if self.buckets is not None:
            out["buckets"] = self.buckets
        return out


@dataclass(frozen=True)
class TomopelMamba2:
    heads: int
    vdim: int
    state: int
    groups: int = 1
    conv: int = 4
    norm_groups: int = 1

    @classmethod
    def read(cls, keys: KeyReader, where: str) -> "TomopelMamba2":
        out = cls(heads=keys.integer("heads", minimum=1), vdim=keys.integer("vdim", minimum=1),
                  state=keys.integer("state", minimum=1), groups=keys.integer("groups", 1, minimum=1),
                  conv=keys.integer("conv", minimum=1), norm_groups=keys.integer("norm_groups", 1, minimum=1))
        out.check(where)
        return out

    def check(self, where: str) -> None:
        if self.heads % self.groups:
            raise ConfigError(f"{where}: 'heads' ({self.heads}) must be a multiple of 'groups' ({self.groups})")
        if (self.heads * self.vdim) % self.norm_groups:
            raise ConfigError(f"{where}: 'norm_groups' ({self.norm_groups}) must divide the {self.heads * self.vdim} inner channels")

    def to_dict(self) -> dict[str, Any]:
        return {"heads": self.heads, "vdim": self.vdim, "state": self.state, "groups": self.groups, "conv": self.conv,
                "norm_groups": self.norm_groups}


@dataclass(frozen=True)
class TomopelParallel:
    left: TomopelAttention
    right: TomopelMamba2
    left_scale: float = 1.0
    right_scale: float = 1.0

    @classmethod
    def read(cls, keys: KeyReader, where: str) -> "TomopelParallel":
        left, right = _need_sub(keys, "left", where), _need_sub(keys, "right", where)
        return cls(left=TomopelAttention.read(left, where + ":left"), right=TomopelMamba2.read(right, where + ":right"),
                   left_scale=keys.number("left_scale", 1.0), right_scale=keys.number("right_scale", 1.0))

    def check(self, where: str) -> None:
        self.left.check(where + ":left")
        self.right.check(where + ":right")

    def to_dict(self) -> dict[str, Any]:
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale,
                "right_scale": self.right_scale}


@dataclass(frozen=True)
class TomopelMinGRU:
    width: int

    @classmethod
    def read(cls, keys: KeyReader, where: str) -> "TomopelMinGRU":
        return cls(width=keys.integer("width", minimum=1))

    def check(self, where: str) -> None:
        pass

    def to_dict(self) -> dict[str, Any]:
        return {"width": self.width}


@dataclass(frozen=True)
class TomopelDense:
    ff: int

    def to_dict(self) -> dict[str, Any]:
        return {"kind": "dense", "ff": self.ff}


@dataclass(frozen=True)
class TomopelExperts:
    experts: int
    top: int
    ff: int
    shared_ff: int | None = None

    def check(self, where: str) -> None:
        if self.top > self.experts:
            raise ConfigError(f"{where}: 'top' ({self.top}) is more than the {self.experts} experts")

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"kind": "moe", "expert": {"ff": self.ff},
                               "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff is not None:
            out["shared"] = {"ff": self.shared_ff}
        return out


def _read_mlp(keys: KeyReader, where: str) -> "TomopelDense | TomopelExperts":
    kind = keys.string("kind", "dense")
    if kind == "dense":
        return TomopelDense(ff=keys.integer("ff", minimum=1))
    if kind != "moe":
        raise ConfigError(f"{where}: 'kind' must be 'dense' or 'moe', got {kind!r}")
    router, expert, shared = _need_sub(keys, "router", where), _need_sub(keys, "expert", where), keys.sub("shared")
    out = TomopelExperts(experts=router.integer("experts", minimum=1), top=router.integer("top", minimum=1),
                         ff=expert.integer("ff", minimum=1),
                         shared_ff=shared.integer("ff", minimum=1) if shared is not None else None)
    out.check(where)
    return out


MIXERS = {"parallel": TomopelParallel, "mingru": TomopelMinGRU}


@dataclass(frozen=True)
class TomopelLayer:
    type: str
    mixer: "TomopelParallel | TomopelMinGRU"
    mlp: "TomopelDense | TomopelExperts | None" = None

    def to_dict(self) -> dict[str, Any]:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass(frozen=True)
class TomopelConfig(ModelConfig):
    architecture: ClassVar[str] = "Tomopel"

    vocab: int
    width: int
    layers: tuple[TomopelLayer, ...]
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    residual_mult: float = 1.0
    streams: int | None = None       # None: one stream and the plain residual sum (no connection tensors)

    def __post_init__(self) -> None:
        if self.vocab < 1 or self.width < 1 or not self.layers:
            raise ConfigError("config.json: 'vocab' and 'width' must be >= 1 and 'layers' must not be empty")
        if self.streams is not None and self.streams < 1:
            raise ConfigError(f"config.json: 'streams' must be >= 1, got {self.streams}")
        object.__setattr__(self, "layers", tuple(self.layers))
        for index, layer in enumerate(self.layers):
            where = f"config.json:layers[{index}]"
            if layer.type not in MIXERS:
                raise ConfigError(f"{where}: 'type' must be one of {tuple(MIXERS)}, got {layer.type!r}")
            if not isinstance(layer.mixer, MIXERS[layer.type]):
                raise ConfigError(f"{where}: the mixer's sizes do not belong to a layer of type {layer.type!r}")
            layer.mixer.check(where + ":mixer")
            if isinstance(layer.mlp, TomopelExperts):
                layer.mlp.check(where + ":mlp")

    def fitted_to(self, shapes: dict[str, tuple[int, ...]]) -> "TomopelConfig":
        """What config.json leaves to the checkpoint: the rows of each layer's bias table, and, where config.json says
        one stream or nothing, whether the layers have connection tensors."""
        layers = []
        for index, layer in enumerate(self.layers):
            shape = shapes.get(f"l{index}.mix.left.rel")
            if layer.type == "parallel" and layer.mixer.left.buckets is None and shape is not None and len(shape) == 2:
                left = dataclasses.replace(layer.mixer.left, buckets=int(shape[0]))
                layer = dataclasses.replace(layer, mixer=dataclasses.replace(layer.mixer, left=left))
            layers.append(layer)
        streams = self.streams
        connected = any(".hc1." in name for name in shapes)
        if streams == 1 and not connected:
            streams = None
        elif streams is None and connected:
            streams = int(next(shape[0] for name, shape in shapes.items() if name.endswith(".hc1.in")))
        return dataclasses.replace(self, layers=tuple(layers), streams=streams)

    @classmethod
    def from_dict(cls, data: dict[str, Any]) -> "TomopelConfig":
        keys = KeyReader(data)
        raw_layers = keys.raw("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        layers = []
        for index, raw in enumerate(raw_layers):
            where = f"config.json:layers[{index}]"
            layer = KeyReader(raw, where)
            kind = layer.string("type")
            if kind not in MIXERS:
                raise ConfigError(f"{where}: 'type' must be one of {tuple(MIXERS)}, got {kind!r}")
            mixer = MIXERS[kind].read(_need_sub(layer, "mixer", where), where + ":mixer")
            mlp = layer.sub("mlp")
            layers.append(TomopelLayer(type=kind, mixer=mixer, mlp=None if mlp is None else _read_mlp(mlp, where + ":mlp")))
        norm, embedding = keys.sub("norm"), keys.sub("embedding")
        return cls(vocab=keys.integer("vocab", minimum=1), width=keys.integer("width", minimum=1), layers=tuple(layers),
                   norm_eps=norm.number("eps", 1e-6, positive=True) if norm else 1e-6,
                   embedding_scale=embedding.number("scale", 1.0) if embedding else 1.0,
                   residual_mult=keys.number("residual_mult", 1.0), streams=keys.optional_integer("streams", minimum=1))

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                               "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale},
                               "residual_mult": self.residual_mult, "layers": [layer.to_dict() for layer in self.layers]}
        if self.streams is not None:
            out["streams"] = self.streams
        return out
