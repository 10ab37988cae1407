"""Typed configuration of the Pusazen decoder: layers whose norm sits on the residual sum, with a mixer that is mLSTM, lightning
attention or chunked grouped-query attention with a sink, and a dense squared-relu feed-forward, a mixture of experts or none.

config.json keys: ``architecture`` ("Pusazen"), ``vocab``, ``width``, ``norm.eps``, ``postln_alpha``, ``logit_scale`` and
``layers``, a list with one object per layer: ``type`` ("mlstm", "lightning" or "attention"), ``mixer`` with that mixer's
sizes, and ``mlp`` (``{"kind": "dense", "ff": ...}``, ``{"kind": "moe", ...}`` or null).

``mixer`` of an mLSTM layer: ``heads``, ``dim``, ``vdim``, ``gate_cap``; of a lightning layer: ``heads``, ``dim``, ``vdim``,
``decay`` (one number a head); of an attention layer: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``softcap``,
``rot`` (``base``, ``dims``) and ``mask`` (``size``).  ``mlp`` of kind moe: ``router`` (``experts``, ``top``), ``expert``
(``ff``) and optionally ``shared`` (``ff``).
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, ClassVar

from .base import ConfigError, KeyReader, ModelConfig


def _need_sub(keys: KeyReader, key: str, where: str) -> KeyReader:
    sub = keys.sub(key)
    if sub is None:
        raise ConfigError(f"{where}: required key '{key}' is missing")
    return sub


@dataclass(frozen=True)
class PusazenMLSTM:
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    @classmethod
    def read(cls, keys: KeyReader, where: str) -> "PusazenMLSTM":
        dim = keys.integer("dim", minimum=1)
        return cls(heads=keys.integer("heads", minimum=1), dim=dim, vdim=keys.integer("vdim", dim, minimum=1),
                   gate_cap=keys.number("gate_cap", positive=True))

    def check(self, where: str) -> None:
        pass

    def to_dict(self) -> dict[str, Any]:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "gate_cap": self.gate_cap}


@dataclass(frozen=True)
class PusazenLightning:
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]

    @classmethod
    def read(cls, keys: KeyReader, where: str) -> "PusazenLightning":
        decay = keys.raw("decay")
        if not isinstance(decay, list) or any(isinstance(d, bool) or not isinstance(d, (int, float)) for d in decay):
            raise ConfigError(f"{where}: 'decay' must be a list of numbers, got {decay!r}")
        dim = keys.integer("dim", minimum=1)
        out = cls(heads=keys.integer("heads", minimum=1), dim=dim, vdim=keys.integer("vdim", dim, minimum=1),
                  decay=tuple(float(d) for d in decay))
        out.check(where)
        return out

    def check(self, where: str) -> None:
        if len(self.decay) != self.heads:
            raise ConfigError(f"{where}: 'decay' must hold one number for each of the {self.heads} heads, got {len(self.decay)}")

    def to_dict(self) -> dict[str, Any]:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}


@dataclass(frozen=True)
class PusazenAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float | None = None
    rot_base: float | None = None       # None: no rotation
    rot_dims: int = 0
    chunk: int | None = None            # None: every earlier key is seen

    @classmethod
    def read(cls, keys: KeyReader, where: str) -> "PusazenAttention":
        heads, dim = keys.integer("heads", minimum=1), keys.integer("dim", minimum=1)
        rot, mask = keys.sub("rot"), keys.sub("mask")
        out = cls(heads=heads, kv_heads=keys.integer("kv_heads", heads, minimum=1), dim=dim,
                  vdim=keys.integer("vdim", dim, minimum=1), scale=keys.number("scale", dim ** -0.5, positive=True),
                  softcap=keys.number("softcap", positive=True) if keys.has("softcap") else None,
                  rot_base=rot.number("base", positive=True) if rot is not None else None,
                  rot_dims=rot.integer("dims", minimum=2) if rot is not None else 0,
                  chunk=mask.integer("size", minimum=1) if mask is not None else None)
        out.check(where)
        return out

    def check(self, where: str) -> None:
        if self.heads % self.kv_heads:
            raise ConfigError(f"{where}: 'heads' ({self.heads}) must be a multiple of 'kv_heads' ({self.kv_heads})")
        if self.rot_base is not None and (self.rot_dims % 2 or not 0 < self.rot_dims <= self.dim):
            raise ConfigError(f"{where}: 'rot.dims' ({self.rot_dims}) must be even and within the {self.dim} channels of a head")

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim,
                               "scale": self.scale}
        if self.softcap is not None:
            out["softcap"] = self.softcap
        if self.rot_base is not None:
            out["rot"] = {"base": self.rot_base, "dims": self.rot_dims}
        if self.chunk is not None:
            out["mask"] = {"size": self.chunk}
        return out


@dataclass(frozen=True)
class PusazenDense:
    ff: int

    def check(self, where: str) -> None:
        pass

    def to_dict(self) -> dict[str, Any]:
        return {"kind": "dense", "ff": self.ff}


@dataclass(frozen=True)
class PusazenExperts:
    experts: int
    top: int
    ff: int
    shared_ff: int | None = None

    def check(self, where: str) -> None:
        if self.top > self.experts:
            raise ConfigError(f"{where}: 'top' ({self.top}) is more than the {self.experts} experts")

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"kind": "moe", "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff is not None:
            out["shared"] = {"ff": self.shared_ff}
        return out


def _read_mlp(keys: KeyReader, where: str) -> "PusazenDense | PusazenExperts":
    kind = keys.string("kind", "dense")
    if kind == "dense":
        return PusazenDense(ff=keys.integer("ff", minimum=1))
    if kind != "moe":
        raise ConfigError(f"{where}: 'kind' must be 'dense' or 'moe', got {kind!r}")
    router, expert, shared = _need_sub(keys, "router", where), _need_sub(keys, "expert", where), keys.sub("shared")
    out = PusazenExperts(experts=router.integer("experts", minimum=1), top=router.integer("top", minimum=1),
                         ff=expert.integer("ff", minimum=1),
                         shared_ff=shared.integer("ff", minimum=1) if shared is not None else None)
    out.check(where)
    return out


MIXERS = {"mlstm": PusazenMLSTM, "lightning": PusazenLightning, "attention": PusazenAttention}


@dataclass(frozen=True)
class PusazenLayer:
    type: str
    mixer: "PusazenMLSTM | PusazenLightning | PusazenAttention"
    mlp: "PusazenDense | PusazenExperts | None" = None

    def to_dict(self) -> dict[str, Any]:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass(frozen=True)
class PusazenConfig(ModelConfig):
    architecture: ClassVar[str] = "Pusazen"

    vocab: int
    width: int
    layers: tuple[PusazenLayer, ...]
    norm_eps: float = 1e-6
    alpha: float = 1.0
    logit_scale: float = 1.0

    def __post_init__(self) -> None:
        if self.vocab < 1 or self.width < 1 or not self.layers:
            raise ConfigError("config.json: 'vocab' and 'width' must be >= 1 and 'layers' must not be empty")
        object.__setattr__(self, "layers", tuple(self.layers))
        for index, layer in enumerate(self.layers):
            where = f"config.json:layers[{index}]"
            if layer.type not in MIXERS:
                raise ConfigError(f"{where}: 'type' must be one of {tuple(MIXERS)}, got {layer.type!r}")
            if not isinstance(layer.mixer, MIXERS[layer.type]):
                raise ConfigError(f"{where}: the mixer's sizes do not belong to a layer of type {layer.type!r}")
            layer.mixer.check(where + ":mixer")
            if layer.mlp is not None:
                layer.mlp.check(where + ":mlp")

    @classmethod
    def from_dict(cls, data: dict[str, Any]) -> "PusazenConfig":
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
            layers.append(PusazenLayer(type=kind, mixer=mixer, mlp=None if mlp is None else _read_mlp(mlp, where + ":mlp")))
        norm = keys.sub("norm")
        return cls(vocab=keys.integer("vocab", minimum=1), width=keys.integer("width", minimum=1), layers=tuple(layers),
                   norm_eps=norm.number("eps", 1e-6, positive=True) if norm else 1e-6,
                   alpha=keys.number("postln_alpha", 1.0), logit_scale=keys.number("logit_scale", 1.0))

    def to_dict(self) -> dict[str, Any]:
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "postln_alpha": self.alpha, "logit_scale": self.logit_scale, "layers": [layer.to_dict() for layer in self.layers]}
