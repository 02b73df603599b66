"""Typed configuration of the Mazanex decoder, read from ``config.json``.

The file lists the layers one by one: each has a ``type`` (which mixer it has), the mixer's sizes
and constants (``mixer``), and its feed-forward (``mlp``, or null for a layer with the mixer only).
``mlstm``: a matrix memory with exponential gates.  ``gla``: linear attention with a decay per key
channel.  ``parallel``: a pair of mixers on one input, a ``left`` one (attention over chunks of positions
with a sink, short convolutions and a gate per channel) and a ``right`` one (a recurrent state whose
projections read mixes of the current and the previous token), each normed, half the sum of both.
Sizes that the file does not name (the ranks of the decay projections) are read off the tensors'
shapes when the weights are loaded.
"""
from __future__ import annotations

import dataclasses
import math
from typing import Any, Dict, Optional, Tuple

from .errors import ConfigError
from .qwen2 import _require, _typed


@dataclasses.dataclass(frozen=True)
class MazanexFeedForward:
    kind: str
    ff: int


@dataclasses.dataclass(frozen=True)
class MazanexRotation:
    dims: int
    base: float


@dataclasses.dataclass(frozen=True)
class MazanexAttention:
    """The ``left`` half of a ``parallel`` layer.  ``chunk`` None: every earlier position is seen."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    conv: int
    rot: Optional[MazanexRotation] = None
    chunk: Optional[int] = None

    @classmethod
    def from_dict(cls, m, at: str) -> "MazanexAttention":
        if not isinstance(m, dict):
            raise ConfigError(f"{at} must be an object")
        heads = _require(m, "heads", int, at)
        kv_heads, rot, mask = m.get("kv_heads"), m.get("rot"), m.get("mask")
        for value, name in ((rot, "rot"), (mask, "mask")):
            if value is not None and not isinstance(value, dict):
                raise ConfigError(f"{at}: '{name}' is an object")
        if rot is not None:
            rot = MazanexRotation(_require(rot, "dims", int, at + ".rot"), _require(rot, "base", float, at + ".rot"))
        chunk = (mask or {}).get("size")
        return cls(heads=heads, kv_heads=heads if kv_heads is None else _typed(kv_heads, "kv_heads", int, at),
                   dim=_require(m, "dim", int, at), vdim=_require(m, "vdim", int, at),
                   scale=_require(m, "scale", float, at), conv=_typed(m.get("conv", 0), "conv", int, at), rot=rot,
                   chunk=None if chunk is None else _typed(chunk, "mask.size", int, at))

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = dict(conv=self.conv, dim=self.dim, heads=self.heads, kv_heads=self.kv_heads, scale=self.scale,
                                   vdim=self.vdim)
        if self.rot is not None:
            out["rot"] = dict(base=self.rot.base, dims=self.rot.dims)
        if self.chunk is not None:
            out["mask"] = dict(size=self.chunk)
        return out

    def check(self, at: str) -> None:
        if min(self.heads, self.kv_heads, self.dim, self.vdim) <= 0:
            raise ConfigError(f"{at}: heads, kv_heads, dim and vdim must be positive")
        if self.heads % self.kv_heads:
            raise ConfigError(f"{at}: heads {self.heads} is not a multiple of kv_heads {self.kv_heads}")
        if not math.isfinite(self.scale):
            raise ConfigError(f"{at}: scale must be finite")
        if self.conv < 0:
            raise ConfigError(f"{at}: conv counts taps, got {self.conv}")
        if self.chunk is not None and self.chunk <= 0:
            raise ConfigError(f"{at}: mask.size must be positive, got {self.chunk}")
        if self.rot is not None:
            if self.rot.dims < 0 or self.rot.dims % 2 or self.rot.dims > self.dim:
                raise ConfigError(f"{at}: rot.dims {self.rot.dims} must be even and at most the head's {self.dim} channels")
            if not (math.isfinite(self.rot.base) and self.rot.base > 0.0):
                raise ConfigError(f"{at}: rot.base must be finite and > 0, got {self.rot.base}")


@dataclasses.dataclass(frozen=True)
class MazanexRecurrent:
    """Sizes of a recurrent mixer: ``gla`` (``tau``), ``mlstm`` (``gate_cap``), or the ``right`` half of a
    ``parallel`` layer (``vdim`` is its ``dim``)."""

    heads: int
    dim: int
    vdim: int
    tau: Optional[float] = None
    gate_cap: Optional[float] = None

    def check(self, at: str) -> None:
        if min(self.heads, self.dim, self.vdim) <= 0:
            raise ConfigError(f"{at}: heads, dim and vdim must be positive")
        for value, name in ((self.tau, "tau"), (self.gate_cap, "gate_cap")):
            if value is not None and not (math.isfinite(value) and value > 0.0):
                raise ConfigError(f"{at}: {name} must be finite and > 0, got {value}")


@dataclasses.dataclass(frozen=True)
class MazanexLayer:
    """``type`` "gla" or "mlstm": ``recurrent``.  ``type`` "parallel": ``left`` and ``right``."""

    type: str
    mlp: Optional[MazanexFeedForward] = None
    recurrent: Optional[MazanexRecurrent] = None
    left: Optional[MazanexAttention] = None
    right: Optional[MazanexRecurrent] = None


@dataclasses.dataclass(frozen=True)
class MazanexConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[MazanexLayer, ...]
    eos_token_ids: Tuple[int, ...] = ()
    architecture: str = "Mazanex"

    ARCHITECTURE = "Mazanex"
    MAX_POSITIONS = 1 << 20          # the design has no position table: the engine's own bound
    DEFAULT_DECAY_RANK = 16          # random-weights mode: the configuration names no rank

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], where: str = "config.json") -> "MazanexConfig":
        name = raw.get("architecture", (raw.get("architectures") or [cls.ARCHITECTURE])[0])
        if name != cls.ARCHITECTURE:
            raise ConfigError(f"{where}: architecture must be '{cls.ARCHITECTURE}', got {name!r}")
        norm = raw.get("norm")
        if not isinstance(norm, dict):
            raise ConfigError(f"{where}: required key 'norm' (with 'eps') is missing")
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError(f"{where}: key 'layers' must be a non-empty list")
        layers = []
        for i, entry in enumerate(listed):
            at = f"{where}: layers[{i}]"
            if not isinstance(entry, dict) or not isinstance(entry.get("mixer"), dict):
                raise ConfigError(f"{at} must be an object with 'type' and 'mixer'")
            kind, m = _require(entry, "type", str, at), entry["mixer"]
            mlp = entry.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, dict):
                    raise ConfigError(f"{at}: 'mlp' is an object or null")
                mlp = MazanexFeedForward(_typed(mlp.get("kind", "dense"), "mlp.kind", str, at),
                                         _require(mlp, "ff", int, at + ".mlp"))
            sizes = lambda r, where_: dict(heads=_require(r, "heads", int, where_), dim=_require(r, "dim", int, where_))
            if kind == "gla":
                layers.append(MazanexLayer(kind, mlp, recurrent=MazanexRecurrent(
                    vdim=_require(m, "vdim", int, at), tau=_require(m, "tau", float, at), **sizes(m, at))))
            elif kind == "mlstm":
                layers.append(MazanexLayer(kind, mlp, recurrent=MazanexRecurrent(
                    vdim=_require(m, "vdim", int, at), gate_cap=_require(m, "gate_cap", float, at), **sizes(m, at))))
            elif kind == "parallel":
                right = m.get("right")
                if not isinstance(right, dict):
                    raise ConfigError(f"{at}: 'mixer.right' must be an object")
                dims = sizes(right, at + ".right")
                layers.append(MazanexLayer(kind, mlp, left=MazanexAttention.from_dict(m.get("left"), at + ".left"),
                                           right=MazanexRecurrent(vdim=dims["dim"], **dims)))
            else:
                raise ConfigError(f"{at}: unknown layer type '{kind}' (known: gla, mlstm, parallel)")
        eos = raw.get("eos_token_id")
        eos_ids = () if eos is None else tuple(_typed(e, "eos_token_id", int, where)
                                               for e in (eos if isinstance(eos, list) else [eos]))
        cfg = cls(vocab=_require(raw, "vocab", int, where), width=_require(raw, "width", int, where),
                  norm_eps=_require(norm, "eps", float, where + ": norm"), layers=tuple(layers),
                  eos_token_ids=eos_ids)
        cfg.validate(where)
        return cfg

    def validate(self, where: str = "config") -> None:
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError(f"{where}: 'vocab' and 'width' must be positive")
        if not (math.isfinite(self.norm_eps) and self.norm_eps > 0):
            raise ConfigError(f"{where}: norm.eps must be finite and > 0, got {self.norm_eps}")
        for i, l in enumerate(self.layers):
            at = f"{where}: layers[{i}]"
            if l.mlp is not None and (l.mlp.kind != "dense" or l.mlp.ff <= 0):
                raise ConfigError(f"{at}: the feed-forward is of kind 'dense' with a positive 'ff', got {l.mlp}")
            if l.type == "parallel":
                l.left.check(at + ".left")
                l.right.check(at + ".right")
            else:
                l.recurrent.check(at)
        for e in self.eos_token_ids:
            if not 0 <= e < self.vocab:
                raise ConfigError(f"{where}: eos_token_id {e} is outside the vocabulary")

    def to_dict(self) -> Dict[str, Any]:
        layers = []
        for l in self.layers:
            if l.type == "parallel":
                mixer = dict(left=l.left.to_dict(), right=dict(dim=l.right.dim, heads=l.right.heads))
            else:
                mixer = {k: v for k, v in dataclasses.asdict(l.recurrent).items() if v is not None}
            layers.append(dict(type=l.type, mixer=mixer,
                               mlp=None if l.mlp is None else dict(ff=l.mlp.ff, kind=l.mlp.kind)))
        out: Dict[str, Any] = dict(architecture=self.architecture, layers=layers, norm=dict(eps=self.norm_eps),
                                   vocab=self.vocab, width=self.width)
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out
