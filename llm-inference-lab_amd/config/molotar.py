"""Typed configuration of the Molotar decoder, read from ``config.json``.

The file lists the layers one by one: each has a ``type`` (which mixer it has), the mixer's sizes and
constants (``mixer``), and its feed-forward (``mlp``, or null for a layer with the mixer only).
``attention``: grouped-query attention through a sliding window, turned by position, perhaps reading an
earlier layer's keys and values (``kv_from``).  ``rglru``: a recurrence of single numbers with block-diagonal
gates behind a short convolution.  Beside them: ``embedding`` (the scale of the token vectors and the
hashed table of token pairs), ``norm.eps``, and ``postln_alpha``, the stream's factor in every sum.
"""
from __future__ import annotations

import dataclasses
import math
from typing import Any, Dict, Optional, Tuple

from .errors import ConfigError
from .qwen2 import _require, _typed


def _object(raw, key: str, at: str, required: bool = True):
    value = raw.get(key)
    if value is None and not required:
        return None
    if not isinstance(value, dict):
        raise ConfigError(f"{at}: key '{key}' must be an object")
    return value


@dataclasses.dataclass(frozen=True)
class MolotarExperts:
    """``experts`` clamped feed-forwards ``ff`` wide of which a token takes ``top``, out of the ``groups_keep`` best
    of ``groups`` groups of neighbours."""

    ff: int
    limit: float
    experts: int
    top: int
    scale: float = 1.0
    groups: int = 1
    groups_keep: int = 1

    @classmethod
    def from_dict(cls, mlp, at: str) -> Optional["MolotarExperts"]:
        if mlp is None:
            return None
        if not isinstance(mlp, dict):
            raise ConfigError(f"{at} is an object or null")
        kind = _typed(mlp.get("kind", "moe"), "kind", str, at)
        if kind != "moe":
            raise ConfigError(f"{at}: unknown feed-forward kind '{kind}' (known: moe)")
        e, r = _object(mlp, "expert", at), _object(mlp, "router", at)
        g = _object(r, "groups", at + ".router", required=False) or dict(count=1, keep=1)
        return cls(ff=_require(e, "ff", int, at + ".expert"), limit=_require(e, "limit", float, at + ".expert"),
                   experts=_require(r, "experts", int, at + ".router"), top=_require(r, "top", int, at + ".router"),
                   scale=_typed(r.get("scale", 1.0), "scale", float, at + ".router"),
                   groups=_require(g, "count", int, at + ".router.groups"),
                   groups_keep=_require(g, "keep", int, at + ".router.groups"))

    def check(self, at: str) -> None:
        if self.ff <= 0 or not (math.isfinite(self.limit) and self.limit > 0):
            raise ConfigError(f"{at}: expert.ff and expert.limit must be positive, got {self.ff} and {self.limit}")
        if not math.isfinite(self.scale):
            raise ConfigError(f"{at}: router.scale must be finite")
        if not 0 < self.top <= self.experts:
            raise ConfigError(f"{at}: a router of {self.experts} experts cannot take the top {self.top}")
        if self.groups <= 0 or self.experts % self.groups or not 0 < self.groups_keep <= self.groups:
            raise ConfigError(f"{at}: {self.experts} experts do not form {self.groups} equal groups of which "
                              f"{self.groups_keep} are kept")
        if self.groups_keep * (self.experts // self.groups) < self.top:
            raise ConfigError(f"{at}: the kept groups hold fewer experts than a token takes")

    def to_dict(self) -> Dict[str, Any]:
        return dict(expert=dict(ff=self.ff, limit=self.limit), kind="moe",
                    router=dict(experts=self.experts, groups=dict(count=self.groups, keep=self.groups_keep), scale=self.scale,
                                top=self.top))


@dataclasses.dataclass(frozen=True)
class MolotarScaling:
    factor: float
    low: float
    high: float
    original: float


@dataclasses.dataclass(frozen=True)
class MolotarRotation:
    dims: int
    base: float
    scaling: Optional[MolotarScaling] = None


@dataclasses.dataclass(frozen=True)
class MolotarAttention:
    """``window`` None: every earlier position is seen.  ``kv_from``: the layer whose keys and values are read."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None
    rot: Optional[MolotarRotation] = None
    kv_from: Optional[int] = None

    @classmethod
    def from_dict(cls, m, at: str) -> "MolotarAttention":
        heads, dim = _require(m, "heads", int, at), _require(m, "dim", int, at)
        rot, mask = _object(m, "rot", at, required=False), _object(m, "mask", at, required=False)
        if rot is not None:
            sc = _object(rot, "scaling", at + ".rot", required=False)
            if sc is not None:
                sc = MolotarScaling(*(_require(sc, k, float, at + ".rot.scaling") for k in ("factor", "low", "high", "original")))
            rot = MolotarRotation(_require(rot, "dims", int, at + ".rot"), _require(rot, "base", float, at + ".rot"), sc)
        optional = lambda raw, key: None if raw.get(key) is None else _typed(raw[key], key, int, at)
        kv_heads, vdim = optional(m, "kv_heads"), optional(m, "vdim")
        return cls(heads=heads, kv_heads=heads if kv_heads is None else kv_heads, dim=dim,
                   vdim=dim if vdim is None else vdim, scale=_require(m, "scale", float, at),
                   window=optional(mask or {}, "size"), rot=rot, kv_from=optional(m, "kv_from"))

    def check(self, at: str) -> None:
        if min(self.heads, self.kv_heads, self.dim, self.vdim) <= 0:
            raise ConfigError(f"{at}: heads, kv_heads, dim and vdim must be positive")
        if self.heads % self.kv_heads:
            raise ConfigError(f"{at}: heads {self.heads} is not a multiple of kv_heads {self.kv_heads}")
        if not math.isfinite(self.scale):
            raise ConfigError(f"{at}: scale must be finite")
        if self.window is not None and self.window <= 0:
            raise ConfigError(f"{at}: mask.size must be positive, got {self.window}")
        r = self.rot
        if r is None:
            return
        if r.dims < 0 or r.dims % 2 or r.dims > self.dim:
            raise ConfigError(f"{at}: rot.dims {r.dims} must be even and at most the head's {self.dim} channels")
        if not (math.isfinite(r.base) and r.base > 0.0):
            raise ConfigError(f"{at}: rot.base must be finite and > 0, got {r.base}")
        s = r.scaling
        if s is not None and not (all(math.isfinite(v) and v > 0 for v in dataclasses.astuple(s)) and s.low <= s.high):
            raise ConfigError(f"{at}: rot.scaling needs positive numbers with low <= high, got {s}")

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = dict(dim=self.dim, heads=self.heads, kv_heads=self.kv_heads, scale=self.scale, vdim=self.vdim)
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        if self.window is not None:
            out["mask"] = dict(size=self.window)
        if self.rot is not None:
            out["rot"] = dict(base=self.rot.base, dims=self.rot.dims)
            if self.rot.scaling is not None:
                out["rot"]["scaling"] = dataclasses.asdict(self.rot.scaling)
        return out


@dataclasses.dataclass(frozen=True)
class MolotarRecurrence:
    """``width`` channels in ``blocks`` parts, behind a convolution of ``conv`` taps."""

    width: int
    blocks: int
    conv: int

    @classmethod
    def from_dict(cls, m, at: str) -> "MolotarRecurrence":
        return cls(*(_require(m, k, int, at) for k in ("width", "blocks", "conv")))

    def check(self, at: str) -> None:
        if min(self.width, self.blocks, self.conv) <= 0 or self.width % self.blocks:
            raise ConfigError(f"{at}: width, blocks and conv must be positive and the width {self.width} a multiple of the "
                              f"{self.blocks} blocks")

    def to_dict(self) -> Dict[str, Any]:
        return dataclasses.asdict(self)


@dataclasses.dataclass(frozen=True)
class MolotarLayer:
    """``type`` "attention" or "rglru"; ``mixer`` of the matching class."""

    type: str
    mixer: Any
    mlp: Optional[MolotarExperts] = None


@dataclasses.dataclass(frozen=True)
class MolotarBigram:
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclasses.dataclass(frozen=True)
class MolotarConfig:
    vocab: int
    width: int
    norm_eps: float
    alpha: float
    layers: Tuple[MolotarLayer, ...]
    embedding_scale: float = 1.0
    bigram: Optional[MolotarBigram] = None
    eos_token_ids: Tuple[int, ...] = ()
    architecture: str = "Molotar"

    ARCHITECTURE = "Molotar"
    MAX_POSITIONS = 1 << 20          # the design has no position table: the engine's own bound
    MIXERS = {"attention": MolotarAttention, "rglru": MolotarRecurrence}

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], where: str = "config.json") -> "MolotarConfig":
        name = raw.get("architecture", (raw.get("architectures") or [cls.ARCHITECTURE])[0])
        if name != cls.ARCHITECTURE:
            raise ConfigError(f"{where}: architecture must be '{cls.ARCHITECTURE}', got {name!r}")
        norm = _object(raw, "norm", where)
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError(f"{where}: key 'layers' must be a non-empty list")
        layers = []
        for i, entry in enumerate(listed):
            at = f"{where}: layers[{i}]"
            if not isinstance(entry, dict):
                raise ConfigError(f"{at} must be an object with 'type' and 'mixer'")
            kind, m = _require(entry, "type", str, at), _object(entry, "mixer", at)
            if kind not in cls.MIXERS:
                raise ConfigError(f"{at}: unknown layer type '{kind}' (known: {', '.join(sorted(cls.MIXERS))})")
            layers.append(MolotarLayer(kind, cls.MIXERS[kind].from_dict(m, at + ".mixer"),
                                       MolotarExperts.from_dict(entry.get("mlp"), at + ".mlp")))
        emb = _object(raw, "embedding", where, required=False) or {}
        big = _object(emb, "bigram", where + ": embedding", required=False)
        if big is not None:
            big = MolotarBigram(*(_require(big, k, int, where + ": embedding.bigram")
                                  for k in ("buckets", "mul_prev", "mul_cur")))
        eos = raw.get("eos_token_id")
        eos_ids = () if eos is None else tuple(_typed(e, "eos_token_id", int, where)
                                               for e in (eos if isinstance(eos, list) else [eos]))
        cfg = cls(vocab=_require(raw, "vocab", int, where), width=_require(raw, "width", int, where),
                  norm_eps=_require(norm, "eps", float, where + ": norm"),
                  alpha=_require(raw, "postln_alpha", float, where), layers=tuple(layers),
                  embedding_scale=_typed(emb.get("scale", 1.0), "scale", float, where + ": embedding"), bigram=big,
                  eos_token_ids=eos_ids)
        cfg.validate(where)
        return cfg

    def validate(self, where: str = "config") -> None:
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError(f"{where}: 'vocab' and 'width' must be positive")
        if not (math.isfinite(self.norm_eps) and self.norm_eps > 0):
            raise ConfigError(f"{where}: norm.eps must be finite and > 0, got {self.norm_eps}")
        if not (math.isfinite(self.alpha) and math.isfinite(self.embedding_scale)):
            raise ConfigError(f"{where}: postln_alpha and embedding.scale must be finite")
        if self.bigram is not None and (self.bigram.buckets <= 0 or self.bigram.mul_prev < 0 or self.bigram.mul_cur < 0):
            raise ConfigError(f"{where}: embedding.bigram needs buckets > 0 and multipliers >= 0")
        for i, l in enumerate(self.layers):
            at = f"{where}: layers[{i}]"
            l.mixer.check(at + ".mixer")
            if l.mlp is not None:
                l.mlp.check(at + ".mlp")
            source = getattr(l.mixer, "kv_from", None)
            if source is None:
                continue
            if not 0 <= source < i or self.layers[source].type != "attention" or self.layers[source].mixer.kv_from is not None:
                raise ConfigError(f"{at}: kv_from {source} must name an earlier attention layer with keys and values of its own")
            s, m = self.layers[source].mixer, l.mixer
            if (s.kv_heads, s.dim, s.vdim) != (m.kv_heads, m.dim, m.vdim):
                raise ConfigError(f"{at}: kv_heads, dim and vdim must equal those of layer {source}, whose keys and values it reads")
        for e in self.eos_token_ids:
            if not 0 <= e < self.vocab:
                raise ConfigError(f"{where}: eos_token_id {e} is outside the vocabulary")

    def to_dict(self) -> Dict[str, Any]:
        emb: Dict[str, Any] = dict(scale=self.embedding_scale)
        if self.bigram is not None:
            emb["bigram"] = dataclasses.asdict(self.bigram)
        layers = [dict(type=l.type, mixer=l.mixer.to_dict(), mlp=None if l.mlp is None else l.mlp.to_dict()) for l in self.layers]
        out: Dict[str, Any] = dict(architecture=self.architecture, embedding=emb, layers=layers, norm=dict(eps=self.norm_eps),
                                   postln_alpha=self.alpha, vocab=self.vocab, width=self.width)
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out
