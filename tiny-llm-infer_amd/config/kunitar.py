"""Typed configuration of the Kunitar decoder, read from its config.json.

Keys: ``architecture`` ("Kunitar"), ``vocab``, ``width``, ``embedding.scale``, ``norm.eps``,
``token_side.dim`` (of a token's own vector a layer), ``max_positions`` (optional: the design itself
sets no limit) and ``layers``: a list with one entry a layer, ``{"type": "latent_attention" | "wkv",
"mixer": {...}, "mlp": {...} or null}``.

A latent mixer gives ``heads``, ``dim`` and ``rot_dim`` (the parts of a query/key head that are not and
that are turned), ``vdim``, ``kv_rank`` and ``q_rank`` (of the latent vectors), ``scale``, ``mask.size`` (a row
sees itself and the size - 1 positions before it), ``rot.base``, ``rot.dims`` (equal to ``rot_dim``), and
optionally ``kv_from``: j, the layer whose cached vectors it reads instead of making its own.  A wkv mixer
gives ``heads`` and ``dim``, and optionally ``decay_rank``, the inner size of its decay's two matrices for
random weights (a checkpoint's own shapes say it otherwise).  A feed-forward gives ``kind``: "dense" with
``ff``, or "moe" with ``expert.ff``, ``router.experts|top`` and optionally ``shared.ff``.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple, Union

from .base import ConfigError, JsonReader

ARCHITECTURE = "Kunitar"
NO_POSITION_LIMIT = 1 << 20          # what a config.json without ``max_positions`` is taken to allow
DECAY_RANK = 64                      # of random weights, where the configuration does not say


@dataclass(frozen=True)
class KunitarLatent:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    scale: float
    window: Optional[int]            # None: every earlier position is seen
    rot_base: float
    kv_from: Optional[int] = None    # None: a layer with latent vectors of its own

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim,
                               "kv_rank": self.kv_rank, "q_rank": self.q_rank, "scale": self.scale,
                               "rot": {"dims": self.rot_dim, "base": self.rot_base}}
        if self.window is not None:
            out["mask"] = {"size": self.window}
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass(frozen=True)
class KunitarTimeMix:
    heads: int
    dim: int
    decay_rank: Optional[int] = None

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"heads": self.heads, "dim": self.dim}
        if self.decay_rank is not None:
            out["decay_rank"] = self.decay_rank
        return out


@dataclass(frozen=True)
class KunitarDense:
    ff: int

    def to_dict(self) -> Dict[str, Any]:
        return {"kind": "dense", "ff": self.ff}


@dataclass(frozen=True)
class KunitarExperts:
    experts: int
    top: int
    ff: int
    shared_ff: Optional[int]         # None: no shared expert

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"kind": "moe", "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff is not None:
            out["shared"] = {"ff": self.shared_ff}
        return out


@dataclass(frozen=True)
class KunitarLayer:
    kind: str                                        # "latent_attention" or "wkv"
    mixer: Union[KunitarLatent, KunitarTimeMix]
    mlp: Optional[Union[KunitarDense, KunitarExperts]]

    def to_dict(self) -> Dict[str, Any]:
        return {"type": self.kind, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


def _part(r: JsonReader, key: str, where: str) -> JsonReader:
    return JsonReader(r.raw(key) or {}, f"{where}.{key}")


def _positive(r: JsonReader, key: str, where: str) -> float:
    v = r.number(key)
    if not (v > 0.0 and math.isfinite(v)):
        raise ConfigError(f"{where}: {key} must be positive")
    return v


def _latent(m: JsonReader, where: str) -> KunitarLatent:
    rot_dim = m.integer("rot_dim", minimum=2)
    rot = _part(m, "rot", where)
    dims = rot.integer("dims", rot_dim)
    if dims != rot_dim or rot_dim % 2:
        raise ConfigError(f"{where}: rot.dims {dims} must be rot_dim {rot_dim}, an even number")
    window = None
    if m.raw("mask") is not None:
        window = _part(m, "mask", where).integer("size", minimum=1)
    dim = m.integer("dim", minimum=1)
    return KunitarLatent(m.integer("heads", minimum=1), dim, rot_dim, m.integer("vdim", dim, minimum=1),
                         m.integer("kv_rank", minimum=1), m.integer("q_rank", minimum=1), m.number("scale"), window,
                         _positive(rot, "base", where + ".rot"), m.integer("kv_from", None, minimum=0))


def _time_mix(m: JsonReader, where: str) -> KunitarTimeMix:
    return KunitarTimeMix(m.integer("heads", minimum=1), m.integer("dim", minimum=1), m.integer("decay_rank", None, minimum=1))


def _dense(f: JsonReader, where: str) -> KunitarDense:
    return KunitarDense(f.integer("ff", minimum=1))


def _experts(f: JsonReader, where: str) -> KunitarExperts:
    r = _part(f, "router", where)
    experts, top = r.integer("experts", minimum=1), r.integer("top", minimum=1)
    if top > experts:
        raise ConfigError(f"{where}.router: {top} of {experts} experts cannot be chosen")
    shared_ff = None if f.raw("shared") is None else _part(f, "shared", where).integer("ff", minimum=1)
    return KunitarExperts(experts, top, _part(f, "expert", where).integer("ff", minimum=1), shared_ff)


_MIXERS = {"latent_attention": _latent, "wkv": _time_mix}
_FEED_FORWARDS = {"dense": _dense, "moe": _experts}


@dataclass(frozen=True)
class KunitarConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    side_dim: int
    layers: Tuple[KunitarLayer, ...]
    max_positions: Optional[int] = None
    eos_token_ids: Tuple[int, ...] = ()

    @staticmethod
    def from_dict(data: Dict[str, Any], origin: str = "config.json") -> "KunitarConfig":
        r = JsonReader(data, origin)
        name = r.string("architecture")
        if name != ARCHITECTURE:
            raise ConfigError(f"{origin}: architecture '{name}' is not '{ARCHITECTURE}'")
        raw_layers = r.raw("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError(f"{origin}: 'layers' must be a non-empty list")
        layers = []
        for i, entry in enumerate(raw_layers):
            where = f"{origin}: layers[{i}]"
            lr = JsonReader(entry, where)
            kind = lr.string("type")
            if kind not in _MIXERS:
                raise ConfigError(f"{where}: layer type '{kind}' is not known; known: {', '.join(sorted(_MIXERS))}")
            mixer = _MIXERS[kind](_part(lr, "mixer", where), where + ".mixer")
            mlp = None
            if lr.raw("mlp") is not None:
                f = _part(lr, "mlp", where)
                if f.string("kind") not in _FEED_FORWARDS:
                    raise ConfigError(f"{where}.mlp: feed-forward kind '{f.string('kind')}' is not known; known: "
                                      f"{', '.join(sorted(_FEED_FORWARDS))}")
                mlp = _FEED_FORWARDS[f.string("kind")](f, where + ".mlp")
            layers.append(KunitarLayer(kind, mixer, mlp))
        for i, layer in enumerate(layers):
            j = getattr(layer.mixer, "kv_from", None)
            if j is None:
                continue
            owner = layers[j].mixer if j < i else None
            if not isinstance(owner, KunitarLatent) or owner.kv_from is not None:
                raise ConfigError(f"{origin}: layers[{i}]: kv_from must name an earlier layer with latent vectors of its own")
            m = layer.mixer
            if (owner.kv_rank, owner.rot_dim, owner.rot_base) != (m.kv_rank, m.rot_dim, m.rot_base):
                raise ConfigError(f"{origin}: layers[{i}] reads the vectors of layer {j} but has another latent size or rotation")
        return KunitarConfig(vocab=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1),
                             norm_eps=_positive(_part(r, "norm", origin), "eps", origin + ": norm"),
                             embedding_scale=_part(r, "embedding", origin).number("scale", 1.0),
                             side_dim=_part(r, "token_side", origin).integer("dim", minimum=1), layers=tuple(layers),
                             max_positions=r.integer("max_positions", None, minimum=1),
                             eos_token_ids=tuple(r.int_list("eos_token_id", [])))

    def to_dict(self) -> Dict[str, Any]:
        """The config.json this configuration is read back from."""
        out: Dict[str, Any] = {
            "architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
            "embedding": {"scale": self.embedding_scale}, "token_side": {"dim": self.side_dim},
            "layers": [layer.to_dict() for layer in self.layers],
        }
        if self.max_positions is not None:
            out["max_positions"] = self.max_positions
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out
