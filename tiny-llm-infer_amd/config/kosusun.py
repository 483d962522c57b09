"""Typed configuration of the Kosusun decoder, read from its config.json.

Keys: ``architecture`` ("Kosusun"), ``vocab``, ``width``, ``embedding.scale``, ``logit_scale``,
``residual_mult``, ``norm.eps``, ``max_positions`` (optional: the design itself sets no limit) and
``layers``: a list with one entry a layer, ``{"type": "mlstm" | "parallel", "mixer": {...}, "mlp":
{"kind": "dense", "ff": n} or null}``.

An mlstm mixer gives ``heads``, ``dim``, ``vdim`` and ``gate_cap``.  A parallel mixer gives
``left_scale``, ``right_scale``, and two mixers: ``left``, an attention over a window and pooled blocks
(``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``mask.size``, ``mask.pool``, ``rot``), and ``right``, a
retention (``heads``, ``dim``, ``vdim``, ``decay``: one number a head, ``rot``).  A ``rot`` gives ``dims``, ``base``
and optionally ``scaling.factor``.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple, Union

from .base import ConfigError, JsonReader

ARCHITECTURE = "Kosusun"
NO_POSITION_LIMIT = 1 << 20          # what a config.json without ``max_positions`` is taken to allow


@dataclass(frozen=True)
class KosusunRotation:
    dims: int
    base: float
    factor: float                    # every frequency is divided by it

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"dims": self.dims, "base": self.base}
        if self.factor != 1.0:
            out["scaling"] = {"factor": self.factor}
        return out


@dataclass(frozen=True)
class KosusunWindow:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int
    pool: int
    rot: KosusunRotation

    def to_dict(self) -> Dict[str, Any]:
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
                "mask": {"size": self.window, "pool": self.pool}, "rot": self.rot.to_dict()}


@dataclass(frozen=True)
class KosusunRetention:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    rot: KosusunRotation

    def to_dict(self) -> Dict[str, Any]:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay), "rot": self.rot.to_dict()}


@dataclass(frozen=True)
class KosusunParallel:
    left: KosusunWindow
    right: KosusunRetention
    left_scale: float
    right_scale: float

    def to_dict(self) -> Dict[str, Any]:
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale,
                "right_scale": self.right_scale}


@dataclass(frozen=True)
class KosusunMemory:
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    def to_dict(self) -> Dict[str, Any]:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "gate_cap": self.gate_cap}


@dataclass(frozen=True)
class KosusunLayer:
    kind: str                                         # "parallel" or "mlstm"
    mixer: Union[KosusunParallel, KosusunMemory]
    ff: Optional[int]                                 # None: no feed-forward

    def to_dict(self) -> Dict[str, Any]:
        return {"type": self.kind, "mixer": self.mixer.to_dict(), "mlp": None if self.ff is None else {"kind": "dense", "ff": self.ff}}


def _part(r: JsonReader, key: str, where: str) -> JsonReader:
    return JsonReader(r.raw(key) or {}, f"{where}.{key}")


def _positive(r: JsonReader, key: str, where: str, default=None) -> float:
    v = r.number(key) if default is None else r.number(key, default)
    if not (v > 0.0 and math.isfinite(v)):
        raise ConfigError(f"{where}: {key} must be positive")
    return v


def _rotation(m: JsonReader, where: str, dim: int) -> KosusunRotation:
    rot = _part(m, "rot", where)
    dims = rot.integer("dims", dim, minimum=2)
    if dims % 2 or dims > dim:
        raise ConfigError(f"{where}: rot.dims {dims} must be even and at most dim {dim}")
    factor = 1.0
    if rot.raw("scaling") is not None:
        factor = _positive(_part(rot, "scaling", where + ".rot"), "factor", where + ".rot.scaling")
    return KosusunRotation(dims, _positive(rot, "base", where + ".rot"), factor)


def _window(m: JsonReader, where: str) -> KosusunWindow:
    heads = m.integer("heads", minimum=1)
    kv_heads = m.integer("kv_heads", heads, minimum=1)
    if heads % kv_heads:
        raise ConfigError(f"{where}: heads {heads} must be a multiple of kv_heads {kv_heads}")
    dim = m.integer("dim", minimum=2)
    mask = _part(m, "mask", where)
    return KosusunWindow(heads, kv_heads, dim, m.integer("vdim", dim, minimum=1), m.number("scale"),
                         mask.integer("size", minimum=1), mask.integer("pool", minimum=1), _rotation(m, where, dim))


def _retention(m: JsonReader, where: str) -> KosusunRetention:
    heads = m.integer("heads", minimum=1)
    dim = m.integer("dim", minimum=2)
    decay = m.raw("decay")
    if (not isinstance(decay, (list, tuple)) or len(decay) != heads
            or any(isinstance(x, bool) or not isinstance(x, (int, float)) for x in decay)):
        raise ConfigError(f"{where}: 'decay' must be a list of {heads} numbers, one a head")
    return KosusunRetention(heads, dim, m.integer("vdim", dim, minimum=1), tuple(float(x) for x in decay),
                            _rotation(m, where, dim))


def _parallel(m: JsonReader, where: str) -> KosusunParallel:
    return KosusunParallel(_window(_part(m, "left", where), where + ".left"), _retention(_part(m, "right", where), where + ".right"),
                           m.number("left_scale"), m.number("right_scale"))


def _memory(m: JsonReader, where: str) -> KosusunMemory:
    dim = m.integer("dim", minimum=1)
    return KosusunMemory(m.integer("heads", minimum=1), dim, m.integer("vdim", dim, minimum=1), _positive(m, "gate_cap", where))


_MIXERS = {"parallel": _parallel, "mlstm": _memory}


@dataclass(frozen=True)
class KosusunConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    residual_mult: float
    logit_scale: float
    layers: Tuple[KosusunLayer, ...]
    max_positions: Optional[int] = None
    eos_token_ids: Tuple[int, ...] = ()

    @staticmethod
    def from_dict(data: Dict[str, Any], origin: str = "config.json") -> "KosusunConfig":
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
            ff = None
            if lr.raw("mlp") is not None:
                mlp = _part(lr, "mlp", where)
                if mlp.string("kind") != "dense":
                    raise ConfigError(f"{where}.mlp: feed-forward kind '{mlp.string('kind')}' is not known; known: dense")
                ff = mlp.integer("ff", minimum=1)
            layers.append(KosusunLayer(kind, mixer, ff))
        return KosusunConfig(vocab=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1),
                             norm_eps=_positive(_part(r, "norm", origin), "eps", origin + ": norm"),
                             embedding_scale=_part(r, "embedding", origin).number("scale", 1.0),
                             residual_mult=r.number("residual_mult", 1.0), logit_scale=r.number("logit_scale", 1.0),
                             layers=tuple(layers), max_positions=r.integer("max_positions", None, minimum=1),
                             eos_token_ids=tuple(r.int_list("eos_token_id", [])))

    def to_dict(self) -> Dict[str, Any]:
        """The config.json this configuration is read back from."""
        out: Dict[str, Any] = {
            "architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
            "embedding": {"scale": self.embedding_scale}, "residual_mult": self.residual_mult, "logit_scale": self.logit_scale,
            "layers": [layer.to_dict() for layer in self.layers],
        }
        if self.max_positions is not None:
            out["max_positions"] = self.max_positions
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out
