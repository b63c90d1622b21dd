"""Typed configuration of the Besulix design, read from config.json.

    {"architecture": "Besulix", "vocab": V, "width": W, "norm": {"eps": e}, "logit_softcap": c,
     "layers": [{"type": "parallel" | "mlstm", "mixer": {...}, "mlp": {"kind": "dense", "ff": F, "limit": L} | null}, ...]}

Every layer entry carries its own sizes, so layers of different kinds and sizes may follow each other in any order.
`parallel` mixer: left {heads, kv_heads, dim, vdim, scale, rot {base, dims}, mask {size}} (chunked softmax attention),
right {heads, dim} (time mixing), left_scale, right_scale.  `mlstm` mixer: heads, dim, vdim, gate_cap (matrix memory).
The inner size of the time mixing's decay projection is that of the checkpoint's tensor (`decay_rank` may name it for a
model made without a checkpoint; without both, a quarter of dim, at least 16).
"""
from __future__ import annotations

import copy
import math
from dataclasses import dataclass, field

from .. import limits
from .base import ConfigError, ConfigReader
from .rafilix import _section

MIXER_TYPES = ("parallel", "mlstm")
RECURRENT_DIM_MAX = 256      # key channels a head that the recurrence kernel holds


@dataclass(frozen=True)
class ChunkedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int
    rot_base: float
    chunk: int


@dataclass(frozen=True)
class TimeMixConfig:
    heads: int
    dim: int
    decay_rank: int | None = None


@dataclass(frozen=True)
class SideBySideConfig:
    left: ChunkedAttentionConfig
    right: TimeMixConfig
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class MatrixMemoryConfig:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass(frozen=True)
class DenseConfig:
    ff: int
    limit: float


@dataclass(frozen=True)
class BesulixLayer:
    type: str
    mixer: object      # SideBySideConfig or MatrixMemoryConfig
    mlp: DenseConfig | None


def _recurrent_dim(r: ConfigReader) -> int:
    dim = r.integer("dim", minimum=1)
    if dim > RECURRENT_DIM_MAX:
        raise ConfigError(f"{r.where}: dim {dim} is more than the recurrence kernel's {RECURRENT_DIM_MAX} key channels a head")
    return dim


def _attention(r: ConfigReader) -> ChunkedAttentionConfig:
    heads, kv = r.integer("heads", minimum=1), r.integer("kv_heads", minimum=1)
    if heads % kv:
        raise ConfigError(f"{r.where}: heads {heads} is not a multiple of kv_heads {kv}")
    dim, vdim = r.integer("dim", minimum=1), r.integer("vdim", minimum=1)
    if max(dim, vdim) > limits.HEAD_DIM_MAX:
        raise ConfigError(f"{r.where}: head sizes {dim} / {vdim} are more than the attention kernels' {limits.HEAD_DIM_MAX}")
    if vdim % 2:
        raise ConfigError(f"{r.where}: vdim {vdim} must be even: values are turned in pairs")
    rr = _section(r, "rot")
    dims = rr.integer("dims", minimum=0)
    if dims % 2 or dims > dim:
        raise ConfigError(f"{rr.where}: dims {dims} must be even and at most dim {dim}")
    return ChunkedAttentionConfig(heads, kv, dim, vdim, r.number("scale", positive=True), dims, rr.number("base", positive=True),
                                  _section(r, "mask").integer("size", minimum=1))


def _parallel(r: ConfigReader) -> SideBySideConfig:
    rr = _section(r, "right")
    right = TimeMixConfig(rr.integer("heads", minimum=1), _recurrent_dim(rr), rr.optional_integer("decay_rank", minimum=1))
    return SideBySideConfig(_attention(_section(r, "left")), right, _finite(r, "left_scale"), _finite(r, "right_scale"))


def _finite(r: ConfigReader, key: str) -> float:
    v = r.number(key)
    if not math.isfinite(v):
        raise ConfigError(f"{r.where}: key '{key}' must be finite, got {v}")
    return v


def _mlstm(r: ConfigReader) -> MatrixMemoryConfig:
    return MatrixMemoryConfig(r.integer("heads", minimum=1), _recurrent_dim(r), r.integer("vdim", minimum=1),
                              r.number("gate_cap", positive=True))


def _mlp(r: ConfigReader | None) -> DenseConfig | None:
    if r is None:
        return None
    kind = r.string("kind", "dense")
    if kind != "dense":
        raise ConfigError(f"{r.where}: feed-forward kind '{kind}' is not one this design has (dense)")
    return DenseConfig(r.integer("ff", minimum=1), r.number("limit", positive=True))


@dataclass(frozen=True)
class BesulixConfig:
    vocab: int
    width: int
    eps: float
    logit_softcap: float
    layers: tuple
    raw: dict = field(default_factory=dict, compare=False, repr=False)
    eos_token_id: int | tuple | None = None
    max_positions: int = 32768            # the design names no limit; the optional key `max_positions` does (it sizes the default cache)
    defaulted_keys: tuple = field(default=(), compare=False)

    architecture = "Besulix"
    model_type = "besulix"

    @classmethod
    def from_dict(cls, raw: dict, where: str = "config.json") -> "BesulixConfig":
        r = ConfigReader(raw, where)
        vocab, width = r.integer("vocab", minimum=1), r.integer("width", minimum=1)
        eps = _section(r, "norm").number("eps", positive=True)
        softcap = r.number("logit_softcap", positive=True)
        entries = raw.get("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError(f"{where}: key 'layers' must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(entries):
            lr = ConfigReader(entry, f"{where}: layers[{i}]")
            kind = lr.string("type")
            if kind not in MIXER_TYPES:
                raise ConfigError(f"{lr.where}: type '{kind}' is not one of {', '.join(MIXER_TYPES)}")
            mr = _section(lr, "mixer")
            layers.append(BesulixLayer(kind, {"parallel": _parallel, "mlstm": _mlstm}[kind](mr),
                                       _mlp(_section(lr, "mlp", required=False))))
        eos = raw.get("eos_token_id")
        if isinstance(eos, list):
            eos = tuple(int(e) for e in eos)
        return cls(vocab, width, eps, softcap, tuple(layers), copy.deepcopy(raw), eos,
                   r.integer("max_positions", 32768, minimum=1), tuple(r.defaulted))

    def to_dict(self) -> dict:
        out = copy.deepcopy(self.raw)
        out.setdefault("architecture", self.architecture)
        return out
