"""Typed configuration of the Zazerax design, read from config.json.

    {"architecture": "Zazerax", "vocab": V, "width": W, "norm": {"eps": e}, "embedding": {"scale": s},
     "layers": [{"type": "attention" | "latent_attention" | "latent_attention_2", "mixer": {...},
                 "mlp": {"kind": "dense", "ff": F} | null, "weights_of": j}, ...]}

Every layer entry carries its own sizes, so layers of different kinds and sizes may follow each other in any order.
`attention` mixer: heads, kv_heads, dim, vdim, scale, bias_max (the distance that the last row of the distance biases
begins to serve), mask {size} (the window).  `latent_attention` mixer: heads, dim (unrotated query/key dimensions a head), rot_dim
(rotated ones), vdim, kv_rank, scale, rot {base, dims, optional scaling {factor, original, fast, slow}};
`latent_attention_2`: the same and q_rank.  `weights_of` j: the layer runs with layer j's tensors (the rest of its entry
equals layer j's).  The number of rows of the distance biases is that of the checkpoint's tensor (`bias_rows` may name it
for a model made without a checkpoint; without both, 32).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field

from .. import limits
from .base import ConfigError, ConfigReader
from .fokinex import RampedRotaryConfig
from .rafilix import _section

MIXER_TYPES = ("attention", "latent_attention", "latent_attention_2")


@dataclass(frozen=True)
class BiasedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: int
    window: int | None
    bias_rows: int | None = None


@dataclass(frozen=True)
class LatentAttentionConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int | None
    kv_rank: int
    scale: float
    rot: RampedRotaryConfig | None


@dataclass(frozen=True)
class DenseConfig:
    ff: int


@dataclass(frozen=True)
class ZazeraxLayer:
    type: str
    mixer: object      # BiasedAttentionConfig or LatentAttentionConfig
    mlp: DenseConfig | None
    weights_of: int | None = None


def _attention(r: ConfigReader) -> BiasedAttentionConfig:
    heads, kv = r.integer("heads", minimum=1), r.integer("kv_heads", minimum=1)
    if heads % kv:
        raise ConfigError(f"{r.where}: heads {heads} is not a multiple of kv_heads {kv}")
    dim, vdim = r.integer("dim", minimum=1), r.integer("vdim", minimum=1)
    if max(dim, vdim) > limits.HEAD_DIM_MAX:
        raise ConfigError(f"{r.where}: head sizes {dim} / {vdim} are more than the attention kernels' {limits.HEAD_DIM_MAX}")
    mr = _section(r, "mask", required=False)
    return BiasedAttentionConfig(heads, kv, dim, vdim, r.number("scale", positive=True), r.integer("bias_max", minimum=1),
                                 mr.integer("size", minimum=1) if mr is not None else None, r.optional_integer("bias_rows", minimum=2))


def _rotation(r: ConfigReader, rot_dim: int) -> RampedRotaryConfig | None:
    rr = _section(r, "rot", required=False)
    if rr is None:
        return None
    dims = rr.integer("dims", minimum=0)
    if dims % 2 or dims > rot_dim:
        raise ConfigError(f"{rr.where}: dims {dims} must be even and at most rot_dim {rot_dim}")
    base, scaling = rr.number("base", positive=True), None
    sr = _section(rr, "scaling", required=False)
    if sr is not None:
        scaling = tuple(sr.number(key, positive=True) for key in ("factor", "original", "fast", "slow"))
        if base == 1.0:
            raise ConfigError(f"{rr.where}: a base of 1 has no wavelengths to scale")
    return RampedRotaryConfig(dims, base, scaling) if dims else None


def _latent(r: ConfigReader, with_query_latent: bool) -> LatentAttentionConfig:
    heads, dim, vdim = (r.integer(key, minimum=1) for key in ("heads", "dim", "vdim"))
    rot_dim, kv_rank = r.integer("rot_dim", minimum=0), r.integer("kv_rank", minimum=1)
    q_rank = r.integer("q_rank", minimum=1) if with_query_latent else None
    if kv_rank + rot_dim > limits.HEAD_DIM_MAX_ANY:
        raise ConfigError(f"{r.where}: kv_rank {kv_rank} + rot_dim {rot_dim} is more than the attention kernels' {limits.HEAD_DIM_MAX_ANY}")
    return LatentAttentionConfig(heads, dim, rot_dim, vdim, q_rank, kv_rank, r.number("scale", positive=True), _rotation(r, rot_dim))


_MIXERS = {"attention": _attention, "latent_attention": lambda r: _latent(r, False), "latent_attention_2": lambda r: _latent(r, True)}


def _mlp(r: ConfigReader | None) -> DenseConfig | None:
    if r is None:
        return None
    kind = r.string("kind", "dense")
    if kind != "dense":
        raise ConfigError(f"{r.where}: feed-forward kind '{kind}' is not one this design has (dense)")
    return DenseConfig(r.integer("ff", minimum=1))


def _resolve_owners(layers: list, where: str) -> list:
    """`weights_of` followed to the layer that has tensors."""
    out = []
    for i, layer in enumerate(layers):
        owner, seen = layer.weights_of, {i}
        while owner is not None:
            if owner >= len(layers) or owner in seen:
                raise ConfigError(f"{where}: layers[{i}]: weights_of names no layer with tensors of its own")
            seen.add(owner)
            if (layers[owner].type, layers[owner].mixer, layers[owner].mlp) != (layer.type, layer.mixer, layer.mlp):
                raise ConfigError(f"{where}: layers[{i}] uses the weights of layer {owner}, but is not like it")
            if layers[owner].weights_of is None:
                break
            owner = layers[owner].weights_of
        out.append(ZazeraxLayer(layer.type, layer.mixer, layer.mlp, owner))
    return out


@dataclass(frozen=True)
class ZazeraxConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    layers: tuple
    raw: dict = field(default_factory=dict, compare=False, repr=False)
    eos_token_id: int | tuple | None = None
    max_positions: int = 32768            # the design names no limit; the optional key `max_positions` does (it sizes the default cache)
    defaulted_keys: tuple = field(default=(), compare=False)

    architecture = "Zazerax"
    model_type = "zazerax"

    @classmethod
    def from_dict(cls, raw: dict, where: str = "config.json") -> "ZazeraxConfig":
        r = ConfigReader(raw, where)
        vocab, width = r.integer("vocab", minimum=1), r.integer("width", minimum=1)
        eps = _section(r, "norm").number("eps", positive=True)
        er = _section(r, "embedding", required=False)
        emb_scale = er.number("scale", 1.0) if er is not None else 1.0
        entries = raw.get("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError(f"{where}: key 'layers' must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(entries):
            lr = ConfigReader(entry, f"{where}: layers[{i}]")
            kind = lr.string("type")
            if kind not in MIXER_TYPES:
                raise ConfigError(f"{lr.where}: type '{kind}' is not one of {', '.join(MIXER_TYPES)}")
            layers.append(ZazeraxLayer(kind, _MIXERS[kind](_section(lr, "mixer")), _mlp(_section(lr, "mlp", required=False)),
                                       lr.optional_integer("weights_of", minimum=0)))
        eos = raw.get("eos_token_id")
        if isinstance(eos, list):
            eos = tuple(int(e) for e in eos)
        return cls(vocab, width, eps, emb_scale, tuple(_resolve_owners(layers, where)), copy.deepcopy(raw), eos,
                   r.integer("max_positions", 32768, minimum=1), tuple(r.defaulted))

    def to_dict(self) -> dict:
        out = copy.deepcopy(self.raw)
        out.setdefault("architecture", self.architecture)
        return out
