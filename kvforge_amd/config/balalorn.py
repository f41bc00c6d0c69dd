"""Typed configuration of the Balalorn decoder, read from its own ``config.json`` keys.

A Balalorn ``config.json`` names its model with ``"architecture": "Balalorn"`` and describes every
layer by itself under ``"layers"``: ``type`` (``"mamba2"``, ``"delta"`` or ``"latent_attention"``),
``mixer`` (that mixer's sizes and constants) and ``mlp`` (``kind`` ``"dense"`` with ``ff``, or ``"moe"``
with ``expert.ff``, ``router.experts`` and ``router.top``; ``null`` for none).  Top-level keys:
``vocab``, ``width``, ``norm.eps``.  The design has no position limit of its own; ``max_positions``
may be given, and is otherwise ``DEFAULT_MAX_POSITIONS``.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any

from kvforge_amd.config.fogorax import _positive
from kvforge_amd.config.model import ConfigError, ModelConfig, _require
from kvforge_amd.config.rudorax import DEFAULT_MAX_POSITIONS, RotaryConfig, _number

MAX_KEY_SIZE = 256     # key size of a memory's head, as the kernels take it
MAX_TAPS = 8           # taps of a short convolution
MAX_LATENT_ROW = 640   # rotated key part and latent of a token together, as the attention kernels take them


def _taps(d: dict[str, Any], where: str) -> int:
    taps = _positive(d, "conv", where)
    if taps > MAX_TAPS:
        raise ConfigError(f"{where}: convolutions of more than {MAX_TAPS} taps are not supported, got {taps}")
    return taps


def _key_size(d: dict[str, Any], key: str, where: str) -> int:
    size = _positive(d, key, where)
    if size > MAX_KEY_SIZE:
        raise ConfigError(f"{where}: {key!r} of more than {MAX_KEY_SIZE} is not supported, got {size}")
    return size


def _shared_by(d: dict[str, Any], key: str, heads: int, where: str) -> int:
    """How many groups share the heads: a divisor of their number (a file may leave it out: one each)."""
    groups = _positive(d, key, where) if d.get(key) is not None else heads
    if heads % groups:
        raise ConfigError(f"{where}: heads ({heads}) must be a multiple of {key} ({groups})")
    return groups


@dataclass(frozen=True)
class Mamba2Config:
    """``heads`` memories of ``state`` x ``vdim``; ``groups`` of heads share B and C; the output row is
    normalised in ``norm_groups`` equal parts; ``conv`` taps."""

    heads: int
    vdim: int
    state: int
    groups: int
    norm_groups: int
    conv: int

    @classmethod
    def from_dict(cls, d: dict[str, Any], where: str) -> "Mamba2Config":
        heads, vdim = _positive(d, "heads", where), _positive(d, "vdim", where)
        parts = _positive(d, "norm_groups", where) if d.get("norm_groups") is not None else 1
        if heads * vdim % parts:
            raise ConfigError(f"{where}: heads * vdim ({heads * vdim}) must be a multiple of norm_groups ({parts})")
        return cls(heads, vdim, _key_size(d, "state", where), _shared_by(d, "groups", heads, where), parts,
                   _taps(d, where))

    def to_dict(self) -> dict[str, Any]:
        return {"conv": self.conv, "groups": self.groups, "heads": self.heads, "norm_groups": self.norm_groups,
                "state": self.state, "vdim": self.vdim}


@dataclass(frozen=True)
class DeltaConfig:
    """``heads`` memories of ``dim`` x ``vdim`` written by the delta rule, over ``kv_heads`` query/key
    heads; ``conv`` taps."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    @classmethod
    def from_dict(cls, d: dict[str, Any], where: str) -> "DeltaConfig":
        heads, dim = _positive(d, "heads", where), _key_size(d, "dim", where)
        return cls(heads, _shared_by(d, "kv_heads", heads, where), dim,
                   _positive(d, "vdim", where) if d.get("vdim") is not None else dim, _taps(d, where))

    def to_dict(self) -> dict[str, Any]:
        return {"conv": self.conv, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "vdim": self.vdim}


@dataclass(frozen=True)
class GatedLatentConfig:
    """Latent attention with a gate per head: per head ``dim`` plain and ``rot_dim`` rotated query/key
    elements and ``vdim`` value elements, keys and values read out of a latent of ``kv_rank`` elements.
    ``kv_from``: the layer whose latents and rotated key parts this layer uses (``None``: its own)."""

    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot: RotaryConfig | None
    kv_from: int | None = None

    @classmethod
    def from_dict(cls, d: dict[str, Any], where: str) -> "GatedLatentConfig":
        sizes = {}
        for key in ("dim", "rot_dim"):
            v = d.get(key) or 0
            if not isinstance(v, int) or isinstance(v, bool) or v < 0:
                raise ConfigError(f"{where}: {key!r} must be a non-negative integer, got {v!r}")
            sizes[key] = v
        if sizes["dim"] + sizes["rot_dim"] <= 0:
            raise ConfigError(f"{where}: 'dim' and 'rot_dim' must not both be zero")
        rot = d.get("rot")
        rot = RotaryConfig.from_dict(rot, where) if rot else None
        if rot is not None and rot.dims > sizes["rot_dim"]:
            raise ConfigError(f"{where}: rot.dims ({rot.dims}) exceeds rot_dim ({sizes['rot_dim']})")
        if sizes["rot_dim"] + _positive(d, "kv_rank", where) > MAX_LATENT_ROW:
            raise ConfigError(f"{where}: rot_dim + kv_rank must not exceed {MAX_LATENT_ROW} (the attention kernels' head size)")
        src = d.get("kv_from")
        if src is not None and (not isinstance(src, int) or isinstance(src, bool) or src < 0):
            raise ConfigError(f"{where}: 'kv_from' must name an earlier layer, got {src!r}")
        return cls(_positive(d, "heads", where), sizes["dim"], sizes["rot_dim"], _positive(d, "vdim", where),
                   _positive(d, "kv_rank", where), _number(d, "scale", where), rot, src)

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"dim": self.dim, "heads": self.heads}
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        out.update({"kv_rank": self.kv_rank,
                    "rot": {"base": self.rot.base, "dims": self.rot.dims} if self.rot else None,
                    "rot_dim": self.rot_dim, "scale": self.scale, "vdim": self.vdim})
        return out


@dataclass(frozen=True)
class BalalornMlpConfig:
    """``kind`` ``"dense"``: a silu-gated feed-forward of width ``ff``.  ``"moe"``: ``experts`` of them, of
    width ``ff``, of which a token uses the ``top`` of largest score."""

    kind: str
    ff: int
    experts: int = 0
    top: int = 0

    @classmethod
    def from_dict(cls, d: dict[str, Any], where: str) -> "BalalornMlpConfig":
        kind = _require(d, "kind")
        if kind == "dense":
            return cls("dense", _positive(d, "ff", where))
        if kind != "moe":
            raise ConfigError(f"{where}: feed-forward kind {kind!r} is not supported (known: ('dense', 'moe'))")
        r = _require(d, "router")
        experts, top = _positive(r, "experts", where), _positive(r, "top", where)
        if top > experts:
            raise ConfigError(f"{where}: router.top ({top}) exceeds the {experts} experts")
        return cls("moe", _positive(_require(d, "expert"), "ff", where), experts, top)

    def to_dict(self) -> dict[str, Any]:
        if self.kind == "dense":
            return {"ff": self.ff, "kind": "dense"}
        return {"expert": {"ff": self.ff}, "kind": "moe", "router": {"experts": self.experts, "top": self.top}}


@dataclass(frozen=True)
class BalalornLayerConfig:
    type: str
    mixer: "Mamba2Config | DeltaConfig | GatedLatentConfig"
    mlp: BalalornMlpConfig | None

    MIXERS = {"mamba2": Mamba2Config, "delta": DeltaConfig, "latent_attention": GatedLatentConfig}

    @classmethod
    def from_dict(cls, d: dict[str, Any], index: int) -> "BalalornLayerConfig":
        where = f"layer {index}"
        kind = _require(d, "type")
        if kind not in cls.MIXERS:
            raise ConfigError(f"{where}: mixer type {kind!r} is not supported (known: {tuple(cls.MIXERS)})")
        mlp = d.get("mlp")
        return cls(kind, cls.MIXERS[kind].from_dict(_require(d, "mixer"), where),
                   BalalornMlpConfig.from_dict(mlp, where) if mlp is not None else None)

    def to_dict(self) -> dict[str, Any]:
        return {"mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None, "type": self.type}


@dataclass
class BalalornConfig(ModelConfig):
    """``vocab_size`` of the base class is the file's ``vocab``."""

    width: int = 0
    norm_eps: float = 0.0
    layers: list[BalalornLayerConfig] = field(default_factory=list)

    NAME = "Balalorn"

    def __post_init__(self) -> None:
        if self.width <= 0 or self.vocab_size <= 0 or self.max_position_embeddings <= 0:
            raise ConfigError("vocab, width and max_positions must be positive")
        if not self.layers:
            raise ConfigError("a model needs at least one layer")
        for i, layer in enumerate(self.layers):
            src = getattr(layer.mixer, "kv_from", None)
            if src is None:
                continue
            m, o = layer.mixer, self.layers[src].mixer if src < i else None
            if not isinstance(o, GatedLatentConfig) or o.kv_from is not None:
                raise ConfigError(f"layer {i}: kv_from ({src}) must name an earlier latent-attention layer with "
                                  f"latents of its own")
            if (m.kv_rank, m.rot_dim, m.rot) != (o.kv_rank, o.rot_dim, o.rot):
                raise ConfigError(f"layer {i}: kv_rank, rot_dim and rot must equal those of layer {src}, whose "
                                  f"latents it uses")

    @classmethod
    def from_dict(cls, d: dict[str, Any]) -> "BalalornConfig":
        layers = _require(d, "layers")
        if not isinstance(layers, list):
            raise ConfigError("'layers' must be a list")
        return cls(
            architecture=cls.NAME,
            vocab_size=_positive(d, "vocab", "config.json"),
            max_position_embeddings=(_positive(d, "max_positions", "config.json")
                                     if d.get("max_positions") is not None else DEFAULT_MAX_POSITIONS),
            bos_token_id=d.get("bos_token_id"), eos_token_id=d.get("eos_token_id"),
            width=_positive(d, "width", "config.json"),
            norm_eps=_number(_require(d, "norm"), "eps", "norm", positive=False),
            layers=[BalalornLayerConfig.from_dict(x, i) for i, x in enumerate(layers)])

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "architecture": self.NAME,
            "layers": [x.to_dict() for x in self.layers],
            "max_positions": self.max_position_embeddings,
            "norm": {"eps": self.norm_eps},
            "vocab": self.vocab_size,
            "width": self.width,
        }
        for key in ("bos_token_id", "eos_token_id"):
            if getattr(self, key) is not None:
                out[key] = getattr(self, key)
        return out

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)
