"""Typed configuration of the Depolix decoder, read from its own ``config.json`` keys.

A Depolix ``config.json`` names its model with ``"architecture": "Depolix"`` and describes every layer
by itself under ``"layers"``: ``type`` (``"latent_attention"`` or ``"parallel"``), ``mixer`` (that mixer's sizes
and constants; a ``parallel`` mixer holds ``left`` and ``right``) and ``mlp`` (``kind`` ``"dense"`` with ``ff`` and
``limit``, or ``"moe"`` with ``expert.ff``, ``expert.limit``, ``router.experts`` and ``router.top``; ``null`` for none).
Top-level keys: ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``, ``residual_mult`` and ``logit_scale``.  The
design has no position limit of its own; ``max_positions`` may be given, and is otherwise
``DEFAULT_MAX_POSITIONS``.  The rows of a distance-bias table and the ranks of a memory's low-rank gates
are the checkpoint's; ``buckets``, ``a_rank`` and ``g_rank`` may name them (a model with random weights needs
them).
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any

from kvforge_amd.config.balalorn import MAX_LATENT_ROW, _key_size, _shared_by, _taps
from kvforge_amd.config.fogorax import WindowMask, _positive
from kvforge_amd.config.ludelix import LudelixRotary, _heads
from kvforge_amd.config.model import ConfigError, ModelConfig, _require
from kvforge_amd.config.rudorax import DEFAULT_MAX_POSITIONS, YarnScaling, _number

MAX_HEAD = 256      # elements of an attention head, as the kernels take them


def _optional(d: dict[str, Any], key: str, where: str) -> int | None:
    return _positive(d, key, where) if d.get(key) is not None else None


@dataclass(frozen=True)
class QueryLatentConfig:
    """Latent attention whose queries go through a latent of ``q_rank`` elements: per head ``dim`` plain and
    ``rot_dim`` rotated query/key elements and ``vdim`` value elements, keys and values read out of a latent of
    ``kv_rank`` elements."""

    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot: LudelixRotary | None

    @classmethod
    def from_dict(cls, d: dict[str, Any], where: str) -> "QueryLatentConfig":
        sizes = {}
        for key in ("dim", "rot_dim"):
            v = d.get(key) or 0
            if not isinstance(v, int) or isinstance(v, bool) or v < 0:
                raise ConfigError(f"{where}: {key!r} must be a non-negative integer, got {v!r}")
            sizes[key] = v
        if sizes["dim"] + sizes["rot_dim"] <= 0:
            raise ConfigError(f"{where}: 'dim' and 'rot_dim' must not both be zero")
        rot = d.get("rot")
        rot = LudelixRotary.from_dict(rot, where, "halves", YarnScaling) if rot else None
        if rot is not None and rot.dims > sizes["rot_dim"]:
            raise ConfigError(f"{where}: rot.dims ({rot.dims}) exceeds rot_dim ({sizes['rot_dim']})")
        rank = _positive(d, "kv_rank", where)
        if sizes["rot_dim"] + rank > MAX_LATENT_ROW:
            raise ConfigError(f"{where}: rot_dim + kv_rank must not exceed {MAX_LATENT_ROW} (the attention kernels' head size)")
        return cls(_positive(d, "heads", where), sizes["dim"], sizes["rot_dim"], _positive(d, "vdim", where),
                   _positive(d, "q_rank", where), rank, _number(d, "scale", where), rot)

    def to_dict(self) -> dict[str, Any]:
        return {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "q_rank": self.q_rank,
                "rot": self.rot.to_dict() if self.rot else None, "rot_dim": self.rot_dim, "scale": self.scale,
                "vdim": self.vdim}


@dataclass(frozen=True)
class BiasAttentionConfig:
    """Grouped attention behind short convolutions (``conv`` taps) with a learned bias by distance, whose
    buckets reach up to ``bias_max``, and a window with kept first keys (``mask``; ``None``: every earlier key).
    ``buckets``: rows of the bias table (``None``: the checkpoint's)."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    conv: int
    bias_max: float
    mask: WindowMask | None
    buckets: int | None = None

    @classmethod
    def from_dict(cls, d: dict[str, Any], where: str) -> "BiasAttentionConfig":
        heads, kv_heads, dim, vdim = _heads(d, where)
        if max(dim, vdim) > MAX_HEAD:
            raise ConfigError(f"{where}: heads of more than {MAX_HEAD} elements are not supported, got {dim} / {vdim}")
        mask = d.get("mask")
        return cls(heads, kv_heads, dim, vdim, _number(d, "scale", where), _taps(d, where), _number(d, "bias_max", where),
                   WindowMask.from_dict(mask, where) if mask else None, _optional(d, "buckets", where))

    def to_dict(self) -> dict[str, Any]:
        whole = int(self.bias_max) if self.bias_max == int(self.bias_max) else self.bias_max
        out: dict[str, Any] = {"bias_max": whole}
        if self.buckets is not None:
            out["buckets"] = self.buckets
        out.update({"conv": self.conv, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads})
        if self.mask is not None:
            out["mask"] = self.mask.to_dict()
        out.update({"scale": self.scale, "vdim": self.vdim})
        return out


@dataclass(frozen=True)
class ChannelDeltaConfig:
    """``heads`` memories of ``dim`` x ``vdim`` written by the delta rule, a decay per head and key channel, over
    ``kv_heads`` query/key heads; ``conv`` taps.  ``a_rank``, ``g_rank``: ranks of the gates of decay and output
    (``None``: the checkpoint's)."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    a_rank: int | None = None
    g_rank: int | None = None

    @classmethod
    def from_dict(cls, d: dict[str, Any], where: str) -> "ChannelDeltaConfig":
        heads, dim = _positive(d, "heads", where), _key_size(d, "dim", where)
        return cls(heads, _shared_by(d, "kv_heads", heads, where), dim,
                   _positive(d, "vdim", where) if d.get("vdim") is not None else dim, _taps(d, where),
                   _optional(d, "a_rank", where), _optional(d, "g_rank", where))

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {}
        if self.a_rank is not None:
            out["a_rank"] = self.a_rank
        out.update({"conv": self.conv, "dim": self.dim})
        if self.g_rank is not None:
            out["g_rank"] = self.g_rank
        out.update({"heads": self.heads, "kv_heads": self.kv_heads, "vdim": self.vdim})
        return out


@dataclass(frozen=True)
class NormedPairConfig:
    """Half the sum of two mixers' outputs, each first normed over the width."""

    left: BiasAttentionConfig
    right: ChannelDeltaConfig

    @classmethod
    def from_dict(cls, d: dict[str, Any], where: str) -> "NormedPairConfig":
        return cls(BiasAttentionConfig.from_dict(_require(d, "left"), where + " (left)"),
                   ChannelDeltaConfig.from_dict(_require(d, "right"), where + " (right)"))

    def to_dict(self) -> dict[str, Any]:
        return {"left": self.left.to_dict(), "right": self.right.to_dict()}


@dataclass(frozen=True)
class DepolixMlpConfig:
    """``kind`` ``"dense"``: a gated feed-forward of width ``ff`` with biases, its pairs limited by ``limit``.
    ``"moe"``: ``experts`` of them without biases, of which a token uses the ``top`` of largest router logit."""

    kind: str
    ff: int
    limit: float
    experts: int = 0
    top: int = 0

    @classmethod
    def from_dict(cls, d: dict[str, Any], where: str) -> "DepolixMlpConfig":
        kind = _require(d, "kind")
        if kind == "dense":
            return cls("dense", _positive(d, "ff", where), _number(d, "limit", where))
        if kind != "moe":
            raise ConfigError(f"{where}: feed-forward kind {kind!r} is not supported (known: ('dense', 'moe'))")
        r, e = _require(d, "router"), _require(d, "expert")
        experts, top = _positive(r, "experts", where), _positive(r, "top", where)
        if top > experts:
            raise ConfigError(f"{where}: router.top ({top}) exceeds the {experts} experts")
        return cls("moe", _positive(e, "ff", where), _number(e, "limit", where), experts, top)

    def to_dict(self) -> dict[str, Any]:
        if self.kind == "dense":
            return {"ff": self.ff, "kind": "dense", "limit": self.limit}
        return {"expert": {"ff": self.ff, "limit": self.limit}, "kind": "moe",
                "router": {"experts": self.experts, "top": self.top}}


@dataclass(frozen=True)
class DepolixLayerConfig:
    type: str
    mixer: "QueryLatentConfig | NormedPairConfig"
    mlp: DepolixMlpConfig | None

    MIXERS = {"latent_attention": QueryLatentConfig, "parallel": NormedPairConfig}

    @classmethod
    def from_dict(cls, d: dict[str, Any], index: int) -> "DepolixLayerConfig":
        where = f"layer {index}"
        kind = _require(d, "type")
        if kind not in cls.MIXERS:
            raise ConfigError(f"{where}: mixer type {kind!r} is not supported (known: {tuple(cls.MIXERS)})")
        mlp = d.get("mlp")
        return cls(kind, cls.MIXERS[kind].from_dict(_require(d, "mixer"), where),
                   DepolixMlpConfig.from_dict(mlp, where) if mlp is not None else None)

    def to_dict(self) -> dict[str, Any]:
        return {"mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None, "type": self.type}


@dataclass
class DepolixConfig(ModelConfig):
    """``vocab_size`` of the base class is the file's ``vocab``."""

    width: int = 0
    norm_eps: float = 0.0
    embedding_scale: float = 1.0
    residual_mult: float = 1.0
    logit_scale: float = 1.0
    layers: list[DepolixLayerConfig] = field(default_factory=list)

    NAME = "Depolix"

    def __post_init__(self) -> None:
        if self.width <= 0 or self.vocab_size <= 0 or self.max_position_embeddings <= 0:
            raise ConfigError("vocab, width and max_positions must be positive")
        if not self.layers:
            raise ConfigError("a model needs at least one layer")

    @classmethod
    def from_dict(cls, d: dict[str, Any]) -> "DepolixConfig":
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
            embedding_scale=_number(_require(d, "embedding"), "scale", "embedding", positive=False),
            residual_mult=_number(d, "residual_mult", "config.json", positive=False),
            logit_scale=_number(d, "logit_scale", "config.json"),
            layers=[DepolixLayerConfig.from_dict(x, i) for i, x in enumerate(layers)])

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "architecture": self.NAME,
            "embedding": {"scale": self.embedding_scale},
            "layers": [x.to_dict() for x in self.layers],
            "logit_scale": self.logit_scale,
            "max_positions": self.max_position_embeddings,
            "norm": {"eps": self.norm_eps},
            "residual_mult": self.residual_mult,
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
