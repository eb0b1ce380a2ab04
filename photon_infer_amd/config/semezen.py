"""Typed configuration of the Semezen architecture, read from its config.json.

The file names every size and every constant that may differ between models of the design:
``vocab``, ``width``, ``streams`` (how many copies of the residual stream run side by side), ``norm.eps``
and a list ``layers`` whose entries give a ``type`` (the kind of mixer: ``attention`` or
``mingru``), the sizes of that mixer (``mixer``) and, where the layer has one, its feed-forward (``mlp``: ``kind`` ``dense`` or
``moe``).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple, Union

from ..errors import ConfigError, UnsupportedModelError
from .base import ConfigReader
from .llama import RopeScaling

DEFAULT_MAX_POSITIONS = 1 << 20      # nothing in the design bounds a position: the rotation is computed, states have no length


@dataclass(frozen=True)
class WindowAttentionConfig:
    heads: int
    kv_heads: int
    dim: int                                # keys, and values: they are the keys as projected
    scale: float
    rot_dims: int                           # 0: no rotation
    rot_base: float
    rot_scaling: Optional[RopeScaling]      # None: frequencies as they are
    window: Optional[int]                   # None: every earlier position is seen

    @classmethod
    def read(cls, r: ConfigReader) -> "WindowAttentionConfig":
        rot, mask = r.mapping("rot"), r.mapping("mask")
        scaling = None
        sc = rot.mapping("scaling") if rot is not None else None
        if sc is not None:
            scaling = RopeScaling("llama3", sc.number("factor"), sc.number("low"), sc.number("high"), sc.integer("original"))
            if not scaling.high_freq_factor > scaling.low_freq_factor:
                raise ConfigError(f"{sc.where}: 'high' ({scaling.high_freq_factor}) must be above 'low' ({scaling.low_freq_factor})")
        cfg = cls(heads=r.integer("heads"), kv_heads=r.integer("kv_heads"), dim=r.integer("dim"), scale=r.number("scale"),
                  rot_dims=rot.integer("dims", minimum=0) if rot is not None else 0,
                  rot_base=rot.number("base") if rot is not None else 1.0, rot_scaling=scaling,
                  window=mask.integer("size") if mask is not None else None)
        if cfg.heads % cfg.kv_heads:
            raise ConfigError(f"{r.where}: heads ({cfg.heads}) must be a multiple of kv_heads ({cfg.kv_heads})")
        if r.integer("vdim", cfg.dim) != cfg.dim:
            raise ConfigError(f"{r.where}: vdim ({r.integer('vdim')}) must be dim ({cfg.dim}): the values are the keys")
        if cfg.rot_dims % 2 or cfg.rot_dims > cfg.dim:
            raise ConfigError(f"{r.where}: rot.dims ({cfg.rot_dims}) must be even and at most dim ({cfg.dim})")
        return cfg

    def to_dict(self) -> dict:
        d = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.dim}
        if self.window is not None:
            d["mask"] = {"size": self.window}
        if self.rot_dims:
            d["rot"] = {"base": self.rot_base, "dims": self.rot_dims}
            s = self.rot_scaling
            if s is not None:
                d["rot"]["scaling"] = {"factor": s.factor, "high": s.high_freq_factor, "low": s.low_freq_factor,
                                       "original": s.original_max_position_embeddings}
        return d


@dataclass(frozen=True)
class MinGruConfig:
    width: int

    @classmethod
    def read(cls, r: ConfigReader) -> "MinGruConfig":
        return cls(width=r.integer("width"))

    def to_dict(self) -> dict:
        return {"width": self.width}


@dataclass(frozen=True)
class MlpConfig:
    kind: str                      # "dense" or "moe"
    ff: int                        # dense: the unit's width; moe: an expert's
    limit: float = 0.0             # moe: where an expert's gate and up values are clamped
    experts: int = 0
    top: int = 0

    @classmethod
    def read(cls, r: ConfigReader) -> "MlpConfig":
        kind = r.string("kind")
        if kind == "dense":
            return cls(kind, r.integer("ff"))
        if kind != "moe":
            raise UnsupportedModelError(f"{r.where}: feed-forward kind '{kind}' is not known (dense, moe)")
        expert, router = r.mapping("expert"), r.mapping("router")
        if expert is None or router is None:
            raise ConfigError(f"{r.where}: a mixture of experts needs 'expert' and 'router'")
        cfg = cls(kind, expert.integer("ff"), limit=expert.number("limit"), experts=router.integer("experts"), top=router.integer("top"))
        if cfg.top > cfg.experts:
            raise ConfigError(f"{r.where}: router.top ({cfg.top}) is more than the {cfg.experts} experts")
        return cfg

    def to_dict(self) -> dict:
        if self.kind == "dense":
            return {"ff": self.ff, "kind": self.kind}
        return {"expert": {"ff": self.ff, "limit": self.limit}, "kind": self.kind, "router": {"experts": self.experts, "top": self.top}}


MIXER_CONFIGS = {"attention": WindowAttentionConfig, "mingru": MinGruConfig}


@dataclass(frozen=True)
class SemezenLayer:
    type: str
    mixer: Union[WindowAttentionConfig, MinGruConfig]
    mlp: Optional[MlpConfig]

    @classmethod
    def read(cls, r: ConfigReader) -> "SemezenLayer":
        kind = r.string("type")
        if kind not in MIXER_CONFIGS:
            raise UnsupportedModelError(f"{r.where}: layer type '{kind}' is not known ({', '.join(sorted(MIXER_CONFIGS))})")
        mixer = r.mapping("mixer")
        if mixer is None:
            raise ConfigError(f"{r.where}: required key 'mixer' is missing")
        mlp = r.mapping("mlp")
        return cls(kind, MIXER_CONFIGS[kind].read(mixer), MlpConfig.read(mlp) if mlp is not None else None)

    def to_dict(self) -> dict:
        return {"mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp is not None else None, "type": self.type}


@dataclass(frozen=True)
class SemezenConfig:
    architecture: str
    vocab: int
    width: int
    streams: int
    norm_eps: float
    layers: Tuple[SemezenLayer, ...]
    max_positions: int = DEFAULT_MAX_POSITIONS

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str = "config.json") -> "SemezenConfig":
        r = ConfigReader(raw, where)
        norm = r.mapping("norm")
        if norm is None:
            raise ConfigError(f"{where}: required key 'norm' is an object")
        entries = raw.get("layers")
        if not isinstance(entries, (list, tuple)) or not entries:
            raise ConfigError(f"{where}: 'layers' must be a non-empty list")
        return cls(architecture=r.string("architecture", "Semezen"), vocab=r.integer("vocab"), width=r.integer("width"),
                   streams=r.integer("streams"), norm_eps=norm.number("eps"),
                   layers=tuple(SemezenLayer.read(ConfigReader(e, f"{where}:layers[{i}]")) for i, e in enumerate(entries)),
                   max_positions=r.integer("max_positions", DEFAULT_MAX_POSITIONS))

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "layers": [l.to_dict() for l in self.layers], "norm": {"eps": self.norm_eps},
             "streams": self.streams, "vocab": self.vocab, "width": self.width}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            d["max_positions"] = self.max_positions
        return d

    # what the engine's front ends ask of any configuration
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width
