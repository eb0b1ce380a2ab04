"""Typed configuration of the Roserax architecture, read from its config.json.

The file names every size and every constant that may differ between models of the design: ``vocab``, ``width``,
``embedding.scale``, ``logit_scale``, ``norm.eps`` and a list ``layers`` whose entries give a ``type`` (the kind of
mixer: ``attention``, ``latent_attention`` or ``retention``), the sizes and constants of that mixer (``mixer``) and, where
there is one, a feed-forward (``mlp``: ``kind`` ``dense`` or ``moe``).  Features that may be left out: an attention layer's ``mask`` (it then
sees every earlier position), the mask's ``keep_first``, a router's ``groups``, a retention layer's ``rot``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple, Union

from ..errors import ConfigError, UnsupportedModelError
from .base import ConfigReader

DEFAULT_MAX_POSITIONS = 1 << 20      # nothing in the design bounds a position: a bound for the block tables only


def _required(r: ConfigReader, key: str) -> ConfigReader:
    m = r.mapping(key)
    if m is None:
        raise ConfigError(f"{r.where}: required key '{key}' is missing")
    return m


@dataclass(frozen=True)
class RotationConfig:
    base: float
    dims: int

    @classmethod
    def read(cls, r: ConfigReader, width: int) -> "RotationConfig":
        cfg = cls(r.number("base"), r.integer("dims"))
        if cfg.dims % 2 or cfg.dims > width:
            raise ConfigError(f"{r.where}: dims ({cfg.dims}) must be even and within the {width} features of a head")
        return cfg

    def to_dict(self) -> dict:
        return {"base": self.base, "dims": self.dims}


@dataclass(frozen=True)
class KeptWindowAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int]         # None: every earlier position is seen
    keep_first: int

    @classmethod
    def read(cls, r: ConfigReader) -> "KeptWindowAttentionConfig":
        mask = r.mapping("mask")
        cfg = cls(heads=r.integer("heads"), kv_heads=r.integer("kv_heads"), dim=r.integer("dim"), vdim=r.integer("vdim"),
                  scale=r.number("scale"), window=mask.integer("size") if mask is not None else None,
                  keep_first=mask.integer("keep_first", 0, minimum=0) if mask is not None else 0)
        if cfg.heads % cfg.kv_heads:
            raise ConfigError(f"{r.where}: heads ({cfg.heads}) must be a multiple of kv_heads ({cfg.kv_heads})")
        return cfg

    def to_dict(self) -> dict:
        d = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.vdim}
        if self.window is not None:
            d["mask"] = {"keep_first": self.keep_first, "size": self.window}
        return d


@dataclass(frozen=True)
class GatedLatentAttentionConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot: RotationConfig

    @classmethod
    def read(cls, r: ConfigReader) -> "GatedLatentAttentionConfig":
        rot_dim = r.integer("rot_dim")
        rot = RotationConfig.read(_required(r, "rot"), rot_dim)
        if rot.dims != rot_dim:
            raise ConfigError(f"{r.where}: rot.dims ({rot.dims}) must equal rot_dim ({rot_dim})")
        return cls(heads=r.integer("heads"), dim=r.integer("dim"), rot_dim=rot_dim, vdim=r.integer("vdim"), q_rank=r.integer("q_rank"),
                   kv_rank=r.integer("kv_rank"), scale=r.number("scale"), rot=rot)

    def to_dict(self) -> dict:
        return {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "q_rank": self.q_rank, "rot": self.rot.to_dict(),
                "rot_dim": self.rot_dim, "scale": self.scale, "vdim": self.vdim}


@dataclass(frozen=True)
class RetentionConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    rot: Optional[RotationConfig]

    @classmethod
    def read(cls, r: ConfigReader) -> "RetentionConfig":
        heads, dim = r.integer("heads"), r.integer("dim")
        decay = r.raw.get("decay")
        if not isinstance(decay, (list, tuple)) or len(decay) != heads or any(isinstance(d, bool) or not isinstance(d, (int, float)) or not 0.0 <= d <= 1.0
                                                                              for d in decay):
            raise ConfigError(f"{r.where}: 'decay' must list {heads} numbers between 0 and 1, got {decay!r}")
        rot = r.mapping("rot")
        return cls(heads, dim, r.integer("vdim"), tuple(float(d) for d in decay), RotationConfig.read(rot, dim) if rot is not None else None)

    def to_dict(self) -> dict:
        d = {"decay": list(self.decay), "dim": self.dim, "heads": self.heads, "vdim": self.vdim}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclass(frozen=True)
class RoseraxFeedForward:
    kind: str
    ff: int
    experts: int = 0
    top: int = 0
    groups: int = 1
    keep: int = 1

    @classmethod
    def read(cls, r: ConfigReader) -> "RoseraxFeedForward":
        kind = r.string("kind")
        if kind == "dense":
            return cls(kind, r.integer("ff"))
        if kind != "moe":
            raise UnsupportedModelError(f"{r.where}: feed-forward kind '{kind}' is not known (dense, moe)")
        router = _required(r, "router")
        groups = router.mapping("groups")
        cfg = cls(kind, _required(r, "expert").integer("ff"), router.integer("experts"), router.integer("top"),
                  groups.integer("count") if groups is not None else 1, groups.integer("keep") if groups is not None else 1)
        if cfg.experts % cfg.groups or cfg.keep > cfg.groups or cfg.top > cfg.experts // cfg.groups * cfg.keep:
            raise ConfigError(f"{r.where}: {cfg.experts} experts in {cfg.groups} groups of which {cfg.keep} are kept cannot give {cfg.top} choices")
        return cfg

    def to_dict(self) -> dict:
        if self.kind == "dense":
            return {"ff": self.ff, "kind": "dense"}
        router = {"experts": self.experts, "top": self.top}
        if self.groups > 1:
            router["groups"] = {"count": self.groups, "keep": self.keep}
        return {"expert": {"ff": self.ff}, "kind": "moe", "router": router}


MIXER_CONFIGS = {"attention": KeptWindowAttentionConfig, "latent_attention": GatedLatentAttentionConfig, "retention": RetentionConfig}
RoseraxMixer = Union[KeptWindowAttentionConfig, GatedLatentAttentionConfig, RetentionConfig]


@dataclass(frozen=True)
class RoseraxLayer:
    type: str
    mixer: RoseraxMixer
    mlp: Optional[RoseraxFeedForward]

    @classmethod
    def read(cls, r: ConfigReader) -> "RoseraxLayer":
        kind = r.string("type")
        if kind not in MIXER_CONFIGS:
            raise UnsupportedModelError(f"{r.where}: layer type '{kind}' is not known ({', '.join(sorted(MIXER_CONFIGS))})")
        mlp = r.mapping("mlp")
        return cls(kind, MIXER_CONFIGS[kind].read(_required(r, "mixer")), RoseraxFeedForward.read(mlp) if mlp is not None else None)

    def to_dict(self) -> dict:
        return {"mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp is not None else None, "type": self.type}


@dataclass(frozen=True)
class RoseraxConfig:
    architecture: str
    vocab: int
    width: int
    embedding_scale: float
    logit_scale: float
    norm_eps: float
    layers: Tuple[RoseraxLayer, ...]
    max_positions: int = DEFAULT_MAX_POSITIONS

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str = "config.json") -> "RoseraxConfig":
        r = ConfigReader(raw, where)
        entries = raw.get("layers")
        if not isinstance(entries, (list, tuple)) or not entries:
            raise ConfigError(f"{where}: 'layers' must be a non-empty list")
        layers = tuple(RoseraxLayer.read(ConfigReader(e, f"{where}:layers[{i}]")) for i, e in enumerate(entries))
        return cls(architecture=r.string("architecture", "Roserax"), vocab=r.integer("vocab"), width=r.integer("width"),
                   embedding_scale=_required(r, "embedding").number("scale", positive=False), logit_scale=r.number("logit_scale", positive=False),
                   norm_eps=_required(r, "norm").number("eps"), layers=layers, max_positions=r.integer("max_positions", DEFAULT_MAX_POSITIONS))

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale}, "layers": [l.to_dict() for l in self.layers],
             "logit_scale": self.logit_scale, "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width}
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
