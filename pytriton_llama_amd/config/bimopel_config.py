"""Typed configuration of the Bimopel design: a list of layers, each with one of two mixers (Mamba-2;
softmax attention inside chunks and gated linear attention side by side) and a dense feed-forward
or none, an RMS norm behind every residual sum, sinusoidal positions at the embedding and capped
logits. Every size and every constant that can differ between models of the design is read from
config.json (the rank of the decays' projection from the checkpoint); nothing is defaulted from a
known model.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .model_config import ConfigError
from .rubasun_config import _need
from .virusun_config import _positive


@dataclass(frozen=True)
class Mamba2Config:
    heads: int
    vdim: int                  # values a head
    state: int                 # state entries a value
    groups: int                # B and C are shared by the heads of a group
    conv: int                  # taps of the causal convolution
    norm_groups: int           # equal parts of the heads' values that are normed on their own

    @classmethod
    def from_dict(cls, d, where) -> "Mamba2Config":
        c = cls(**{k: int(_need(d, k, where)) for k in ("heads", "vdim", "state", "groups", "conv", "norm_groups")})
        _positive(where, heads=c.heads, vdim=c.vdim, state=c.state, groups=c.groups, conv=c.conv,
                  norm_groups=c.norm_groups)
        if c.heads % c.groups:
            raise ConfigError(f"{where}: {c.heads} heads are not a multiple of {c.groups} groups")
        if (c.heads * c.vdim) % c.norm_groups:
            raise ConfigError(f"{where}: {c.heads} heads of {c.vdim} do not divide into {c.norm_groups} norm_groups")
        return c


@dataclass(frozen=True)
class ChunkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: Optional[int]       # a query sees the tokens of its own chunk of so many; None: all before it

    @classmethod
    def from_dict(cls, d, where) -> "ChunkAttentionConfig":
        mask = d.get("mask")
        c = cls(heads=int(_need(d, "heads", where)), kv_heads=int(_need(d, "kv_heads", where)),
                dim=int(_need(d, "dim", where)), vdim=int(_need(d, "vdim", where)),
                scale=float(_need(d, "scale", where)),
                chunk=None if mask is None else int(_need(mask, "size", where + ".mask")))
        _positive(where, heads=c.heads, kv_heads=c.kv_heads, dim=c.dim, vdim=c.vdim)
        if c.heads % c.kv_heads:
            raise ConfigError(f"{where}: {c.heads} heads are not a multiple of {c.kv_heads} kv_heads")
        if c.chunk is not None and c.chunk <= 0:
            raise ConfigError(f"{where}.mask: size must be positive")
        return c


@dataclass(frozen=True)
class GatedLinearConfig:
    heads: int
    dim: int
    vdim: int
    tau: float
    rank: Optional[int]        # rows of the decays' first projection; None: the checkpoint says

    @classmethod
    def from_dict(cls, d, where) -> "GatedLinearConfig":
        c = cls(heads=int(_need(d, "heads", where)), dim=int(_need(d, "dim", where)),
                vdim=int(_need(d, "vdim", where)), tau=float(_need(d, "tau", where)),
                rank=None if d.get("rank") is None else int(d["rank"]))
        _positive(where, heads=c.heads, dim=c.dim, vdim=c.vdim, tau=c.tau)
        if c.rank is not None:
            _positive(where, rank=c.rank)
        return c


@dataclass(frozen=True)
class ChunkParallelConfig:
    left: ChunkAttentionConfig
    right: GatedLinearConfig

    @classmethod
    def from_dict(cls, d, where) -> "ChunkParallelConfig":
        return cls(left=ChunkAttentionConfig.from_dict(_need(d, "left", where), where + ".left"),
                   right=GatedLinearConfig.from_dict(_need(d, "right", where), where + ".right"))


MIXER_CONFIGS = {"mamba2": Mamba2Config, "parallel": ChunkParallelConfig}


@dataclass(frozen=True)
class BimopelLayerConfig:
    kind: str                  # "mamba2" | "parallel"
    mixer: Any
    ff: int                    # 0: no feed-forward


@dataclass(frozen=True)
class BimopelConfig:
    vocab_size: int
    hidden_size: int
    norm_eps: float
    embedding_scale: float
    postln_alpha: float        # factor on the stream in front of every residual sum
    logit_softcap: Optional[float]
    layers: Tuple[BimopelLayerConfig, ...]
    eos_token_id: Any = None
    initializer_range: float = 0.05
    architectures: Tuple[str, ...] = ("Bimopel",)
    raw: Any = None

    @property
    def eos_token_ids(self) -> Tuple[int, ...]:
        e = self.eos_token_id
        if e is None:
            return ()
        return tuple(int(x) for x in e) if isinstance(e, (list, tuple)) else (int(e),)

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "BimopelConfig":
        layers = []
        for i, e in enumerate(_need(d, "layers", "the model")):
            where = f"layers[{i}]"
            kind = _need(e, "type", where)
            if kind not in MIXER_CONFIGS:
                raise ConfigError(f"{where}: unknown layer type {kind!r} (known: {sorted(MIXER_CONFIGS)})")
            m = MIXER_CONFIGS[kind].from_dict(_need(e, "mixer", where), where + ".mixer")
            mlp, ff = e.get("mlp"), 0
            if mlp is not None:
                if _need(mlp, "kind", where + ".mlp") != "dense":
                    raise ConfigError(f"{where}.mlp: unknown feed-forward kind {mlp['kind']!r} (known: 'dense')")
                ff = int(_need(mlp, "ff", where + ".mlp"))
                _positive(where + ".mlp", ff=ff)
            layers.append(BimopelLayerConfig(kind, m, ff))
        if not layers:
            raise ConfigError("config.json: 'layers' is empty")
        cap = d.get("logit_softcap")
        cfg = cls(vocab_size=int(_need(d, "vocab", "the model")), hidden_size=int(_need(d, "width", "the model")),
                  norm_eps=float(_need(_need(d, "norm", "the model"), "eps", "norm")),
                  embedding_scale=float(_need(_need(d, "embedding", "the model"), "scale", "embedding")),
                  postln_alpha=float(_need(d, "postln_alpha", "the model")),
                  logit_softcap=None if cap is None else float(cap), layers=tuple(layers),
                  eos_token_id=d.get("eos_token_id"), initializer_range=float(d.get("initializer_range", 0.05)),
                  raw=dict(d))
        if cfg.vocab_size <= 0 or cfg.hidden_size <= 0 or cfg.norm_eps < 0:
            raise ConfigError("vocab and width must be positive, norm.eps not negative")
        if cfg.logit_softcap is not None and cfg.logit_softcap <= 0:
            raise ConfigError("logit_softcap must be positive")
        return cfg

    def to_dict(self) -> Dict[str, Any]:
        return dict(self.raw)
