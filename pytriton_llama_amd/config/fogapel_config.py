"""Typed configuration of the Fogapel design: a list of layers, each with one of two mixers (softmax
attention inside chunks behind short convolutions; the time mixer of RWKV) and a dense, a routed or
no feed-forward beside it, and a scaled embedding. Every size and every constant that can
differ between models of the design is read from config.json (the rank of the time mixer's decays
from the checkpoint); nothing is defaulted from a known model.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .model_config import ConfigError
from .rubasun_config import _need
from .virusun_config import _positive


@dataclass(frozen=True)
class ConvAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    conv: int                  # taps of the convolutions behind the projections; 0: none
    rot_dims: int              # entries of a head that turn; 0: none
    rot_base: float
    softcap: Optional[float]   # bound on the scores; None: none
    chunk: Optional[int]       # a query sees the tokens of its own chunk of so many; None: all before it

    @classmethod
    def from_dict(cls, d, where) -> "ConvAttentionConfig":
        mask, rot, cap, conv = d.get("mask"), d.get("rot"), d.get("softcap"), d.get("conv")
        c = cls(heads=int(_need(d, "heads", where)), kv_heads=int(_need(d, "kv_heads", where)),
                dim=int(_need(d, "dim", where)), vdim=int(_need(d, "vdim", where)),
                scale=float(_need(d, "scale", where)), conv=0 if conv is None else int(conv),
                rot_dims=0 if rot is None else int(_need(rot, "dims", where + ".rot")),
                rot_base=1.0 if rot is None else float(_need(rot, "base", where + ".rot")),
                softcap=None if cap is None else float(cap),
                chunk=None if mask is None else int(_need(mask, "size", where + ".mask")))
        _positive(where, heads=c.heads, kv_heads=c.kv_heads, dim=c.dim, vdim=c.vdim)
        if c.heads % c.kv_heads:
            raise ConfigError(f"{where}: {c.heads} heads are not a multiple of {c.kv_heads} kv_heads")
        if c.conv < 0 or (conv is not None and c.conv == 0):
            raise ConfigError(f"{where}: conv must be positive")
        if c.rot_dims % 2 or not 0 <= c.rot_dims <= c.dim:
            raise ConfigError(f"{where}: rot.dims {c.rot_dims} must be even and at most dim {c.dim}")
        if c.rot_base <= 0:
            raise ConfigError(f"{where}: rot.base must be positive")
        if c.softcap is not None and c.softcap <= 0:
            raise ConfigError(f"{where}: softcap must be positive")
        if c.chunk is not None and c.chunk <= 0:
            raise ConfigError(f"{where}.mask: size must be positive")
        return c


@dataclass(frozen=True)
class TimeMixerConfig:
    heads: int
    dim: int
    rank: Optional[int]        # rows of the decays' first projection; None: the checkpoint says

    @classmethod
    def from_dict(cls, d, where) -> "TimeMixerConfig":
        c = cls(heads=int(_need(d, "heads", where)), dim=int(_need(d, "dim", where)),
                rank=None if d.get("rank") is None else int(d["rank"]))
        _positive(where, heads=c.heads, dim=c.dim)
        if c.rank is not None:
            _positive(where, rank=c.rank)
        return c


MIXER_CONFIGS = {"attention": ConvAttentionConfig, "wkv": TimeMixerConfig}


@dataclass(frozen=True)
class FogapelMlpConfig:
    kind: str                  # "dense" | "moe"
    ff: int                    # dense: its own; moe: an expert's
    limit: float = 0.0         # dense
    experts: int = 0           # moe
    top: int = 0
    shared_ff: int = 0         # 0: no shared expert

    @classmethod
    def from_dict(cls, d, where) -> Optional["FogapelMlpConfig"]:
        if d is None:
            return None
        kind = _need(d, "kind", where)
        if kind == "dense":
            c = cls("dense", int(_need(d, "ff", where)), limit=float(_need(d, "limit", where)))
            _positive(where, ff=c.ff, limit=c.limit)
            return c
        if kind != "moe":
            raise ConfigError(f"{where}: unknown feed-forward kind {kind!r} (known: 'dense', 'moe')")
        router, shared = _need(d, "router", where), d.get("shared")
        c = cls("moe", int(_need(_need(d, "expert", where), "ff", where + ".expert")),
                experts=int(_need(router, "experts", where + ".router")), top=int(_need(router, "top", where + ".router")),
                shared_ff=0 if shared is None else int(_need(shared, "ff", where + ".shared")))
        _positive(where, ff=c.ff)
        if shared is not None:
            _positive(where + ".shared", ff=c.shared_ff)
        if not 0 < c.top <= c.experts:
            raise ConfigError(f"{where}: top {c.top} of {c.experts} experts")
        return c


@dataclass(frozen=True)
class FogapelLayerConfig:
    kind: str                  # "attention" | "wkv"
    mixer: Any
    mlp: Optional[FogapelMlpConfig]


@dataclass(frozen=True)
class FogapelConfig:
    vocab_size: int
    hidden_size: int
    norm_eps: float
    embedding_scale: float
    layers: Tuple[FogapelLayerConfig, ...]
    eos_token_id: Any = None
    initializer_range: float = 0.05
    architectures: Tuple[str, ...] = ("Fogapel",)
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
    def from_dict(cls, d: Dict[str, Any]) -> "FogapelConfig":
        layers = []
        for i, e in enumerate(_need(d, "layers", "the model")):
            where = f"layers[{i}]"
            kind = _need(e, "type", where)
            if kind not in MIXER_CONFIGS:
                raise ConfigError(f"{where}: unknown layer type {kind!r} (known: {sorted(MIXER_CONFIGS)})")
            layers.append(FogapelLayerConfig(
                kind, MIXER_CONFIGS[kind].from_dict(_need(e, "mixer", where), where + ".mixer"),
                FogapelMlpConfig.from_dict(e.get("mlp"), where + ".mlp")))
        if not layers:
            raise ConfigError("config.json: 'layers' is empty")
        cfg = cls(vocab_size=int(_need(d, "vocab", "the model")), hidden_size=int(_need(d, "width", "the model")),
                  norm_eps=float(_need(_need(d, "norm", "the model"), "eps", "norm")),
                  embedding_scale=float(_need(_need(d, "embedding", "the model"), "scale", "embedding")),
                  layers=tuple(layers), eos_token_id=d.get("eos_token_id"),
                  initializer_range=float(d.get("initializer_range", 0.05)), raw=dict(d))
        if cfg.vocab_size <= 0 or cfg.hidden_size <= 0 or cfg.norm_eps < 0:
            raise ConfigError("vocab and width must be positive, norm.eps not negative")
        return cfg

    def to_dict(self) -> Dict[str, Any]:
        return dict(self.raw)
