"""Typed configuration of the Tukedra decoder.

config.json names the design in `architecture` and gives `vocab`, `width`, `streams` (copies of the residual),
`norm.eps`, optionally `embedding.scale`, `logit_scale`, `logit_softcap` (none: logits are not capped), and `layers`,
one entry a layer: `type`, `mixer` and `mlp`.

* type "lightning": linear attention with a fixed decay a head.  `mixer`: `heads`, `dim`, `vdim`, `decay` (a number a
  head).
* type "retention": the same keys and `rot` (`base`, `dims`): queries and keys are rotated by position.
* type "attention": softmax attention within chunks of positions whose values are its keys.  `mixer`: `heads`,
  `kv_heads`, `dim` (`vdim` is `dim`), `scale`, `rot` (`base`, `dims`, optionally `scaling`: `factor`, `original`,
  `fast`, `slow`) and `mask.size` (the chunk; no `mask`: every earlier position).
* `mlp`: `{"kind": "dense", "ff"}`, `{"kind": "moe", "expert": {"ff"}, "router": {"experts", "top"}, "shared": {"ff"}}`
  (`shared` may be absent) or null.

Every error names its key.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .base import ConfigError, ModelConfig, coerce
from .vupelorn import Rotary, _get

LINEAR_TYPES = ("lightning", "retention")


@dataclass(frozen=True)
class LinearHeads:
    """A layer of linear attention; `rot` is set for the kind that rotates its queries and keys."""
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    rot: Optional[Rotary]

    @classmethod
    def from_dict(cls, d, where, rotates: bool):
        heads = _get(d, "heads", where, least=1)
        dim = _get(d, "dim", where, least=1)
        decay = d.get("decay")
        if not isinstance(decay, list) or len(decay) != heads:
            raise ConfigError(f"config.json: '{where}.decay' must be a list of {heads} numbers, one a head, found {decay!r}")
        decay = tuple(coerce(v, f"{where}.decay", float) for v in decay)
        if not all(0.0 <= v <= 1.0 for v in decay):
            raise ConfigError(f"config.json: '{where}.decay' must lie between 0 and 1, found {list(decay)}")
        rot = None
        if rotates:
            rot = Rotary.from_dict(d.get("rot"), where + ".rot", whole=dim - dim % 2)
            if rot.dims > dim:
                raise ConfigError(f"config.json: '{where}.rot.dims' ({rot.dims}) is more than dim ({dim})")
        return cls(heads, dim, _get(d, "vdim", where, least=1, default=dim), decay, rot)

    def to_dict(self):
        d: Dict[str, Any] = {"decay": list(self.decay), "dim": self.dim, "heads": self.heads, "vdim": self.vdim}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclass(frozen=True)
class ChunkedHeads:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    chunk: int  # 0: every earlier position
    rot: Optional[Rotary]

    @classmethod
    def from_dict(cls, d, where):
        heads = _get(d, "heads", where, least=1)
        dim = _get(d, "dim", where, least=1)
        mask, rot = d.get("mask"), d.get("rot")
        vdim = _get(d, "vdim", where, least=1, default=dim)
        c = cls(heads, _get(d, "kv_heads", where, least=1, default=heads), dim, _get(d, "scale", where, float),
                0 if mask is None else _get(mask, "size", where + ".mask", least=1),
                None if rot is None else Rotary.from_dict(rot, where + ".rot", whole=dim - dim % 2))
        if c.heads % c.kv_heads:
            raise ConfigError(f"config.json: '{where}.heads' ({c.heads}) is no multiple of kv_heads ({c.kv_heads})")
        if vdim != dim:
            raise ConfigError(f"config.json: '{where}.vdim' ({vdim}) must be dim ({dim}): the values are the keys")
        if c.rot is not None and c.rot.dims > dim:
            raise ConfigError(f"config.json: '{where}.rot.dims' ({c.rot.dims}) is more than dim ({dim})")
        return c

    def to_dict(self):
        d: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale,
                             "vdim": self.dim}
        if self.chunk:
            d["mask"] = {"size": self.chunk}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclass(frozen=True)
class TukedraFeedForward:
    kind: str  # "dense" | "moe"
    ff: int  # inner size (of an expert, for "moe")
    experts: int = 0
    top: int = 0
    shared_ff: int = 0  # 0: no shared expert

    @classmethod
    def from_dict(cls, d, where):
        kind = d.get("kind") if isinstance(d, dict) else None
        if kind == "dense":
            return cls("dense", _get(d, "ff", where, least=1))
        if kind != "moe":
            raise ConfigError(f"config.json: '{where}.kind' must be 'dense' or 'moe' (or mlp null), found {kind!r}")
        router, shared, w = d.get("router"), d.get("shared"), where + ".router"
        c = cls("moe", _get(d.get("expert"), "ff", where + ".expert", least=1), _get(router, "experts", w, least=1),
                _get(router, "top", w, least=1), 0 if shared is None else _get(shared, "ff", where + ".shared", least=1))
        if c.top > c.experts:
            raise ConfigError(f"config.json: '{w}.top' ({c.top}) is more than its {c.experts} experts")
        return c

    def to_dict(self):
        if self.kind == "dense":
            return {"ff": self.ff, "kind": "dense"}
        d: Dict[str, Any] = {"expert": {"ff": self.ff}, "kind": "moe",
                             "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff:
            d["shared"] = {"ff": self.shared_ff}
        return d


@dataclass(frozen=True)
class TukedraLayer:
    type: str  # "lightning" | "retention" | "attention"
    linear: Optional[LinearHeads]
    attention: Optional[ChunkedHeads]
    mlp: Optional[TukedraFeedForward]

    @classmethod
    def from_dict(cls, d, i: int):
        where = f"layers[{i}]"
        if not isinstance(d, dict):
            raise ConfigError(f"config.json: '{where}' must be an object")
        kind, mixer, mlp, w = d.get("type"), d.get("mixer"), d.get("mlp"), where + ".mixer"
        if kind not in LINEAR_TYPES + ("attention",):
            raise ConfigError(f"config.json: '{where}.type' must be 'lightning', 'retention' or 'attention', found {kind!r}")
        if not isinstance(mixer, dict):
            raise ConfigError(f"config.json: required key '{w}' is missing")
        return cls(kind, LinearHeads.from_dict(mixer, w, kind == "retention") if kind in LINEAR_TYPES else None,
                   ChunkedHeads.from_dict(mixer, w) if kind == "attention" else None,
                   None if mlp is None else TukedraFeedForward.from_dict(mlp, where + ".mlp"))

    def to_dict(self):
        return {"mixer": (self.linear or self.attention).to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict(),
                "type": self.type}


@dataclass(frozen=True)
class TukedraConfig(ModelConfig):
    vocab: int
    width: int
    streams: int
    norm_eps: float
    embedding_scale: float
    logit_scale: float
    logit_softcap: float  # 0: none
    layers: Tuple[TukedraLayer, ...]
    architecture: str = "Tukedra"

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "TukedraConfig":
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        if not isinstance(d.get("norm"), dict):
            raise ConfigError("config.json: 'norm' must be an object")
        emb = d.get("embedding")
        c = cls(vocab=_get(d, "vocab", "config", least=1), width=_get(d, "width", "config", least=1),
                streams=_get(d, "streams", "config", least=1), norm_eps=_get(d["norm"], "eps", "norm", float),
                embedding_scale=1.0 if emb is None else _get(emb, "scale", "embedding", float, default=1.0),
                logit_scale=_get(d, "logit_scale", "config", float, default=1.0),
                logit_softcap=_get(d, "logit_softcap", "config", float, default=0.0),
                layers=tuple(TukedraLayer.from_dict(x, i) for i, x in enumerate(layers)),
                architecture=str(d.get("architecture", "Tukedra")))
        if c.logit_softcap < 0:
            raise ConfigError(f"config.json: 'logit_softcap' must not be negative, found {c.logit_softcap}")
        return c

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale},
                             "layers": [x.to_dict() for x in self.layers], "logit_scale": self.logit_scale,
                             "norm": {"eps": self.norm_eps}, "streams": self.streams, "vocab": self.vocab,
                             "width": self.width}
        if self.logit_softcap:
            d["logit_softcap"] = self.logit_softcap
        return copy.deepcopy(d)
