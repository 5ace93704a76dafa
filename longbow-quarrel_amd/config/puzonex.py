"""Typed configuration of the Puzonex decoder.

config.json names the design in `architecture` and gives `vocab`, `width`, `norm.eps` and `layers`, one entry a layer:
`type`, `mixer` and `mlp`.

* type "attention": windowed softmax attention with a learned sink and a logarithmic distance bias.  `mixer`: `heads`,
  `kv_heads`, `dim`, `vdim`, `scale`, `softcap` (none: scores are not capped) and `mask.size` (the sliding window; no
  `mask`: every earlier position).
* type "mamba1": the selective scan.  `mixer`: `inner`, `state`, `dt_rank`, `conv` (taps).
* type "parallel": `mixer.left` is windowed attention whose values are its keys (the keys above and `bias_max`, the
  distance at which its table of biases ends; `vdim` is `dim`), `mixer.right` a matrix memory (`heads`, `dim`, `vdim`,
  `gate_cap`).
* `mlp`: `{"kind": "dense", "ff"}` or null.

One size is in no key, the number of rows of a left side's table of biases: the shape of its tensor gives it
(`completed`); `left.bias_rows` may state it, which a configuration without a file needs.  Every error names its key.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, replace
from typing import Any, Dict, Mapping, Optional, Tuple

from .base import ConfigError, ModelConfig
from .vupelorn import _get


@dataclass(frozen=True)
class ShapedHeads:
    """Sizes and constants of softmax attention; `bias_max` is set for the kind whose values are its keys."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float  # 0: none
    window: int  # 0: every earlier position
    bias_max: Optional[float] = None
    bias_rows: Optional[int] = None

    @classmethod
    def from_dict(cls, d, where, tied_values: bool):
        if not isinstance(d, dict):
            raise ConfigError(f"config.json: required key '{where}' is missing")
        heads = _get(d, "heads", where, least=1)
        dim = _get(d, "dim", where, least=1)
        mask = d.get("mask")
        c = cls(heads, _get(d, "kv_heads", where, least=1, default=heads), dim,
                _get(d, "vdim", where, least=1, default=dim), _get(d, "scale", where, float),
                _get(d, "softcap", where, float, default=0.0),
                0 if mask is None else _get(mask, "size", where + ".mask", least=1),
                _get(d, "bias_max", where, float) if tied_values else None,
                _get(d, "bias_rows", where, least=2, default=None) if tied_values else None)
        if c.heads % c.kv_heads:
            raise ConfigError(f"config.json: '{where}.heads' ({c.heads}) is no multiple of kv_heads ({c.kv_heads})")
        if c.softcap < 0:
            raise ConfigError(f"config.json: '{where}.softcap' must not be negative, found {c.softcap}")
        if tied_values and c.vdim != c.dim:
            raise ConfigError(f"config.json: '{where}.vdim' ({c.vdim}) must be dim ({c.dim}): the values are the keys")
        c.check_bias(where)
        return c

    def check_bias(self, where: str) -> None:
        if self.bias_rows is not None and not self.bias_max > self.bias_rows // 2:
            raise ConfigError(f"config.json: '{where}.bias_max' ({self.bias_max}) must be beyond the {self.bias_rows // 2} "
                              "distances that have a row of their own")

    def to_dict(self):
        d: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale,
                             "vdim": self.vdim}
        if self.softcap:
            d["softcap"] = self.softcap
        if self.window:
            d["mask"] = {"size": self.window}
        if self.bias_max is not None:
            d["bias_max"] = self.bias_max
        if self.bias_rows is not None:
            d["bias_rows"] = self.bias_rows
        return d


@dataclass(frozen=True)
class SelectiveLayer:
    inner: int
    state: int
    dt_rank: int
    conv: int

    @classmethod
    def from_dict(cls, d, where):
        return cls(*(_get(d, key, where, least=1) for key in ("inner", "state", "dt_rank", "conv")))

    def to_dict(self):
        return {"conv": self.conv, "dt_rank": self.dt_rank, "inner": self.inner, "state": self.state}


@dataclass(frozen=True)
class MemorySide:
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    @classmethod
    def from_dict(cls, d, where):
        dim = _get(d, "dim", where, least=1)
        c = cls(_get(d, "heads", where, least=1), dim, _get(d, "vdim", where, least=1, default=dim),
                _get(d, "gate_cap", where, float))
        if not c.gate_cap > 0:
            raise ConfigError(f"config.json: '{where}.gate_cap' must be positive, found {c.gate_cap}")
        return c

    def to_dict(self):
        return {"dim": self.dim, "gate_cap": self.gate_cap, "heads": self.heads, "vdim": self.vdim}


@dataclass(frozen=True)
class PuzonexLayer:
    type: str  # "attention" | "mamba1" | "parallel"
    attention: Optional[ShapedHeads]
    selective: Optional[SelectiveLayer]
    left: Optional[ShapedHeads]
    right: Optional[MemorySide]
    ff: Optional[int]  # the feed-forward's inner size; None: the layer has none

    @classmethod
    def from_dict(cls, d, i: int):
        where = f"layers[{i}]"
        if not isinstance(d, dict):
            raise ConfigError(f"config.json: '{where}' must be an object")
        kind, mixer, w, mlp = d.get("type"), d.get("mixer"), where + ".mixer", d.get("mlp")
        if kind not in ("attention", "mamba1", "parallel"):
            raise ConfigError(f"config.json: '{where}.type' must be 'attention', 'mamba1' or 'parallel', found {kind!r}")
        if not isinstance(mixer, dict):
            raise ConfigError(f"config.json: required key '{w}' is missing")
        if mlp is not None and (not isinstance(mlp, dict) or mlp.get("kind") != "dense"):
            raise ConfigError(f"config.json: '{where}.mlp.kind' must be 'dense' (or mlp null), found {mlp!r}")
        ff = None if mlp is None else _get(mlp, "ff", where + ".mlp", least=1)
        return cls(kind, ShapedHeads.from_dict(mixer, w, False) if kind == "attention" else None,
                   SelectiveLayer.from_dict(mixer, w) if kind == "mamba1" else None,
                   ShapedHeads.from_dict(mixer.get("left"), w + ".left", True) if kind == "parallel" else None,
                   MemorySide.from_dict(mixer.get("right"), w + ".right") if kind == "parallel" else None, ff)

    def to_dict(self):
        if self.type == "parallel":
            mixer = {"left": self.left.to_dict(), "right": self.right.to_dict()}
        else:
            mixer = (self.attention or self.selective).to_dict()
        return {"mixer": mixer, "mlp": None if self.ff is None else {"ff": self.ff, "kind": "dense"}, "type": self.type}


@dataclass(frozen=True)
class PuzonexConfig(ModelConfig):
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[PuzonexLayer, ...]
    architecture: str = "Puzonex"

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "PuzonexConfig":
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        if not isinstance(d.get("norm"), dict):
            raise ConfigError("config.json: 'norm' must be an object")
        return cls(vocab=_get(d, "vocab", "config", least=1), width=_get(d, "width", "config", least=1),
                   norm_eps=_get(d["norm"], "eps", "norm", float),
                   layers=tuple(PuzonexLayer.from_dict(x, i) for i, x in enumerate(layers)),
                   architecture=str(d.get("architecture", "Puzonex")))

    def completed(self, shapes: Mapping[str, Tuple[int, ...]]) -> "PuzonexConfig":
        """The rows of the tables of biases, from the shapes of a file's tensors (name -> shape)."""
        layers = list(self.layers)
        for i, layer in enumerate(layers):
            left = layer.left
            if left is None or left.bias_rows is not None:
                continue
            shape = shapes.get(f"l{i}.mix.left.rel")
            if shape is None or len(shape) != 2 or shape[0] < 2:
                raise ConfigError(f"layers[{i}]: the file has no table 'l{i}.mix.left.rel' of two rows or more")
            left = replace(left, bias_rows=int(shape[0]))
            left.check_bias(f"layers[{i}].mixer.left")
            layers[i] = replace(layer, left=left)
        return replace(self, layers=tuple(layers))

    def to_dict(self) -> Dict[str, Any]:
        return copy.deepcopy({"architecture": self.architecture, "layers": [x.to_dict() for x in self.layers],
                              "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width})
