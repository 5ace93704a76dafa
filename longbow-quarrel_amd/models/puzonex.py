"""The Puzonex decoder as a `ModelSpec`.

Every layer puts a norm on what its sublayers return and none on what they read, x += N1(mixer(x)); x += N2(ffn(x)),
RMS norms with plain weights.  Three kinds of mixer.  "attention": softmax attention under a sliding window; q, k and v
with biases, q and k normed per head with a weight that the heads share, values divided by their root mean square,
scores capped, a bias that falls with the logarithm of the distance, a learned sink a head.  "mamba1": the selective
scan.  "parallel": two mixers side by side, each result RMS-normed over the width with a weight of its own, half their
sum: windowed attention whose values are its keys (norms over all heads together, a temperature a head, capped scores,
a bias from a table asked by distance, a sigmoid gate an entry, biases on q, k and the output) and a matrix memory with
exponential gates.  The feed-forward is a gated unit with the tanh form of gelu; a layer may have none.  The embedding
adds sinusoids of the position; the head is a matrix of its own.

Tensor names: `embed`, `head`, `final.norm`, and for layer i `l<i>.norm1`, `l<i>.norm2`, `l<i>.mix.*` (a parallel
layer's under `.left` and `.right`, its output weights `l<i>.mix.left.out` and `.right.out`), `l<i>.mlp.*`.
"""
from __future__ import annotations

from ..config.base import ConfigError
from ..config.puzonex import PuzonexConfig, PuzonexLayer
from ..model import ModelSpec, Run
from ..parts.base import PartSpec
from ..registry import register_architecture

#: the base of the position sinusoids' frequencies
SINUSOID_BASE = 10000.0
#: what the matrix memory's denominator is raised by
MEMORY_EPS = 1e-6


def _mixer(cfg: PuzonexConfig, layer: PuzonexLayer, i: int) -> PartSpec:
    prefix = f"l{i}.mix"
    if layer.type == "mamba1":
        m = layer.selective
        return PartSpec("mamba1", {"width": cfg.width, "inner": m.inner, "state": m.state, "dt_rank": m.dt_rank,
                                   "conv": m.conv, "prefix": prefix})
    a = layer.attention or layer.left
    common = {"width": cfg.width, "heads": a.heads, "kv_heads": a.kv_heads, "key_dim": a.dim, "value_dim": a.vdim,
              "scale": a.scale, "softcap": a.softcap, "window": a.window, "keep_first": 0, "qkv_bias": True,
              "norm_eps": cfg.norm_eps}
    if layer.type == "attention":
        return PartSpec("sink_window_attention", {**common, "sink": "learned", "qk_norm": "head", "value_norm": True,
                                                  "log_bias": True, "prefix": prefix})
    if a.bias_rows is None:
        raise ConfigError(f"layers[{i}].mixer.left: the rows of the table of biases are in no key; a model file's tensor "
                          "shape gives them (or state 'bias_rows')")
    left = PartSpec("sink_window_attention", {
        **common, "sink": False, "qk_norm": "row", "values_from_keys": True, "temperature": True, "entry_gate": True,
        "out_bias": True, "table_bias": {"rows": a.bias_rows, "most": a.bias_max}, "prefix": prefix + ".left"})
    r = layer.right
    right = PartSpec("matrix_memory", {"width": cfg.width, "heads": r.heads, "key_dim": r.dim, "value_dim": r.vdim,
                                       "gate_cap": r.gate_cap, "eps": cfg.norm_eps, "den_eps": MEMORY_EPS,
                                       "prefix": prefix + ".right"})
    return PartSpec("side_by_side", {"width": cfg.width, "eps": cfg.norm_eps, "sides": (left, right),
                                     "out_names": (prefix + ".left.out", prefix + ".right.out")})


def puzonex_spec(cfg: PuzonexConfig) -> ModelSpec:
    def norm(name: str) -> PartSpec:
        return PartSpec("rmsnorm", {"width": cfg.width, "eps": cfg.norm_eps, "name": name})

    blocks = [PartSpec("output_norm", {
        "mixer": _mixer(cfg, layer, i), "mixer_norm": norm(f"l{i}.norm1"),
        "feed_forward": None if layer.ff is None else PartSpec("glu", {
            "width": cfg.width, "inner": layer.ff, "prefix": f"l{i}.mlp", "activation": "gelu_tanh"}),
        "ffn_norm": norm(f"l{i}.norm2")}) for i, layer in enumerate(cfg.layers)]
    return ModelSpec(
        vocab_size=cfg.vocab, width=cfg.width,
        embedding=PartSpec("token_table", {"name": "embed", "vocab_size": cfg.vocab, "width": cfg.width,
                                           "sinusoids": SINUSOID_BASE}),
        layers=tuple(blocks), schedule=tuple(Run(i) for i in range(len(blocks))), final_norm=norm("final.norm"),
        head_name="head", tie_head=False,
        max_positions=None,  # nothing in the design depends on a longest sequence
    )


register_architecture("Puzonex", PuzonexConfig, puzonex_spec)
