"""The Tukedra decoder as a `ModelSpec`.

The residual is several streams (hyper-connections): a sublayer reads a learned weighted sum of them, RMS-normed with a
plain weight, and its result is added to every stream with a weight of the stream's own, beside a learned mix of the
old streams.  Three kinds of mixer.  "lightning": linear attention with a fixed decay a head; silu on q, k and v, one
weighted RMS norm over all heads together, a sigmoid gate.  "retention": linear attention with a fixed decay a head;
half-split rotary pairs on q and k, k scaled by dim^(-1/2), every head divided by its root mean square, a silu gate.
"attention": softmax attention within chunks of positions, whose values are the keys as projected; biases on q and k,
interleaved rotary pairs under YaRN scaling, q and k divided by their root mean square after the rotation.  The
feed-forward is a gated silu unit, or a mixture of experts of two matrices around the square of relu, chosen by the
router's logits and weighted by their softmax over the chosen ones, beside a shared expert; a layer may have none.  The
embedding is scaled; the head is a matrix of its own, and the logits are scaled and capped.

Tensor names: `embed`, `head`, `final.norm`, and for layer i `l<i>.norm1`, `l<i>.norm2`, `l<i>.hc1.*`, `l<i>.hc2.*`
(`in`, `mix`, `out`), `l<i>.mix.*`, `l<i>.mlp.*`.
"""
from __future__ import annotations

from ..config.tukedra import TukedraConfig, TukedraLayer
from ..model import ModelSpec, Run, token_table
from ..parts.base import PartSpec
from ..registry import register_architecture


def _rotary(rot, pairing: str):
    if rot is None:
        return None
    sc = rot.scaling
    scaling = None if sc is None else {"rope_type": "yarn", "factor": sc.factor, "original": sc.original, "fast": sc.fast,
                                       "slow": sc.slow}
    return {"dims": rot.dims, "base": rot.base, "scaling": scaling, "pairing": pairing}


def _mixer(cfg: TukedraConfig, layer: TukedraLayer, i: int) -> PartSpec:
    prefix = f"l{i}.mix"
    if layer.type == "attention":
        a = layer.attention
        return PartSpec("sink_window_attention", {
            "width": cfg.width, "heads": a.heads, "kv_heads": a.kv_heads, "key_dim": a.dim, "value_dim": a.dim,
            "scale": a.scale, "chunk": a.chunk, "sink": False, "qkv_bias": True, "values_from_keys": True,
            "rotary": _rotary(a.rot, "interleaved"), "qk_norm": "unit", "norm_eps": cfg.norm_eps, "prefix": prefix})
    m = layer.linear
    sizes = {"width": cfg.width, "heads": m.heads, "key_dim": m.dim, "value_dim": m.vdim, "decay": m.decay,
             "eps": cfg.norm_eps, "prefix": prefix}
    if layer.type == "lightning":
        return PartSpec("decayed_linear_attention", {**sizes, "activation": "silu", "norm": "row", "gate": "sigmoid"})
    return PartSpec("decayed_linear_attention", {**sizes, "rotary": _rotary(m.rot, "half"), "key_scale": m.dim ** -0.5,
                                                 "norm": "head", "gate": "silu"})


def _feed_forward(cfg: TukedraConfig, layer: TukedraLayer, i: int):
    m, prefix = layer.mlp, f"l{i}.mlp"
    if m is None:
        return None
    if m.kind == "dense":
        return PartSpec("swiglu", {"width": cfg.width, "inner": m.ff, "prefix": prefix,
                                   "names": {"gate": "gate", "up": "up", "down": "down"}})
    return PartSpec("moe", {"width": cfg.width, "experts": m.experts, "top": m.top, "inner": m.ff, "prefix": prefix,
                            "weight_input": False, "scoring": "softmax_chosen", "activation": "relu2",
                            "shared_inner": m.shared_ff})


def tukedra_spec(cfg: TukedraConfig) -> ModelSpec:
    def norm(name: str) -> PartSpec:
        return PartSpec("rmsnorm", {"width": cfg.width, "eps": cfg.norm_eps, "name": name})

    blocks = [PartSpec("hyper_connected", {
        "streams": cfg.streams, "mixer": _mixer(cfg, layer, i), "mixer_norm": norm(f"l{i}.norm1"),
        "mixer_links": f"l{i}.hc1", "feed_forward": _feed_forward(cfg, layer, i), "ffn_norm": norm(f"l{i}.norm2"),
        "ffn_links": f"l{i}.hc2"}) for i, layer in enumerate(cfg.layers)]
    step = None
    if cfg.logit_softcap:
        step = PartSpec("softcap", {"cap": cfg.logit_softcap, "factor": cfg.logit_scale})
    elif cfg.logit_scale != 1.0:
        step = PartSpec("scale", {"factor": cfg.logit_scale})
    return ModelSpec(
        vocab_size=cfg.vocab, width=cfg.width, embedding=token_table("embed", cfg.vocab, cfg.width, cfg.embedding_scale),
        layers=tuple(blocks), schedule=tuple(Run(i) for i in range(len(blocks))), final_norm=norm("final.norm"),
        head_name="head", tie_head=False, logits_step=step,
        max_positions=None,  # nothing in the design depends on a longest sequence
    )


register_architecture("Tukedra", TukedraConfig, tukedra_spec)
