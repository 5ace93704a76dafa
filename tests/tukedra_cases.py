"""Configurations, weights and the engine-beside-plain case for the Tukedra tests, shared by the CPU tests (the
engine's own code over the torch stand-in for the kernels) and the GPU tests (the same over the HIP kernels).
Every comparison is against `plain_tukedra`, run over whole sequences in float64.  The scenarios (cuttings,
batches, reuse of slots, long decoding, greedy tokens) are those of `vafodra_cases`, which ask nothing of a case
but its engine, its vocabulary and the plain logits."""
from __future__ import annotations

import copy
import random
from typing import Dict, List, Optional

import torch

import longbow_quarrel_amd as lq
import plain_tukedra as pt
from vafodra_cases import (err, greedy, long_decoding, portions, slots_and_blocks_used_again, tokens,  # noqa: F401
                           unequal_batches, whole_and_token_by_token, write_folder)
from vupelorn_cases import assert_close_bf16  # noqa: F401
from longbow_quarrel_amd.engine import StepEntry


def _lightning(heads, dim, vdim, decay, mlp):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": mlp}


def _retention(heads, dim, vdim, decay, rot, mlp):
    base, dims = rot
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay,
                                           "rot": {"base": base, "dims": dims}}, "mlp": mlp}


def _yarn(base, dims, factor=5.0, original=64, fast=8.0, slow=1.0):
    return {"base": base, "dims": dims, "scaling": {"factor": factor, "original": original, "fast": fast, "slow": slow}}


def _attention(heads, kv_heads, dim, scale, rot, mlp, chunk=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale, "rot": rot}
    if chunk is not None:
        m["mask"] = {"size": chunk}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, experts, top, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        m["shared"] = {"ff": shared}
    return m


def _config(vocab, width, eps, streams, layers, scale=1.0, logit_scale=1.0, softcap=None):
    cfg = {"architecture": "Tukedra", "embedding": {"scale": scale}, "layers": layers, "logit_scale": logit_scale,
           "norm": {"eps": eps}, "streams": streams, "vocab": vocab, "width": width}
    if softcap is not None:
        cfg["logit_softcap"] = softcap
    return cfg


# A: every kind of layer and of feed-forward, some twice; values wider and narrower than keys; a rotation of a part of a
# head and of all of it; chunks inside a cache block, across blocks and none; a layer without feed-forward
CFG_A = _config(173, 80, 1e-5, 3, [
    _retention(3, 24, 40, [0.75, 0.97, 0.9995], (500.0, 16), _dense(56)),
    _attention(6, 2, 24, 0.2, _yarn(1000.0, 12), _moe(24, 5, 2, 40), 20),
    _lightning(4, 20, 12, [0.5, 0.9, 0.99, 1.0], None),
    _attention(3, 3, 40, 0.15, _yarn(300.0, 40, 2.0, 40, 4.0, 0.5), _moe(16, 7, 3), 70),
    _lightning(2, 32, 48, [0.3, 0.998], _moe(40, 3, 3, 8)),
    _attention(2, 1, 16, 0.4, _yarn(50.0, 4), _dense(24)),
], scale=0.7, logit_scale=0.4, softcap=5.0)
# B: sizes that are multiples of nothing (the kernels' size-agnostic ways), an odd width, one head, one stream, one expert
# of two, a chunk of one token, a value size of one
CFG_B = _config(97, 51, 1e-6, 1, [
    _lightning(1, 7, 9, [0.8], _moe(13, 2, 1, 5)),
    _retention(5, 6, 7, [0.1, 0.6, 0.95, 0.99, 0.999], (20.0, 2), _dense(21)),
    _attention(5, 1, 10, 0.5, _yarn(80.0, 6), None, 1),
    _attention(1, 1, 14, 0.3, _yarn(9.0, 14, 8.0, 30, 3.0, 0.7), _moe(9, 4, 4, 33), 5),
    _lightning(3, 1, 5, [0.9, 0.4, 0.97], _dense(10)),
], logit_scale=2.0)
# C: head sizes and widths of the kind that the fast kernels are made for
CFG_C = _config(1000, 256, 1e-5, 4, [
    _lightning(4, 64, 64, [0.9, 0.97, 0.99, 0.999], _dense(384)),
    _retention(2, 128, 128, [0.98, 0.999], (10000.0, 128), _moe(128, 8, 2, 128)),
    _attention(8, 2, 64, 0.14, _yarn(10000.0, 40, 3.0, 256, 16.0, 1.0), _moe(64, 6, 3, 96), 100),
    _lightning(2, 128, 32, [0.95, 0.9999], _moe(96, 4, 1, 64)),
    _attention(2, 1, 128, 0.1, _yarn(10000.0, 128), _dense(128), 192),
], scale=0.6, logit_scale=0.7, softcap=20.0)
# one mechanism a model: what fails here names its mechanism
CFG_LIGHTNING = _config(60, 48, 1e-6, 1, [_lightning(3, 16, 24, [0.6, 0.95, 0.9995], None)])
CFG_RETENTION = _config(60, 48, 1e-6, 1, [_retention(2, 20, 12, [0.8, 0.999], (100.0, 12), None)])
CFG_CHUNKED = _config(60, 48, 1e-6, 1, [_attention(4, 2, 16, 0.3, _yarn(200.0, 8), None, 40)])
CFG_EXPERTS = _config(60, 48, 1e-6, 1, [_lightning(1, 4, 4, [0.5], _moe(24, 6, 2, 16))])
CFG_DENSE = _config(60, 48, 1e-6, 1, [_lightning(1, 4, 4, [0.5], _dense(40))])
CFG_STREAMS = _config(60, 48, 1e-6, 5, [_lightning(1, 4, 4, [0.5], _dense(8)), _lightning(1, 4, 8, [0.9], None),
                                        _lightning(2, 4, 4, [0.9, 0.1], _dense(16))])
CFG_CAPPED = _config(60, 48, 1e-6, 2, [_lightning(1, 4, 4, [0.5], None)], scale=3.0, logit_scale=1.7, softcap=1.5)
CONFIGS = {"a": CFG_A, "b": CFG_B, "c": CFG_C, "lightning": CFG_LIGHTNING, "retention": CFG_RETENTION,
           "chunked": CFG_CHUNKED, "experts": CFG_EXPERTS, "dense": CFG_DENSE, "streams": CFG_STREAMS, "capped": CFG_CAPPED}
ALONE = ["lightning", "retention", "chunked", "experts", "dense", "streams", "capped"]


def chunked(size: Optional[int]) -> dict:
    """One attention layer with chunks of the size given."""
    cfg = copy.deepcopy(CFG_CHUNKED)
    cfg["layers"][0]["mixer"]["mask"] = {"size": size}
    return cfg


def slow(name: str) -> dict:
    """One layer of linear attention whose heads forget slowly."""
    cfg = copy.deepcopy(CONFIGS[name])
    m = cfg["layers"][0]["mixer"]
    m["decay"] = [0.9999, 0.999, 1.0][: m["heads"]]
    return cfg


def random_config(seed: int) -> dict:
    """A configuration drawn from a seed: the layers' kinds and order, sizes, head counts, decays, chunks, rotations, streams,
    experts and constants all vary; some sizes are multiples of 16, some of nothing."""
    rng = random.Random(seed)
    width = rng.choice([40, 51, 64, 72, 100, 128, 136])
    decays = lambda n: [rng.choice([0.2, 0.7, 0.9, 0.97, 0.99, 0.999, 1.0]) for _ in range(n)]

    def mlp():
        kind = rng.choice(["none", "dense", "moe", "moe"])
        if kind == "none":
            return None
        if kind == "dense":
            return _dense(rng.choice([16, 24, 50, 96]))
        experts = rng.randint(1, 9)
        return _moe(rng.choice([8, 13, 16, 40]), experts, rng.randint(1, min(4, experts)), rng.choice([None, 8, 15, 40]))

    layers = []
    for _ in range(rng.randint(1, 5)):
        kind, heads = rng.choice(["attention", "lightning", "retention"]), rng.randint(1, 5)
        dim = rng.choice([8, 12, 16, 20, 32, 48, 64, 130])
        dims = 2 * rng.randint(1, dim // 2)
        if kind == "attention":
            rot = _yarn(rng.choice([10.0, 300.0, 10000.0]), dims, rng.choice([1.0, 2.0, 16.0]), rng.choice([16, 50, 400]),
                        rng.choice([4.0, 32.0]), rng.choice([0.5, 1.0]))
            layers.append(_attention(heads * rng.randint(1, 4), heads, dim, rng.choice([0.1, 0.2, 0.35]), rot, mlp(),
                                     rng.choice([None, 1, 2, 7, 33, 64, 65, 100])))
        elif kind == "retention":
            # (a head of few values divided by its root mean square blows up the rounding of answers near zero)
            layers.append(_retention(heads, dim, rng.choice([8, 11, 15, 32, 70]), decays(heads),
                                     (rng.choice([10.0, 300.0, 10000.0]), dims), mlp()))
        else:
            layers.append(_lightning(heads, dim, rng.choice([1, 8, 15, 32, 70]), decays(heads), mlp()))
    return _config(rng.randint(30, 300), width, rng.choice([1e-6, 1e-5]), rng.randint(1, 6), layers,
                   scale=rng.choice([1.0, 0.3, 2.0]), logit_scale=rng.choice([1.0, 0.5, 3.0]),
                   softcap=rng.choice([None, 2.0, 30.0]))


def make_weights(cfg: dict, seed: int, sharp: float = 1.0) -> Dict[str, torch.Tensor]:
    """Random weights whose values bfloat16 holds exactly (both run dtypes then see the same model), with spreads that
    make every constant matter.  `sharp` multiplies the attention's score scales in `cfg` (in place) so that attention is
    peaked."""
    from longbow_quarrel_amd.model import DecoderModel
    from longbow_quarrel_amd.registry import spec_from_config

    for layer in cfg["layers"]:
        if layer["type"] == "attention":
            layer["mixer"]["scale"] *= sharp
    config = lq.TukedraConfig.from_dict(cfg)
    g = torch.Generator().manual_seed(seed)
    out = {}
    for s in DecoderModel(spec_from_config(config)).tensor_specs():
        if s.optional:
            continue
        n, shape = s.name, tuple(s.shape)
        leaf = n.split(".")[-1]
        normal = lambda std, mean=0.0: torch.empty(shape).normal_(mean, std, generator=g)
        if n == "embed":
            t = normal(1.0)
        elif leaf in ("norm", "norm1", "norm2"):
            t = normal(0.3, 1.0)
        elif leaf in ("in", "out"):
            t = normal(0.4, 0.7)
        elif leaf == "mix":
            t = torch.eye(shape[0]) * 0.7 + normal(0.25)
        elif leaf == "b":
            t = normal(0.7)
        elif leaf == "router":
            t = normal(1.5 / shape[-1] ** 0.5)
        elif leaf == "down" and ".mlp." in n:
            t = normal(1.5 / shape[-1] ** 0.5)
        else:
            t = normal(1.0 / shape[-1] ** 0.5)
        out[n] = t.to(torch.bfloat16).float()
    return out


class Case:
    """An engine (made by `load`, which the CPU and the GPU tests bring) beside the plain implementation."""

    def __init__(self, tmp_path, name, load, dtype: str = "float32", seed: int = 3, sharp: float = 1.0,
                 max_tokens: int = 2048, rounding: bool = False, cfg: Optional[dict] = None) -> None:
        self.cfg = copy.deepcopy(cfg if cfg is not None else CONFIGS[name] if isinstance(name, str)
                                 else random_config(name))
        self.weights = make_weights(self.cfg, seed, sharp)
        self.folder = write_folder(tmp_path, self.cfg, self.weights, f"{name}_{seed}_{sharp}")
        self.eng = load(self.folder, dtype, max_tokens)
        self.vocab = self.cfg["vocab"]
        self.rounding = rounding
        self._want = {}

    def want(self, toks: List[int]) -> torch.Tensor:
        key = tuple(toks)
        if key not in self._want:
            self._want[key] = pt.forward(self.cfg, self.weights, toks, rounding=self.rounding)
        return self._want[key]

    def noise(self, toks: List[int]) -> float:
        """What rounding alone does on these tokens: the median over the rows of the largest difference (over the
        largest logit) between the plain implementation with and without rounding."""
        a = pt.forward(self.cfg, self.weights, toks, rounding=True)
        b = pt.forward(self.cfg, self.weights, toks, rounding=False)
        return float(((a - b).abs().max(-1).values / b.abs().max()).median())

    def run_cut(self, toks: List[int], cuts: List[int]) -> torch.Tensor:
        """The sequence in portions of the sizes `cuts` (the rest token by token), all logits."""
        eng = self.eng
        s = eng.new_sequence()
        got, at = [], 0
        sizes = list(cuts)
        while at < len(toks):
            n = min(sizes.pop(0) if sizes else 1, len(toks) - at)
            got.append(eng.step([StepEntry(s, toks[at : at + n], range(n))]).clone())
            at += n
        eng.release(s)
        return torch.cat(got)

    def layers(self, toks: List[int]):
        """The residual stream after every layer, from the engine's observer and from the plain implementation."""
        got = []

        def see(name, x, pending):
            if name != "embed":
                full = x.float().cpu().clone()
                if pending is not None:
                    full += pending.float().cpu().sum(0) if pending.dim() == 3 else pending.float().cpu()
                got.append(full)

        s = self.eng.new_sequence()
        self.eng.step([StepEntry(s, toks, [])], observe=see)
        self.eng.release(s)
        want = []
        pt.forward(self.cfg, self.weights, toks, rounding=self.rounding, layers_out=want)
        return got, want

    def assert_idle(self) -> None:
        c = self.eng.cache
        assert c.slots.taken_count == 0 and all(g.blocks.taken_count == 0 for g in c.kv_groups)


def a_chunk_off_by_one_would_show(case: Case, toks: List[int]) -> None:
    """The plain implementation with chunks a token longer and a token shorter differs from the true one by much more than
    any tolerance here: were the engine's chunk off by one, the comparison would fail."""
    for other in (+1, -1):
        cfg = copy.deepcopy(case.cfg)
        mask = cfg["layers"][0]["mixer"]["mask"]
        if mask["size"] + other < 1:
            continue
        mask["size"] += other
        wrong = pt.forward(cfg, case.weights, toks)
        first = mask["size"] if other < 0 else mask["size"] - 1  # from here on the chunks differ
        assert err(wrong[first:], case.want(toks)[first:]) > 1e-3, f"chunks off by {other} do not show"
        assert err(wrong[:first], case.want(toks)[:first]) < 1e-12


def flattened(weights: Dict[str, torch.Tensor], **leaves) -> Dict[str, torch.Tensor]:
    """The weights with every tensor of the given last names set to one value: a mechanism taken out of the oracle, to
    show that it matters."""
    return {n: torch.full_like(t, leaves[n.split(".")[-1]]) if n.split(".")[-1] in leaves else t for n, t in weights.items()}
