"""Configurations, weights and the engine-beside-plain case for the Puzonex tests, shared by the CPU tests (the
engine's own code over the torch stand-in for the kernels) and the GPU tests (the same over the HIP kernels).
Every comparison is against `plain_puzonex`, run over whole sequences in float64.  The scenarios (cuttings,
batches, reuse of slots, long decoding, greedy tokens) are those of `vafodra_cases`, which ask nothing of a case
but its engine, its vocabulary and the plain logits."""
from __future__ import annotations

import copy
from typing import Dict, List, Optional

import torch

import longbow_quarrel_amd as lq
import plain_puzonex as pp
from vafodra_cases import (err, greedy, long_decoding, portions, slots_and_blocks_used_again, tokens,  # noqa: F401
                           unequal_batches, whole_and_token_by_token, write_folder)
from vupelorn_cases import assert_close_bf16  # noqa: F401
from longbow_quarrel_amd.engine import StepEntry


def _heads(heads, kv_heads, dim, vdim, scale, window=None, softcap=None, bias_max=None, bias_rows=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if softcap is not None:
        m["softcap"] = softcap
    if window is not None:
        m["mask"] = {"size": window}
    if bias_max is not None:
        m.update(bias_max=bias_max, bias_rows=bias_rows)
    return m


def _mlp(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def _attention(mixer, ff):
    return {"type": "attention", "mixer": mixer, "mlp": _mlp(ff)}


def _mamba(inner, state, dt_rank, conv, ff):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}, "mlp": _mlp(ff)}


def _parallel(left, heads, dim, vdim, cap, ff):
    right = {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": _mlp(ff)}


def _config(vocab, width, eps, layers):
    return {"architecture": "Puzonex", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}


# A: every kind of layer in another order than usual, one of each twice; windows inside a cache block, across blocks
# and none; keys wider and narrower than values; three query heads a kv head and one; caps that bind and none; states
# and ranks that differ; a layer without feed-forward; tables that end near and far; an eps that counts (a sublayer's
# result that happens to be near zero at one token is not blown up to unit size together with its rounding)
CFG_A = _config(173, 80, 1e-2, [
    _parallel(_heads(6, 2, 24, 24, 0.3, 20, 4.0, 60.0, 12), 3, 12, 20, 6.0, 56),
    _attention(_heads(2, 2, 16, 40, 0.6, 70, 3.0), 24),
    _mamba(56, 12, 6, 4, None),
    _attention(_heads(6, 2, 40, 16, 0.2), 72),
    _mamba(40, 20, 3, 3, 16),
    _parallel(_heads(4, 4, 16, 16, 0.5, None, None, 20.0, 8), 2, 24, 8, 15.0, None),
])
# B: sizes that are multiples of nothing (the kernels' size-agnostic ways), an odd width, one head, a window of one
# token, a state, a rank and taps of one, one memory head of one key entry
CFG_B = _config(97, 51, 1e-5, [
    _mamba(29, 1, 1, 1, 21),
    _attention(_heads(1, 1, 10, 7, 0.4, 1, 2.0), 9),
    _parallel(_heads(5, 5, 6, 6, 0.5, 5, 30.0, 3.0, 2), 1, 1, 7, 2.0, 33),
    _parallel(_heads(3, 1, 14, 14, 0.25, 64, 5.0, 7.5, 5), 5, 7, 3, 9.0, None),
    _mamba(13, 33, 7, 5, None),
])
# C: head sizes, ranks and widths of the kind that the fast kernels are made for
CFG_C = _config(1000, 320, 1e-5, [
    _mamba(640, 16, 24, 4, 384),
    _parallel(_heads(4, 2, 64, 64, 0.12, 100, 10.0, 90.0, 16), 4, 32, 64, 15.0, 192),
    _attention(_heads(8, 2, 32, 64, 0.18, 65, 20.0), 256),
    _attention(_heads(2, 1, 128, 128, 0.09, 200, 8.0), None),
    _parallel(_heads(8, 8, 32, 32, 0.18, 63, 25.0, 40.0, 32), 2, 128, 32, 5.0, 64),
])
# one mechanism a model: what fails here names its mechanism
CFG_LOG = _config(60, 48, 1e-6, [_attention(_heads(4, 2, 16, 8, 0.5, 40, 5.0), None)])
CFG_TABLE = _config(60, 48, 1e-6, [_parallel(_heads(4, 2, 16, 16, 0.3, 40, 4.0, 30.0, 10), 1, 4, 4, 5.0, None)])
CFG_MEMORY = _config(60, 48, 1e-3, [_parallel(_heads(1, 1, 8, 8, 0.3, 3, None, 9.0, 4), 4, 12, 20, 4.0, None)])
CFG_SCAN = _config(60, 48, 1e-6, [_mamba(72, 10, 5, 3, None)])
CFG_DENSE = _config(60, 48, 1e-6, [_mamba(8, 2, 1, 2, 40)])
CONFIGS = {"a": CFG_A, "b": CFG_B, "c": CFG_C, "log": CFG_LOG, "table": CFG_TABLE, "memory": CFG_MEMORY,
           "scan": CFG_SCAN, "dense": CFG_DENSE}


def attention_of(cfg: dict) -> dict:
    """The softmax attention of a one-layer configuration."""
    mixer = cfg["layers"][0]["mixer"]
    return mixer.get("left", mixer)


def windowed(kind: str, window: int) -> dict:
    """One attention layer of the kind ("log" or "table") with the window given."""
    cfg = copy.deepcopy(CONFIGS[kind])
    attention_of(cfg)["mask"] = {"size": window}
    return cfg


def long_memory(name: str) -> dict:
    """One recurrent layer; the cap on the memory's gates high enough that its forget gate can come near one."""
    cfg = copy.deepcopy(CONFIGS[name])
    if name == "memory":
        cfg["layers"][0]["mixer"]["right"]["gate_cap"] = 14.0
    return cfg


def random_config(seed: int) -> dict:
    """A configuration drawn from a seed: the layers' kinds and order, sizes, head counts, windows, caps, tables, states,
    ranks, taps and constants all vary; some sizes are multiples of 16, some of nothing."""
    import random

    rng = random.Random(seed)
    width = rng.choice([40, 51, 64, 72, 100, 128, 136])

    def heads(tied):
        kv = rng.randint(1, 3)
        dim = rng.choice([8, 12, 16, 20, 32, 48, 64])
        rows = rng.choice([2, 3, 8, 16, 31])
        return _heads(kv * rng.randint(1, 4), kv, dim, dim if tied else rng.choice([8, 16, 28, 64]),
                      rng.choice([0.1, 0.2, 0.35]), rng.choice([None, 1, 2, 7, 33, 64, 65, 100]),
                      rng.choice([None, 2.0, 6.0, 30.0]), rows // 2 + rng.choice([0.5, 3.0, 50.0, 400.0]) if tied else None,
                      rows)

    layers = []
    for _ in range(rng.randint(1, 5)):
        kind, ff = rng.choice(["attention", "mamba1", "parallel"]), rng.choice([None, 16, 24, 50, 96])
        if kind == "attention":
            layers.append(_attention(heads(False), ff))
        elif kind == "mamba1":
            layers.append(_mamba(rng.choice([16, 24, 50, 96, 130]), rng.choice([1, 4, 8, 9, 16, 40]), rng.randint(1, 12),
                                 rng.randint(1, 5), ff))
        else:
            layers.append(_parallel(heads(True), rng.randint(1, 4), rng.choice([4, 8, 12, 16, 40]),
                                    rng.choice([4, 8, 15, 16, 36]), rng.choice([2.0, 8.0, 15.0]), ff))
    return _config(rng.randint(30, 300), width, rng.choice([1e-6, 1e-5]), layers)


def make_weights(cfg: dict, seed: int, sharp: float = 1.0, memory: float = 0.0) -> Dict[str, torch.Tensor]:
    """Random weights whose values bfloat16 holds exactly (both run dtypes then see the same model), with spreads
    that make every constant matter.  `sharp` multiplies the attention's score scales and caps in `cfg` (in place) so
    that attention is peaked.  `memory` is added to the forget gates' biases and taken off the step sizes', so that the
    recurrent states forget slowly and old tokens stay in them."""
    from longbow_quarrel_amd.model import DecoderModel
    from longbow_quarrel_amd.registry import spec_from_config

    if sharp != 1.0:
        for layer in cfg["layers"]:
            m = layer["mixer"]
            for a in ([m] if layer["type"] == "attention" else [m["left"]] if layer["type"] == "parallel" else []):
                a["scale"] *= sharp
                if a.get("softcap"):
                    a["softcap"] *= sharp
    config = lq.PuzonexConfig.from_dict(cfg)
    g = torch.Generator().manual_seed(seed)
    out = {}
    for s in DecoderModel(spec_from_config(config)).tensor_specs():
        n, shape = s.name, tuple(s.shape)
        leaf = n.split(".")[-1]
        normal = lambda std, mean=0.0: torch.empty(shape).normal_(mean, std, generator=g)
        uniform = lambda lo, hi: torch.empty(shape).uniform_(lo, hi, generator=g)
        if n == "embed":
            t = normal(1.0)
        elif leaf in ("norm", "norm1", "norm2", "out", "D"):
            t = normal(0.3, 1.0)
        elif leaf in ("temp", "r1"):
            t = uniform(0.3, 1.5)
        elif leaf == "r2":
            t = uniform(0.05, 2.0)
        elif leaf in ("sink", "rel"):
            t = normal(1.0)
        elif leaf == "conv":
            t = normal(0.6)
        elif leaf == "A_log":
            t = normal(0.7, 0.0)
        elif n.endswith(".dt.b"):
            t = normal(1.0, -1.0 - memory)
        elif n.endswith(".f.b"):
            t = normal(1.0, 1.0 + memory)
        elif n.endswith(".i.b"):  # (low enough that the bound on a memory's denominator binds at many tokens)
            t = normal(0.5, -1.0)
        elif leaf == "b":
            t = normal(0.5)
        elif leaf in ("i", "f"):  # (several tokens share a memory: one alone would leave its answer to a single product)
            t = normal(0.7 / (shape[-1] ** 0.5))
        else:
            t = normal(1.0 / (shape[-1] ** 0.5))
        out[n] = t.to(torch.bfloat16).float()
    return out


class Case:
    """An engine (made by `load`, which the CPU and the GPU tests bring) beside the plain implementation."""

    def __init__(self, tmp_path, name, load, dtype: str = "float32", seed: int = 3, sharp: float = 1.0,
                 memory: float = 0.0, max_tokens: int = 2048, rounding: bool = False,
                 cfg: Optional[dict] = None) -> None:
        self.cfg = copy.deepcopy(cfg if cfg is not None else CONFIGS[name] if isinstance(name, str)
                                 else random_config(name))
        self.weights = make_weights(self.cfg, seed, sharp, memory)
        self.folder = write_folder(tmp_path, self.cfg, self.weights, f"{name}_{seed}_{sharp}_{memory}")
        self.eng = load(self.folder, dtype, max_tokens)
        self.vocab = self.cfg["vocab"]
        self.rounding = rounding
        self._want = {}

    def want(self, toks: List[int]) -> torch.Tensor:
        key = tuple(toks)
        if key not in self._want:
            self._want[key] = pp.forward(self.cfg, self.weights, toks, rounding=self.rounding)
        return self._want[key]

    def noise(self, toks: List[int]) -> float:
        """What rounding alone does on these tokens: the median over the rows of the largest difference (over the
        largest logit) between the plain implementation with and without rounding."""
        a = pp.forward(self.cfg, self.weights, toks, rounding=True)
        b = pp.forward(self.cfg, self.weights, toks, rounding=False)
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
        pp.forward(self.cfg, self.weights, toks, rounding=self.rounding, layers_out=want)
        return got, want

    def assert_idle(self) -> None:
        c = self.eng.cache
        assert c.slots.taken_count == 0 and all(g.blocks.taken_count == 0 for g in c.kv_groups)


def a_window_off_by_one_would_show(case: Case, toks: List[int], rows) -> None:
    """The plain implementation with the window a token wider and a token narrower differs from the true one at
    `rows` by much more than any tolerance here: were the engine's window off by one, the comparison would fail."""
    for other in (+1, -1):
        cfg = copy.deepcopy(case.cfg)
        mask = attention_of(cfg)["mask"]
        if mask["size"] + other < 1:
            continue
        mask["size"] += other
        wrong = pp.forward(cfg, case.weights, toks)
        assert err(wrong[rows], case.want(toks)[rows]) > 1e-3, f"a window off by {other} does not show"


def flattened(weights: Dict[str, torch.Tensor], **leaves) -> Dict[str, torch.Tensor]:
    """The weights with every tensor of the given last names set to one value: a mechanism taken out of the oracle, to
    show that it matters."""
    return {n: torch.full_like(t, leaves[n.split(".")[-1]]) if n.split(".")[-1] in leaves else t for n, t in weights.items()}
