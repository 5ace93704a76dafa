"""Linear attention with a fixed decay a head, and no softmax or denominator.

q and k are `heads` x `key_dim`, v is `heads` x `value_dim`, projections of the input without biases.  Per head h, with
the state S [key_dim, value_dim] starting at zero and the constant decay_h:

    S <- decay_h S + k v^T,      o = S^T q.

`activation` "silu": q, k and v pass silu first.  `rotary` (`dims`, `base`, optionally `scaling`, and `pairing` "half" or
"interleaved", as `sink_window_attention` takes it) turns the first `dims` entries of every head of q and k by the
position.  k is multiplied by `key_scale`, after both.  The heads' results side by side are RMS-normed: `norm` "row" over
all heads together, times a weight (`<prefix>.norm`, all heads' entries), or "head", every head by itself, without a
weight.  Then they are multiplied by `gate` ("sigmoid" or "silu") of one more projection of the input, and projected.

`activation="silu"`, `norm="row"`, `gate="sigmoid"` is lightning attention (Qin, Sun, Li, Shen, Sun, Zhong: "Lightning
Attention-2: A Free Lunch for Handling Unlimited Sequence Lengths in Large Language Models"); `rotary`, `norm="head"`,
`gate="silu"` is retention (Sun, Dong, Huang, Ma, Xia, Xue, Wang, Wei: "Retentive Network: A Successor to Transformer for
Large Language Models").

How it runs.  One product of the input gives [q | k | v | gate] in 32-bit; `decay_scan` takes activation, rotation and
scale on its way and leaves the results in 32-bit: a step of few tokens a sequence is walked token by token with the
state in registers, a longer one in chunks of 64 tokens whose states are chained (given scratch), the matrix products of
a chunk in 32-bit on the matrix cores.  `gated_rmsnorm` norms and gates."""
from __future__ import annotations

from typing import Dict, List, Mapping, Optional, Sequence

import torch

from .base import (MIXERS, VECTOR32, BuildEnv, Mixer, StateNeed, StepContext, TensorSpec, product_weight, project,
                   project_delta)
from .rope import rotary_frequencies, rotary_magnitude, step_angles


def decay_powers(decay: Sequence[float], most: int) -> torch.Tensor:
    """[heads, most + 1] float32: every decay to the powers 0 .. most, taken in float64."""
    d = torch.tensor([float(v) for v in decay], dtype=torch.float64)
    return torch.stack([d ** n for n in range(most + 1)], dim=1).float()


@MIXERS.register("decayed_linear_attention")
class DecayedLinearAttention(Mixer):
    graph_safe = True
    takes_out = True
    CHUNK = 64  # tokens a chunk of `decay_scan`: it is given the decays' powers so far

    def __init__(self, width: int, heads: int, key_dim: int, value_dim: int, decay: Sequence[float], eps: float, prefix: str,
                 norm: str, gate: str, activation: Optional[str] = None, rotary: Optional[Mapping] = None,
                 key_scale: float = 1.0, names: Optional[Mapping[str, str]] = None) -> None:
        self.width, self.heads, self.key_dim, self.value_dim = int(width), int(heads), int(key_dim), int(value_dim)
        self.eps, self.key_scale, self.norm, self.gate, self.activation = float(eps), float(key_scale), norm, gate, activation
        self.decay = tuple(float(v) for v in decay)
        if len(self.decay) != self.heads:
            raise ValueError(f"{heads} heads need as many decays, found {len(self.decay)}")
        if norm not in ("row", "head") or gate not in ("silu", "sigmoid") or activation not in (None, "silu"):
            raise ValueError(f"the norm is 'row' or 'head' ({norm!r}), the gate 'silu' or 'sigmoid' ({gate!r}), the "
                             f"activation 'silu' or None ({activation!r})")
        self.rot_dims, self.rot_interleaved, self.rot_magnitude, self.freq_table = 0, False, 1.0, []
        if rotary is not None:
            self.rot_dims = int(rotary["dims"])
            pairing = rotary.get("pairing", "half")
            if pairing not in ("half", "interleaved"):
                raise ValueError(f"rotary pairing {pairing!r} is not known (known: 'half', 'interleaved')")
            if self.rot_dims % 2 or not 2 <= self.rot_dims <= self.key_dim:
                raise ValueError(f"{self.rot_dims} rotated entries do not fit a head of {key_dim}")
            scaling = dict(rotary["scaling"]) if rotary.get("scaling") else None
            self.rot_interleaved = pairing == "interleaved"
            self.freq_table: List[float] = rotary_frequencies(self.rot_dims, float(rotary["base"]), scaling)
            self.rot_magnitude = rotary_magnitude(scaling)
        self.qk_width, self.v_width = self.heads * self.key_dim, self.heads * self.value_dim
        n = {"q": "q", "k": "k", "v": "v", "gate": "g", "norm": "norm", "o": "o"}
        n.update(names or {})
        self.names: Dict[str, str] = {key: f"{prefix}.{val}" for key, val in n.items()}

    def tensor_specs(self) -> List[TensorSpec]:
        nm = self.names
        return [
            TensorSpec(nm["q"], (self.qk_width, self.width)),
            TensorSpec(nm["k"], (self.qk_width, self.width)),
            TensorSpec(nm["v"], (self.v_width, self.width)),
            TensorSpec(nm["gate"], (self.v_width, self.width)),
            TensorSpec(nm["o"], (self.width, self.v_width)),
            *([TensorSpec(nm["norm"], (self.v_width,), kind=VECTOR32, init="around_one")] if self.norm == "row" else []),
        ]

    def bind(self, tensors: Mapping[str, torch.Tensor], env: BuildEnv) -> None:
        super().bind(tensors, env)
        nm = self.names
        mats = [tensors[nm[k]] for k in ("q", "k", "v", "gate")]
        if len({m.dtype for m in mats}) != 1:
            raise ValueError(f"{nm['q']}: the projections of one input are stored in different dtypes")
        self.w_in = product_weight(env, torch.cat(mats, dim=0))
        self.w_o = product_weight(env, tensors[nm["o"]])
        self.norm_w = tensors[nm["norm"]].contiguous() if self.norm == "row" else None
        self.powers = decay_powers(self.decay, self.CHUNK).to(env.device)
        self.freqs = torch.tensor(self.freq_table, dtype=torch.float64, device=env.device) if self.rot_dims else None

    def cache_need(self) -> StateNeed:
        # held [head, value_dim, key_dim]: a column of the head's values has its key entries side by side
        return StateNeed((self.heads, self.value_dim, self.key_dim), torch.float32)

    def forward(self, h: torch.Tensor, ctx: StepContext, cache, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        kn = ctx.kernels
        if cache is None or getattr(cache, "state", None) is None:
            raise RuntimeError("linear attention needs its state")
        if not cache.write:
            raise RuntimeError("a recurrent state cannot be shared between runs of the schedule")
        rows, qk, vw = h.shape[0], self.qk_width, self.v_width
        total = 2 * qk + 2 * vw
        u = ctx.ws.alloc((rows, (total + 3) // 4 * 4), torch.float32)[:, :total]
        project(kn, ctx, h, self.w_in, u)
        o = ctx.ws.alloc((rows, vw), torch.float32)
        more = {}
        if self.rot_dims:
            more = dict(cos_sin=step_angles(ctx, self.freqs, self.freq_table), interleaved=self.rot_interleaved,
                        magnitude=self.rot_magnitude)
        ask = getattr(kn, "decay_scan_workspace", None)
        need = ask(rows, ctx.batch, self.heads, self.key_dim, self.value_dim, ctx.max_new) if ask is not None else 0
        if need:
            more.update(max_rows=ctx.max_new, workspace=ctx.ws.alloc((need,), torch.float32))
        kn.decay_scan(u[:, :qk], u[:, qk : 2 * qk], u[:, 2 * qk : 2 * qk + vw], self.powers, cache.state, o, self.heads,
                      self.key_dim, self.value_dim, self.key_scale, ctx.seq_slot, ctx.cu_rows, ctx.batch,
                      activation=self.activation, **more)
        normed = ctx.ws.alloc((rows, vw), ctx.dtype)
        kn.gated_rmsnorm(o, u[:, 2 * qk + vw :], self.norm_w, self.eps, vw if self.norm == "row" else self.value_dim, normed,
                         gate_first=False, gate=self.gate)
        if out is None:
            return project_delta(kn, ctx, normed, self.w_o)
        project(kn, ctx, normed, self.w_o, out)
        return out
