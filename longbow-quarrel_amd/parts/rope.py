"""Rotary position encoding with half-split pairs (i, i + hd/2).

f_i = base^(-2 i / hd), angle = position * f_i
(internal/device/kernels.metal:430-463, host twin internal/device/cpu_ref.go:103-129).
The optional scaling of the frequencies has no counterpart in the reference.
`linear` divides every f_i by the factor.  `llama3`: with wavelength
L_i = 2 pi / f_i, L_i < original / high_freq_factor keeps f_i,
L_i > original / low_freq_factor gives f_i / factor, and between the two
s = (original / L_i - low) / (high - low), f_i' = (1 - s) f_i / factor + s f_i.

`yarn` (Peng, Quesnelle, Fan, Shippole: "YaRN: Efficient Context Window Extension of Large Language Models")
blends per pair: with d(t) = dims ln(original / (2 pi t)) / (2 ln base) the pair index at which a wave turns t
times within `original` positions, lo = max(floor(d(fast)), 0), hi = min(ceil(d(slow)), dims - 1) and
r_i = clamp((i - lo) / max(hi - lo, 0.001), 0, 1): f_i' = r_i f_i / factor + (1 - r_i) f_i; cos and sin are
also multiplied by 0.1 ln(factor) + 1 (`rotary_magnitude`).

The table is computed once in float64 and handed to the kernel as a parameter,
so the kernel knows nothing about scaling types.
"""
from __future__ import annotations

import math
from typing import List, Mapping, Optional

import torch

from .base import POSITION_ENCODINGS, BuildEnv, PositionEncoding, StepContext


def rotary_frequencies(head_dim: int, base: float, scaling: Optional[Mapping] = None) -> List[float]:
    freqs = [base ** (-2.0 * i / head_dim) for i in range(head_dim // 2)]
    if not scaling:
        return freqs
    factor = float(scaling["factor"])
    kind = scaling.get("rope_type", "llama3")
    if kind == "linear":  # positions divided by the factor
        return [f / factor for f in freqs]
    if kind == "yarn":
        original = float(scaling["original"])

        def pair_of(turns: float) -> float:
            return head_dim * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

        lo = max(math.floor(pair_of(float(scaling["fast"]))), 0)
        hi = min(math.ceil(pair_of(float(scaling["slow"]))), head_dim - 1)
        ramps = [min(1.0, max(0.0, (i - lo) / max(hi - lo, 0.001))) for i in range(head_dim // 2)]
        return [f / factor * r + f * (1.0 - r) for f, r in zip(freqs, ramps)]
    if kind != "llama3":
        raise ValueError(f"rope scaling type {kind!r} is not known (known: 'linear', 'llama3', 'yarn')")
    low = float(scaling["low_freq_factor"])
    high = float(scaling["high_freq_factor"])
    original = float(scaling["original_max_position_embeddings"])
    out = []
    for f in freqs:
        wavelen = 2.0 * math.pi / f
        if wavelen < original / high:
            out.append(f)
        elif wavelen > original / low:
            out.append(f / factor)
        else:
            s = (original / wavelen - low) / (high - low)
            out.append((1.0 - s) * f / factor + s * f)
    return out


def rotary_magnitude(scaling: Optional[Mapping] = None) -> float:
    """What cos and sin are multiplied by: 0.1 ln(factor) + 1 under `yarn` scaling, else 1."""
    if scaling and scaling.get("rope_type", "llama3") == "yarn":
        return 0.1 * math.log(float(scaling["factor"])) + 1.0
    return 1.0


def step_angles(ctx: StepContext, freqs: torch.Tensor, table: List[float]) -> torch.Tensor:
    """cos and sin of every row's angles, float32 [rows, pairs, 2]: the same for every layer of a step that rotates with
    these frequencies (`freqs` on the device, `table` the same numbers on the host), so computed once and shared."""
    key = ("rope_cos_sin", tuple(table))
    angles = ctx.shared.get(key)
    if angles is None:
        angles = ctx.ws.alloc((ctx.rows, len(table), 2), torch.float32, keep=True)
        ctx.kernels.rope_table(freqs, ctx.row_pos, angles)
        ctx.shared[key] = angles
    return angles


@POSITION_ENCODINGS.register("rope")
class RotaryEncoding(PositionEncoding):
    graph_safe = True

    def __init__(self, head_dim: int, base: float, scaling: Optional[Mapping] = None) -> None:
        self.head_dim = int(head_dim)
        self.base = float(base)
        self.scaling = dict(scaling) if scaling else None
        self.table = rotary_frequencies(self.head_dim, self.base, self.scaling)

    def bind(self, tensors: Mapping[str, torch.Tensor], env: BuildEnv) -> None:
        super().bind(tensors, env)
        self.rotary_frequencies = torch.tensor(self.table, dtype=torch.float64, device=env.device)

    def cos_sin(self, ctx: StepContext) -> torch.Tensor:
        return step_angles(ctx, self.rotary_frequencies, self.table)

    def apply(self, q: torch.Tensor, k: torch.Tensor, ctx: StepContext) -> None:
        heads = q.shape[1] // self.head_dim
        kv_heads = k.shape[1] // self.head_dim
        ctx.kernels.rope_store(q, None, None, heads, 0, self.head_dim, self.rotary_frequencies, ctx.row_pos)
        ctx.kernels.rope_store(k, None, None, kv_heads, 0, self.head_dim, self.rotary_frequencies, ctx.row_pos)


@POSITION_ENCODINGS.register("none")
class NoPositionEncoding(PositionEncoding):
    graph_safe = True

    """Leaves q and k as they are (the mixer sees order through the causal mask only)."""

    def __init__(self, **_unused) -> None:
        pass

    def apply(self, q: torch.Tensor, k: torch.Tensor, ctx: StepContext) -> None:
        return None
