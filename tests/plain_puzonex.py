"""The Puzonex design, plain and slow: float64, whole sequences, no cache, one function per mechanism, written from
the design's equations and sharing nothing with the library.  `rounding=True` rounds activations to bfloat16 where a
bfloat16 run of the library does (what a matrix product reads, what the cache holds), so that such a run can be held
against it.

A layer:  x += N1(mixer(x));  x += N2(ffn(x)),  N(y) = y / sqrt(mean y^2 + eps) w: the sublayers read the stream.
An "attention" layer's mixer is windowed attention with normed values, a soft cap, a logarithmic distance bias and a
learned sink; a "mamba1" layer's the selective scan; a "parallel" layer's the half sum of windowed attention whose
values are its keys, with a bias from a table asked by distance and a gate, and a matrix memory with exponential gates.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F = torch.float64


def rnd(t: torch.Tensor, rounding: bool) -> torch.Tensor:
    return t.to(torch.bfloat16).to(F) if rounding else t


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1 + torch.exp(-z))


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def log_sigmoid(z: torch.Tensor) -> torch.Tensor:
    return -softplus(-z)


def soft_cap(s: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    return s if not cap else cap * torch.tanh(s / cap)


def sinusoids(T: int, width: int) -> torch.Tensor:
    """[T, width]: neighbouring entries 2i, 2i + 1 are sine and cosine of position * 10000^(-2i / width)."""
    out = torch.zeros(T, width, dtype=F)
    for p in range(T):
        for c in range(width):
            a = p * 10000.0 ** (-(c - c % 2) / width)
            out[p, c] = math.cos(a) if c % 2 else math.sin(a)
    return out


def distances(T: int) -> torch.Tensor:
    return torch.arange(T)[:, None] - torch.arange(T)[None, :]


def window_mask(T: int, size: Optional[int]) -> torch.Tensor:
    """[T, T] true where row i sees column j: 0 <= i - j < size (no size: every j <= i)."""
    n = distances(T)
    return (n >= 0) & (n < (T if size is None else size))


def window_of(m: dict) -> Optional[int]:
    return m["mask"]["size"] if m.get("mask") else None


def log_bias(T: int, r1: float, r2: float) -> torch.Tensor:
    """[T, T]: what a score gets for the distance n between its tokens, -r1 ln(1 + r2 n)."""
    return -r1 * torch.log(1.0 + r2 * distances(T).clamp(min=0).to(F))


def bucket(n: int, rows: int, most: float) -> int:
    """The table's row for a distance: one a distance below rows / 2, then ever wider ones up to `most`."""
    half = rows // 2
    if n < half:
        return n
    steps = math.log(n / half) / math.log(most / half) * (rows - half)
    return min(rows - 1, half + math.floor(steps + 1e-9))


def table_bias(T: int, column: torch.Tensor, most: float) -> torch.Tensor:
    """[T, T] from one head's column [rows] of the table."""
    by_distance = torch.stack([column[bucket(n, column.shape[0], most)] for n in range(T)])
    return by_distance[distances(T).clamp(min=0)]


def softmax_rows(score: torch.Tensor, seen: torch.Tensor, sink: Optional[float] = None) -> torch.Tensor:
    """Softmax over the seen columns of every row; with a sink the denominator has one more term exp(sink)."""
    score = score.masked_fill(~seen, -math.inf)
    top = score.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.clamp(top, min=sink)
    e = torch.exp(score - top)
    total = e.sum(-1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(sink - top)
    return e / total


def attention(h, m: dict, w: Dict[str, torch.Tensor], p: str, eps: float, rounding: bool) -> torch.Tensor:
    T, H, G, d, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + ".q"].T + w[p + ".q.b"]).view(T, H, d)
    k = (h @ w[p + ".k"].T + w[p + ".k.b"]).view(T, G, d)
    v = (h @ w[p + ".v"].T + w[p + ".v.b"]).view(T, G, vd)
    q = rnd(rms(q, eps) * w[p + ".q.norm"], rounding)
    k = rnd(rms(k, eps) * w[p + ".k.norm"], rounding)
    v = rnd(rms(v, eps), rounding)
    seen = window_mask(T, window_of(m))
    out = torch.zeros(T, H, vd, dtype=F)
    for n in range(H):
        g = n // (H // G)
        score = soft_cap((q[:, n] @ k[:, g].T) * m["scale"], m.get("softcap"))
        score = score + log_bias(T, float(w[p + ".r1"][n]), float(w[p + ".r2"][n]))
        out[:, n] = softmax_rows(score, seen, float(w[p + ".sink"][n])) @ v[:, g]
    return rnd(out.reshape(T, H * vd), rounding) @ w[p + ".o"].T


def key_value_attention(h, m: dict, w: Dict[str, torch.Tensor], p: str, eps: float, rounding: bool) -> torch.Tensor:
    """The values are the keys as projected; q and k normed over all heads' entries together."""
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = h @ w[p + ".q"].T + w[p + ".q.b"]
    k = h @ w[p + ".k"].T + w[p + ".k.b"]
    v = rnd(k, rounding).view(T, G, d)
    q = rnd(rms(q, eps) * w[p + ".q.norm"], rounding).view(T, H, d)
    k = rnd(rms(k, eps) * w[p + ".k.norm"], rounding).view(T, G, d)
    seen = window_mask(T, window_of(m))
    out = torch.zeros(T, H, d, dtype=F)
    for n in range(H):
        g = n // (H // G)
        score = (q[:, n] @ k[:, g].T) * m["scale"] * w[p + ".temp"][n]
        score = soft_cap(score, m.get("softcap")) + table_bias(T, w[p + ".rel"][:, n], m["bias_max"])
        out[:, n] = softmax_rows(score, seen) @ v[:, g]
    gate = torch.sigmoid(h @ w[p + ".g"].T)
    return rnd(out.reshape(T, H * d) * gate, rounding) @ w[p + ".o"].T + w[p + ".o.b"]


def short_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """x [T, C], taps [C, n]: y_t = silu(bias + sum_j taps[:, j] x_{t - (n - 1) + j}), zeros before the start."""
    T, C = x.shape
    n = taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, C, dtype=F), x], 0)
    y = torch.zeros(T, C, dtype=F) + bias
    for j in range(n):
        y = y + padded[j : j + T] * taps[:, j]
    return silu(y)


def selective_scan(x, dt, B, C, A, D) -> torch.Tensor:
    """x, dt [T, c]; B, C [T, n]; A [c, n]; D [c]."""
    S = torch.zeros(A.shape, dtype=F)
    y = torch.zeros(x.shape, dtype=F)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba(h, m: dict, w: Dict[str, torch.Tensor], p: str, eps: float, rounding: bool) -> torch.Tensor:
    c, n, r = m["inner"], m["state"], m["dt_rank"]
    xz = h @ w[p + ".in"].T
    x, z = xz[:, :c], xz[:, c:]
    x = rnd(short_conv(x, w[p + ".conv"], w[p + ".conv.b"]), rounding)
    low = x @ w[p + ".x"].T
    dt = softplus(rnd(low[:, :r], rounding) @ w[p + ".dt"].T + w[p + ".dt.b"])
    y = selective_scan(x, dt, low[:, r : r + n], low[:, r + n :], -torch.exp(w[p + ".A_log"]), w[p + ".D"])
    return rnd(y * silu(z), rounding) @ w[p + ".o"].T


def matrix_memory(q, k, v, i, f) -> torch.Tensor:
    """One head: q, k [T, d], v [T, e], i and f [T] (logarithms of the gates)."""
    S, n, m = torch.zeros(q.shape[1], v.shape[1], dtype=F), torch.zeros(q.shape[1], dtype=F), 0.0
    o = torch.zeros(v.shape, dtype=F)
    for t in range(q.shape[0]):
        top = max(float(f[t]) + m, float(i[t]))
        keep, take = math.exp(float(f[t]) + m - top), math.exp(float(i[t]) - top)
        m = top
        S = keep * S + take * torch.outer(k[t], v[t])
        n = keep * n + take * k[t]
        o[t] = (S.T @ q[t]) / (max(abs(float(n @ q[t])), math.exp(-m)) + 1e-6)
    return o


def mlstm(h, m: dict, w: Dict[str, torch.Tensor], p: str, eps: float, rounding: bool) -> torch.Tensor:
    T, H, d, vd, cap = h.shape[0], m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q = (h @ w[p + ".q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[p + ".k"].T).view(T, H, d)
    v = (h @ w[p + ".v"].T).view(T, H, vd)
    i = soft_cap(h @ w[p + ".i"].T + w[p + ".i.b"], cap)
    f = log_sigmoid(soft_cap(h @ w[p + ".f"].T + w[p + ".f.b"], cap))
    o = torch.stack([matrix_memory(q[:, n], k[:, n], v[:, n], i[:, n], f[:, n]) for n in range(H)], dim=1)
    o = rms(o, eps).reshape(T, H * vd) * w[p + ".norm"] * torch.sigmoid(h @ w[p + ".g"].T)
    return rnd(o, rounding) @ w[p + ".o"].T


def side_by_side(h, m: dict, w, p: str, eps: float, rounding: bool) -> torch.Tensor:
    left = key_value_attention(h, m["left"], w, p + ".left", eps, rounding)
    right = mlstm(h, m["right"], w, p + ".right", eps, rounding)
    return 0.5 * (rms(left, eps) * w[p + ".left.out"] + rms(right, eps) * w[p + ".right.out"])


MIXERS = {"attention": attention, "mamba1": mamba, "parallel": side_by_side}


def dense(h, w, p: str, rounding: bool) -> torch.Tensor:
    return rnd(gelu_tanh(h @ w[p + ".gate"].T) * (h @ w[p + ".up"].T), rounding) @ w[p + ".down"].T


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], rounding: bool = False,
            layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence; `layers_out` takes the stream after every layer."""
    w = {k: v.to(F) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens)] + sinusoids(len(tokens), cfg["width"])
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}"
        x = x + rms(MIXERS[layer["type"]](rnd(x, rounding), layer["mixer"], w, p + ".mix", eps, rounding), eps) * w[p + ".norm1"]
        if layer.get("mlp") is not None:
            x = x + rms(dense(rnd(x, rounding), w, p + ".mlp", rounding), eps) * w[p + ".norm2"]
        if layers_out is not None:
            layers_out.append(x.clone())
    return rnd(rms(x, eps) * w["final.norm"], rounding) @ w["head"].T
