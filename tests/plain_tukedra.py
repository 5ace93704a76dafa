"""The Tukedra design, plain and slow: float64, whole sequences, no cache, one function per mechanism, written from
the design's equations and sharing nothing with the library.  `rounding=True` rounds activations to bfloat16 where a
bfloat16 run of the library does (what a matrix product reads, what the cache holds), so that such a run can be held
against it.

The residual is `streams` copies of the stream, all equal to the scaled embedding at the start.  A sublayer reads one
weighted sum of them, normed, and its result goes back to all of them beside a mix of the old copies; the model's
output is their sum.  Mixers: linear attention with a fixed decay a head, in two forms ("lightning": silu on q, k
and v, one norm over all heads; "retention": rotated q and k, a norm a head), and softmax attention within chunks of
positions whose values are its keys ("attention").
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


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return 1 / (1 + torch.exp(-z))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * sigmoid(z)


def relu_squared(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0) ** 2


# ---- positions -----------------------------------------------------------------------------------------------------
def frequencies(dims: int, base: float) -> List[float]:
    return [base ** (-2.0 * i / dims) for i in range(dims // 2)]


def yarn_frequencies(dims: int, base: float, sc: dict) -> List[float]:
    def place(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo, hi = max(math.floor(place(sc["fast"])), 0), min(math.ceil(place(sc["slow"])), dims - 1)
    out = []
    for i, f in enumerate(frequencies(dims, base)):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / sc["factor"] * ramp + f * (1 - ramp))
    return out


def yarn_magnitude(factor: float) -> float:
    return 0.1 * math.log(factor) + 1.0


def rotate(x: torch.Tensor, freqs: List[float], magnitude: float, interleaved: bool) -> torch.Tensor:
    """x [T, heads, d]: the first 2 len(freqs) entries of every head turned by the row's position."""
    out, n = x.clone(), len(freqs)
    for p in range(x.shape[0]):
        for i, f in enumerate(freqs):
            a, b = (2 * i, 2 * i + 1) if interleaved else (i, i + n)
            c, s = math.cos(p * f) * magnitude, math.sin(p * f) * magnitude
            u, v = x[p, :, a], x[p, :, b]
            out[p, :, a], out[p, :, b] = u * c - v * s, v * c + u * s
    return out


# ---- mixers --------------------------------------------------------------------------------------------------------
def decayed_memory(q, k, v, decay: float) -> torch.Tensor:
    """One head: q, k [T, d], v [T, e]; S <- decay S + k v^T, o = S^T q."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=F)
    o = torch.zeros(v.shape, dtype=F)
    for t in range(q.shape[0]):
        S = decay * S + torch.outer(k[t], v[t])
        o[t] = S.T @ q[t]
    return o


def heads_of(h, w, name: str, heads: int) -> torch.Tensor:
    return (h @ w[name].T).view(h.shape[0], heads, -1)


def lightning(h, m: dict, w, p: str, eps: float, rounding: bool) -> torch.Tensor:
    T, H = h.shape[0], m["heads"]
    q, k, v = (silu(heads_of(h, w, f"{p}.{n}", H)) for n in ("q", "k", "v"))
    o = torch.stack([decayed_memory(q[:, n], k[:, n], v[:, n], m["decay"][n]) for n in range(H)], dim=1)
    o = rms(o.reshape(T, -1), eps) * w[p + ".norm"] * sigmoid(h @ w[p + ".g"].T)
    return rnd(o, rounding) @ w[p + ".o"].T


def retention(h, m: dict, w, p: str, eps: float, rounding: bool) -> torch.Tensor:
    T, H, d = h.shape[0], m["heads"], m["dim"]
    freqs = frequencies(m["rot"]["dims"], m["rot"]["base"])
    q = rotate(heads_of(h, w, p + ".q", H), freqs, 1.0, False)
    k = rotate(heads_of(h, w, p + ".k", H), freqs, 1.0, False) * d ** -0.5
    v = heads_of(h, w, p + ".v", H)
    o = torch.stack([decayed_memory(q[:, n], k[:, n], v[:, n], m["decay"][n]) for n in range(H)], dim=1)
    o = rms(o, eps).reshape(T, -1) * silu(h @ w[p + ".g"].T)
    return rnd(o, rounding) @ w[p + ".o"].T


def chunk_mask(T: int, size: Optional[int]) -> torch.Tensor:
    """[T, T] true where row i sees column j: j <= i, and both in one run of `size` positions counted from 0."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & ((i // size == j // size) if size else torch.ones(T, T, dtype=torch.bool))


def softmax_rows(score: torch.Tensor, seen: torch.Tensor) -> torch.Tensor:
    score = score.masked_fill(~seen, -math.inf)
    e = torch.exp(score - score.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def attention(h, m: dict, w, p: str, eps: float, rounding: bool) -> torch.Tensor:
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = (h @ w[p + ".q"].T + w[p + ".q.b"]).view(T, H, -1)
    k = (h @ w[p + ".k"].T + w[p + ".k.b"]).view(T, G, -1)
    v = rnd(k, rounding)  # the keys as projected
    rot = m["rot"]
    sc = rot.get("scaling")
    freqs = yarn_frequencies(rot["dims"], rot["base"], sc) if sc else frequencies(rot["dims"], rot["base"])
    magnitude = yarn_magnitude(sc["factor"]) if sc else 1.0
    q = rnd(rms(rotate(q, freqs, magnitude, True), eps), rounding)
    k = rnd(rms(rotate(k, freqs, magnitude, True), eps), rounding)
    seen = chunk_mask(T, m["mask"]["size"] if m.get("mask") else None)
    out = torch.zeros(T, H, k.shape[2], dtype=F)
    for n in range(H):
        g = n // (H // G)
        out[:, n] = softmax_rows((q[:, n] @ k[:, g].T) * m["scale"], seen) @ v[:, g]
    return rnd(out.reshape(T, -1), rounding) @ w[p + ".o"].T


MIXERS = {"lightning": lightning, "retention": retention, "attention": attention}


# ---- feed-forwards -------------------------------------------------------------------------------------------------
def dense(h, w, p: str, rounding: bool) -> torch.Tensor:
    return rnd(silu(h @ w[p + ".gate"].T) * (h @ w[p + ".up"].T), rounding) @ w[p + ".down"].T


def expert(h, w, p: str, weight, rounding: bool) -> torch.Tensor:
    """`weight`: a number a row, on the expert's activations (its second matrix is linear)."""
    return rnd(relu_squared(h @ w[p + ".up"].T) * weight, rounding) @ w[p + ".down"].T


def route(z: torch.Tensor, top: int) -> torch.Tensor:
    """[T, E] logits -> [T, E]: the softmax over a row's `top` largest, zero elsewhere (the lower index on a tie)."""
    out = torch.zeros_like(z)
    for t in range(z.shape[0]):
        chosen = sorted(range(z.shape[1]), key=lambda e: (-float(z[t, e]), e))[:top]
        out[t, chosen] = torch.softmax(z[t, chosen], 0)
    return out


def mixture(h, m: dict, w, p: str, rounding: bool) -> torch.Tensor:
    weights = route(h @ w[p + ".router"].T, m["router"]["top"])
    y = expert(h, w, p + ".shared", 1.0, rounding) if m.get("shared") else torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        y = y + expert(h, w, f"{p}.e{e}", weights[:, e : e + 1], rounding)
    return y


# ---- the model -----------------------------------------------------------------------------------------------------
def read_streams(X: torch.Tensor, w_in: torch.Tensor) -> torch.Tensor:
    """X [s, T, width] -> the weighted sum [T, width]."""
    return sum(w_in[s] * X[s] for s in range(X.shape[0]))


def write_streams(X: torch.Tensor, y: torch.Tensor, mix: torch.Tensor, w_out: torch.Tensor) -> torch.Tensor:
    """Every new stream from all old ones (mix [from, to]) and the sublayer's result."""
    S = X.shape[0]
    return torch.stack([sum(mix[s, t] * X[s] for s in range(S)) + w_out[t] * y for t in range(S)])


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], rounding: bool = False,
            layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence; `layers_out` takes the sum of the streams after every layer."""
    w = {k: v.to(F) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens)] * (cfg.get("embedding") or {}).get("scale", 1.0)
    X = torch.stack([x] * cfg["streams"])

    def sublayer(X, p, q, fn):
        h = rnd(rms(read_streams(X, w[f"{p}.hc{q}.in"]), eps) * w[f"{p}.norm{q}"], rounding)
        return write_streams(X, fn(h), w[f"{p}.hc{q}.mix"], w[f"{p}.hc{q}.out"])

    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}", layer.get("mlp")
        X = sublayer(X, p, 1, lambda h: MIXERS[layer["type"]](h, layer["mixer"], w, p + ".mix", eps, rounding))
        if m is not None:
            X = sublayer(X, p, 2, lambda h: dense(h, w, p + ".mlp", rounding) if m["kind"] == "dense"
                         else mixture(h, m, w, p + ".mlp", rounding))
        if layers_out is not None:
            layers_out.append(X.sum(0))
    logits = rnd(rms(X.sum(0), eps) * w["final.norm"], rounding) @ w["head"].T * cfg.get("logit_scale", 1.0)
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(logits / cap) if cap else logits
