"""The Puzonex design on the GPU.  First every kernel that the design brought, or widened, alone against the plain
implementation's function of the same mechanism (float64), with inputs made so that a fault shows; then the engine
in float32 and in bfloat16 under every cutting and batching; then generation through the entry point, with captured
steps and direct ones, the command line and the trace replay."""
import copy
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import longbow_quarrel_amd as lq
import plain_puzonex as pp
import puzonex_cases as pc
from longbow_quarrel_amd.engine import StepEntry

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEV = "cuda:0"
# (single rows of these models are ill-conditioned: see the CPU tests' limit)
TOL_F32 = 1e-4
F = torch.float64


@pytest.fixture(scope="module")
def kn():
    from longbow_quarrel_amd.kernels.hip import HipKernels
    return HipKernels()


def rnd(*shape, seed=0, std=1.0, mean=0.0):
    return torch.empty(shape).normal_(mean, std, generator=torch.Generator().manual_seed(seed))


def i32(values):
    return torch.tensor(list(values), dtype=torch.int32, device=DEV)


def dev(t, dtype=torch.float32):
    return t.to(dtype).to(DEV).contiguous()


def load(folder, dtype, max_tokens):
    return lq.load_engine(folder, dtype=dtype, max_tokens=max_tokens, device=DEV, max_slots=8,
                          max_sequence_tokens=max_tokens)


class Paged:
    """A sequence's keys and values in a paged cache whose blocks lie in no particular order."""

    def __init__(self, length, kv_heads, key_dim, value_dim, dtype, bs=64, seed=0):
        n = (length + bs - 1) // bs
        order = torch.randperm(n + 3, generator=torch.Generator().manual_seed(seed)).tolist()
        self.order, self.bs = order, bs
        self.table = torch.tensor([order[:n]], dtype=torch.int32, device=DEV)
        self.k = torch.zeros((n + 3, kv_heads, bs, key_dim), dtype=dtype, device=DEV)
        self.v = torch.zeros((n + 3, kv_heads, value_dim, bs), dtype=dtype, device=DEV)

    def read(self, length):
        """-> keys [length, kv heads, key size], values [length, kv heads, value size]"""
        at = [(self.order[t // self.bs], t % self.bs) for t in range(length)]
        return (torch.stack([self.k[b, :, o, :] for b, o in at]).cpu(), torch.stack([self.v[b, :, :, o] for b, o in at]).cpu())


def two_sequences(seq_rows=((5, 40), (1, 23))):
    """Rows of two sequences in slots out of order, as two steps: -> per step (rows a sequence, slots, cu_rows)."""
    return [dict(slots=i32([2, 0]), cu=i32([0, a, a + b]), rows=(a, b)) for a, b in zip(*seq_rows)]


# ---- the kernels alone -------------------------------------------------------------------------------------------
def plain_shaped(q, k, v, scale, window, temp=None, cap=0.0, r1=None, r2=None, table=None, sinks=None, gate=None):
    """q [T, H, D], k [T, G, D], v [T, G, P]; table [H, n], its last column for all that is farther."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    seen = pp.window_mask(T, window)
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for n in range(H):
        g = n // (H // G)
        s = (q[:, n] @ k[:, g].T) * scale
        if temp is not None:
            s = s * temp[n].double()
        s = pp.soft_cap(s, cap)
        if r1 is not None:
            s = s + pp.log_bias(T, float(r1[n]), float(r2[n]))
        if table is not None:
            s = s + table[n].double()[pp.distances(T).clamp(0, table.shape[1] - 1)]
        out[:, n] = pp.softmax_rows(s, seen, None if sinks is None else float(sinks[n])) @ v[:, g]
    out = out.reshape(T, -1)
    return out if gate is None else out * torch.sigmoid(gate.double())


SHAPES = [
    # query heads, key heads, key size, value size, window, temp, cap, log bias, table entries, sink, gate, generic kernel
    (4, 2, 32, 16, 7, True, 3.0, False, 7, False, True, False), (8, 2, 16, 48, 70, False, 5.0, True, 0, True, False, False),
    (6, 2, 48, 48, 64, True, 0.0, False, 30, False, True, False), (3, 1, 16, 16, 65, False, 0.0, True, 0, True, False, False),
    (8, 1, 64, 64, 0, False, 20.0, True, 0, True, False, False), (4, 4, 64, 64, 0, True, 20.0, False, 90, False, True, False),
    (2, 2, 24, 40, 9, True, 2.0, True, 5, True, True, False), (5, 5, 10, 7, 63, False, 4.0, False, 40, False, True, False),
    (8, 2, 16, 48, 70, False, 5.0, True, 0, True, False, True), (4, 2, 32, 16, 7, True, 3.0, False, 7, False, True, True),
    (16, 1, 32, 32, 130, True, 6.0, True, 100, True, True, False), (1, 1, 128, 128, 1, False, 8.0, True, 0, True, False, False),
]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", SHAPES)
def test_scores_shaped_on_their_way_to_the_softmax(kn, sizes, dtype):
    """Temperature, cap, logarithmic bias, bias by distance, sink and a gate an entry, alone and together; rows of a prompt
    and the same rows as single tokens.  Every eighth row's query is aimed at one key (its score stands out): the key
    just inside the window, just outside it, a key at a cache block's edge, in turn."""
    H, G, D, P, window, temp, cap, log, entries, sink, gate, generic = sizes
    T = 200
    q, k, v = rnd(T, H, D, seed=1), rnd(T, G, D, seed=2), rnd(T, G, P, seed=3)
    w = window if window else T
    for n, i in enumerate(range(70, T, 8)):
        j = [i - w + 1, i - w, (i // 64) * 64, (i // 64) * 64 - 1][n % 4]
        if 0 <= j <= i:
            for h in range(H):
                q[i, h] = k[j, h // (H // G)] * 8.0 / k[j, h // (H // G)].norm()
    q, k, v = (t.to(dtype).double() for t in (q, k, v))  # what the kernel is given, exactly
    scale = 1.3 / math.sqrt(D)
    more, plain = {}, {}
    if temp:
        plain["temp"] = more["temp"] = torch.empty(H).uniform_(0.5, 2.0, generator=torch.Generator().manual_seed(4))
    if cap:
        plain["cap"] = more["softcap"] = cap
    if log:
        plain["r1"], plain["r2"] = rnd(H, seed=5).abs() + 0.2, rnd(H, seed=6).abs() + 0.05
        more["log_bias"] = (dev(plain["r1"]), dev(plain["r2"]))
    if entries:
        plain["table"] = rnd(H, entries, seed=7, std=1.5)
        more["distance_bias"] = dev(plain["table"])
    if sink:
        plain["sinks"] = rnd(H, seed=8, std=2.0)
        more["sink_values"] = dev(plain["sinks"])
    if gate:
        plain["gate"] = rnd(T, H * P, seed=9, std=2.0)
        wide = dev(torch.cat([rnd(T, 3, seed=10), plain["gate"]], 1))[:, 3:]  # a run of columns of a wider row
    if temp:
        more["temp"] = dev(more["temp"])
    want = plain_shaped(q, k, v, scale, w, **plain)
    for name in plain:  # each of them matters (a bias one token's window cannot show aside)
        less = {**plain, name: None if name != "cap" else 0.0}
        if name == "r1":
            less["r2"] = None
        if name != "r2" and not (w == 1 and name in ("r1", "cap", "temp", "table")):
            assert pc.err(plain_shaped(q, k, v, scale, w, **less), want) > 1e-2, name
    cache = Paged(T, G, D, P, dtype, seed=5)
    pos, seq, slot = i32(range(T)), i32([0] * T), i32([0])
    kn.force_generic = generic
    try:
        kn.kv_store(dev(k.reshape(T, -1), dtype), dev(v.reshape(T, -1), dtype), G, D, P, pos, seq, slot, cache.table, cache.k,
                    cache.v, 64)
        qd = dev(q.reshape(T, -1), dtype)
        more.update(window=window, keep_first=0, sink=sink)
        for out_dtype in {dtype, torch.float32}:
            out = torch.zeros((T, H * P), dtype=out_dtype, device=DEV)
            kn.sink_attention(qd, out, H, G, D, P, pos, seq, slot, cache.table, cache.k, cache.v, 64, scale,
                              **more, **({"wide_gate": wide} if gate else {}))
            tol = 1e-5 if dtype == torch.float32 else (1e-2 if out_dtype == torch.bfloat16 else 4e-5)
            # (a bfloat16 cache with 32-bit results: exact products of what the cache holds, 32-bit sums)
            assert pc.err(out, want) < tol, out_dtype
        for r in list(range(60, 76)) + [127, 128, 129, 191, 199]:  # single tokens, over block edges too
            one = torch.zeros((1, H * P), dtype=torch.float32, device=DEV)
            kn.sink_attention(qd[r : r + 1], one, H, G, D, P, i32([r]), i32([0]), slot, cache.table, cache.k, cache.v,
                              64, scale, decode=True, **more, **({"wide_gate": wide[r : r + 1]} if gate else {}))
            assert pc.err(one[0], want[r]) < 4e-5, r
            if dtype == torch.float32 and not generic:
                assert torch.equal(one[0], out[r]), r  # the same sums in the same order
    finally:
        kn.force_generic = False


@pytest.mark.parametrize("sizes", [(4, 1, 32, 48, 0), (8, 2, 64, 64, 700)])
def test_shaped_single_tokens_whose_keys_are_shared_out_over_workgroups(kn, sizes):
    H, G, D, P, window = sizes
    T, dtype = 1500, torch.bfloat16
    q, k, v = (t.to(dtype).double() for t in (rnd(T, H, D, seed=1), rnd(T, G, D, seed=2), rnd(T, G, P, seed=3)))
    r1, r2, temp, table = rnd(H, seed=4).abs() * 0.3, rnd(H, seed=5).abs(), rnd(H, seed=6).abs() + 0.5, rnd(H, 300, seed=7)
    gate, sinks = rnd(T, H * P, seed=8), rnd(H, seed=9) + 2.0
    scale, w = 1.0 / math.sqrt(D), window if window else T
    want = plain_shaped(q, k, v, scale, w, temp, 4.0, r1, r2, table, sinks, gate)
    cache = Paged(T, G, D, P, dtype, seed=5)
    pos, seq, slot = i32(range(T)), i32([0] * T), i32([0])
    kn.kv_store(dev(k.reshape(T, -1), dtype), dev(v.reshape(T, -1), dtype), G, D, P, pos, seq, slot, cache.table, cache.k, cache.v, 64)
    qd, gd = dev(q.reshape(T, -1), dtype), dev(gate)
    more = dict(window=window, sink=True, sink_values=dev(sinks), temp=dev(temp), softcap=4.0, log_bias=(dev(r1), dev(r2)),
                distance_bias=dev(table))
    need = kn.sink_attention_workspace(dtype, 1, 1, H, G, D, P, 64, window, 0, T)
    assert need > 0
    scratch = torch.zeros(need, device=DEV)
    for r in (T - 1, 1100, 800, 767, 700):
        for out_dtype in (torch.float32, dtype):
            one = torch.zeros((1, H * P), dtype=out_dtype, device=DEV)
            kn.sink_attention(qd[r : r + 1], one, H, G, D, P, i32([r]), i32([0]), slot, cache.table, cache.k, cache.v, 64,
                              scale, decode=True, max_len=T, workspace=scratch, wide_gate=gd[r : r + 1], **more)
            assert pc.err(one[0], want[r]) < (4e-5 if out_dtype == torch.float32 else 1e-2), (r, out_dtype)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [
    # heads, kv heads, key size, value size, norm of q and k, norm of v, values are keys, biases
    (4, 2, 16, 40, "head", True, False, True), (6, 2, 24, 24, "row", False, True, True), (3, 1, 7, 7, "row", False, True, True),
    (5, 5, 10, 6, "head", True, False, False), (8, 2, 128, 128, "row", False, True, True), (8, 2, 128, 64, "head", True, False, True),
    (2, 1, 16, 16, None, False, False, True), (32, 8, 64, 64, "row", True, False, True), (1, 1, 600, 600, "head", True, False, True), (4, 1, 384, 384, "head", True, False, True),
    (40, 2, 128, 96, "row", False, False, True),
])
def test_biases_norms_and_the_store_of_q_k_and_v(kn, sizes, dtype):
    H, G, D, P, norm, norm_v, tied, biased = sizes
    T, eps = 75, 1e-2
    qw, kw, vw = H * D, G * D, 0 if tied else G * P
    src, bias = rnd(T, qw + kw + vw, seed=1), rnd(qw + kw + vw, seed=2) if biased else None
    uq, uk = (qw, kw) if norm == "row" else (D, D)
    wq, wk = (rnd(uq, seed=3, mean=1.0, std=0.3), rnd(uk, seed=4, mean=1.0, std=0.3)) if norm else (None, None)
    t = src.double() + (bias.double() if biased else 0.0)
    q, k = t[:, :qw], t[:, qw : qw + kw]
    v = k if tied else t[:, qw + kw :]
    unit = lambda x, w, n: (pp.rms(x.reshape(T, -1, n), eps) * (1.0 if w is None else w.double())).reshape(T, -1)
    if norm:
        q, k = unit(q, wq, uq), unit(k, wk, uk)
    if norm_v:
        v = unit(v, None, P)
    wide = dev(torch.cat([rnd(T, 4, seed=5), src, rnd(T, 4, seed=6)], 1))[:, 4 : 4 + qw + kw + vw]
    cache = Paged(T, G, D, P, dtype, seed=7)
    out = torch.zeros((T, qw), dtype=dtype, device=DEV)
    args = dict(bias=None if bias is None else dev(bias), q_weight=None if wq is None else dev(wq),
                k_weight=None if wk is None else dev(wk), norm_qk=norm, norm_v=norm_v, v_from_k=tied)
    tol = 3e-6 if dtype == torch.float32 else 1e-2
    # the rows in two launches, each without a cache first (q alone)
    for lo, hi in ((0, 70), (70, T)):
        place = dict(row_pos=i32(range(lo, hi)), row_seq=i32([0] * (hi - lo)), seq_slot=i32([0]), block_table=cache.table,
                     kcache=cache.k, vcache=cache.v, block_size=64)
        kn.qkv_norm_store(wide[lo:hi], out[lo:hi], H, G, D, P, eps, **args)
        assert pc.err(out[lo:hi], q[lo:hi]) < tol
        out[lo:hi] = 0
        kn.qkv_norm_store(wide[lo:hi], out[lo:hi], H, G, D, P, eps, **args, **place)
    assert pc.err(out, q) < tol
    gk, gv = cache.read(T)
    assert pc.err(gk.reshape(T, -1), k) < tol and pc.err(gv.reshape(T, -1), v) < tol


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [(40, 16), (300, 16), (50, 1), (13, 8), (64, 9), (129, 33), (24, 64), (5, 130), (3, 500)])
def test_selective_scan(kn, sizes, dtype):
    """Two sequences in unequal portions, in slots out of order; steps from nearly nothing to large and rates from slow to
    fast, so that a decay is near one and near zero in one launch."""
    C, N = sizes
    A_log, D, bias = rnd(C, N, seed=1, std=1.5), rnd(C, seed=2), rnd(C, seed=3, mean=-1.0)
    state = torch.zeros(4, C, N, device=DEV)
    lens = (45, 24)
    full = {}
    for i, n in enumerate(lens):
        x, dt, z = rnd(n, C, seed=10 + i), rnd(n, C, seed=20 + i, std=2.0), rnd(n, C, seed=30 + i)
        B, Cm = rnd(n, N, seed=40 + i), rnd(n, N, seed=50 + i)
        x, z, B, Cm = (t.to(dtype).float() for t in (x, z, B, Cm))
        y = pp.selective_scan(x.double(), pp.softplus(dt.double() + bias.double()), B.double(), Cm.double(),
                              -torch.exp(A_log.double()), D.double())
        full[i] = (x, dt, z, B, Cm, y * pp.silu(z.double()))
    at = [0, 0]
    got = {0: [], 1: []}
    for step in two_sequences():
        part = [[full[i][j][at[i] : at[i] + n] for i, n in enumerate(step["rows"])] for j in range(5)]
        x, dt, z, B, Cm = (torch.cat(p) for p in part)
        rows = x.shape[0]
        out = torch.zeros((rows, C), dtype=dtype, device=DEV)
        bc = dev(torch.cat([B, Cm], 1), dtype)  # runs of columns of one product
        kn.selective_scan(dev(x, dtype), dev(dt), bc[:, :N], bc[:, N:], dev(z, dtype), dev(bias), dev(A_log), dev(D), state, out,
                          step["slots"], step["cu"], 2)
        r = 0
        for i, n in enumerate(step["rows"]):
            got[i].append(out[r : r + n].cpu())
            at[i] += n
            r += n
    for i in (0, 1):
        assert pc.err(torch.cat(got[i]), full[i][5][: at[i]]) < (2e-5 if dtype == torch.float32 else 1e-2), i
    assert bool((state[1] == 0).all()) and bool((state[3] == 0).all())  # nobody's slots


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [(300, 16), (40, 8), (13, 5), (70, 64), (33, 20)])
def test_selective_scan_of_single_tokens(kn, sizes, dtype):
    """A step of single tokens gives the bits that the same tokens give in a longer step."""
    C, N = sizes
    A_log, D, bias = dev(rnd(C, N, seed=1)), dev(rnd(C, seed=2)), dev(rnd(C, seed=3, mean=-1.0))
    x, z, B, Cm = (dev(rnd(12, w, seed=4 + i), dtype) for i, w in enumerate((C, C, N, N)))
    dt = dev(rnd(12, C, seed=9))
    start = rnd(4, C, N, seed=10)
    whole, state = torch.zeros((12, C), dtype=dtype, device=DEV), dev(start)
    kn.selective_scan(x, dt, B, Cm, z, bias, A_log, D, state, whole, i32([3, 1]), i32([0, 6, 12]), 2)
    single = dev(start)
    for t in range(6):
        rows = [t, 6 + t]
        one = torch.zeros((2, C), dtype=dtype, device=DEV)
        kn.selective_scan(*(v[rows].contiguous() for v in (x, dt, B, Cm, z)), bias, A_log, D, single, one, i32([3, 1]),
                          i32([0, 1, 2]), 2)
        assert torch.equal(one, whole[rows]), t
    assert torch.equal(single, state)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [(96, 16), (40, 5)])
def test_selective_scan_of_long_prompts_in_segments(kn, sizes, dtype):
    """Two long sequences and a short one in one launch, given scratch: the long ones run in segments side by side, from
    states that earlier steps left, and leave the same states and results as a launch without scratch."""
    C, N = sizes
    lens = (1300, 90, 2049)
    rows = sum(lens)
    A_log, D, bias = rnd(C, N, seed=1, std=1.5, mean=-2.0), rnd(C, seed=2), rnd(C, seed=3, mean=-3.0)
    x, z = dev(rnd(rows, C, seed=4), dtype), dev(rnd(rows, C, seed=5), dtype)
    dt, B, Cm = dev(rnd(rows, C, seed=6)), dev(rnd(rows, N, seed=7), dtype), dev(rnd(rows, N, seed=8), dtype)
    cu = i32([0, lens[0], lens[0] + lens[1], rows])
    need = kn.selective_scan_workspace(3, C, N, max(lens))
    assert need > 0
    res = []
    for more in ({}, dict(max_rows=max(lens), workspace=torch.zeros(need, device=DEV))):
        state = dev(rnd(3, C, N, seed=9))
        out = torch.zeros((rows, C), dtype=dtype, device=DEV)
        kn.selective_scan(x, dt, B, Cm, z, dev(bias), dev(A_log), dev(D), state, out, i32([2, 0, 1]), cu, 3, **more)
        res.append((out.cpu(), state.cpu()))
    assert pc.err(res[1][0], res[0][0]) < (1e-5 if dtype == torch.float32 else 1e-2)
    assert pc.err(res[1][1], res[0][1]) < 1e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("C,taps", [(40, 4), (256, 4), (1024, 3), (51, 2), (8, 1), (130, 5), (24, 9)])
def test_short_convolution_in_either_dtype(kn, C, taps, dtype):
    w, b = rnd(C, taps, seed=1), rnd(C, seed=2)
    lens = (45, 24)
    xs = [rnd(n, C, seed=3 + i).to(dtype).float() for i, n in enumerate(lens)]
    want = [pp.short_conv(x.double(), w.double(), b.double()) for x in xs]
    state = torch.zeros(4, max(1, taps - 1), C, device=DEV)
    at = [0, 0]
    for rows in ((5, 1), (1, 2), (39, 21)):
        slots, cu = i32([2, 0]), i32([0, rows[0], sum(rows)])
        x = torch.cat([xs[i][at[i] : at[i] + n] for i, n in enumerate(rows)])
        wide = dev(torch.cat([x, rnd(sum(rows), C, seed=9)], 1), dtype)  # a run of columns of a wider row
        out = torch.zeros((sum(rows), C), dtype=dtype, device=DEV)
        start = i32(at)
        pos = i32(list(range(at[0], at[0] + rows[0])) + list(range(at[1], at[1] + rows[1])))
        kn.causal_conv(wide[:, :C], dev(w), dev(b), state, out, pos, i32([0] * rows[0] + [1] * rows[1]), slots, start,
                       i32([at[0] + rows[0], at[1] + rows[1]]), cu, 2)
        r = 0
        for i, n in enumerate(rows):
            assert pc.err(out[r : r + n], want[i][at[i] : at[i] + n]) < (2e-6 if dtype == torch.float32 else 1e-2), (rows, i)
            at[i] += n
            r += n
    if taps > 1:
        assert pc.err(state[2], xs[0][-(taps - 1) :].double()) == 0 and pc.err(state[0], xs[1][-(taps - 1) :].double()) == 0


@pytest.mark.parametrize("sizes", [(1, 4, 3, 2.0), (3, 12, 20, 6.0), (2, 64, 64, 15.0), (4, 130, 7, 9.0), (2, 256, 600, 12.0)])
def test_matrix_memory(kn, sizes):
    """The gates, the scan with the column of ones and the output, two sequences in unequal portions (more and fewer than
    64 tokens, so that the running maximum passes a chunk's edge), in slots out of order; gates that reach their cap."""
    H, d, P, cap = sizes
    eps = 1e-3
    lens = (171, 150)
    bi, bf, w = rnd(H, seed=1), rnd(H, seed=2, mean=2.0), rnd(H * P, seed=3, mean=1.0, std=0.3)
    full = []
    for i, n in enumerate(lens):
        q, k, v = rnd(n, H, d, seed=10 + i), rnd(n, H, d, seed=20 + i), rnd(n, H, P, seed=30 + i)
        zi, zf, z = rnd(n, H, seed=40 + i, std=3.0), rnd(n, H, seed=50 + i, std=5.0), rnd(n, H * P, seed=60 + i)
        gi = pp.soft_cap(zi.double() + bi.double(), cap)
        gf = pp.log_sigmoid(pp.soft_cap(zf.double() + bf.double(), cap))
        o = torch.stack([pp.matrix_memory(q[:, h].double() * d ** -0.5, k[:, h].double(), v[:, h].double(), gi[:, h], gf[:, h])
                         for h in range(H)], dim=1)
        o = pp.rms(o, eps).reshape(n, H * P) * w.double() * torch.sigmoid(z.double())
        full.append((q.reshape(n, -1), k.reshape(n, -1), v.reshape(n, -1), zi, zf, z, o))
    state, top = torch.zeros(4, H, P + 1, d, device=DEV), torch.zeros(4, H, device=DEV)
    at = [0, 0]
    for rows in ((3, 100), (1, 1), (130, 49), (37, 0)):
        live = [i for i in (0, 1) if rows[i]]
        slots = i32([(2, 0)[i] for i in live])
        cu = i32([0] + np.cumsum([rows[i] for i in live]).tolist())
        q, k, v, zi, zf, z = (torch.cat([full[i][j][at[i] : at[i] + rows[i]] for i in live]) for j in range(6))
        n = q.shape[0]
        u = dev(torch.cat([q, k, v, zi, zf, z], 1))  # runs of columns of one product
        c = np.cumsum([0] + [t.shape[1] for t in (q, k, v, zi, zf, z)]).tolist()
        col = [u[:, c[j] : c[j + 1]] for j in range(6)]
        decay, take, floor = (torch.zeros(n, H, device=DEV) for _ in range(3))
        kn.memory_gates(col[3], col[4], dev(bi), dev(bf), cap, top, decay, take, floor, slots, cu, len(live))
        y = torch.zeros(n, H * (P + 1), device=DEV)
        kn.ssd_scan(col[2], col[1], col[0], take, None, None, None, state, y, H, P + 1, d, H, slots, cu, len(live), decay=decay,
                    ones=True)
        for dtype in (torch.float32, torch.bfloat16):
            out = torch.zeros((n, H * P), dtype=dtype, device=DEV)
            kn.memory_out(y, floor, col[5], dev(w), d ** -0.5, 1e-6, eps, out)
            r = 0
            for i in live:
                want = full[i][6][at[i] : at[i] + rows[i]]
                assert pc.err(out[r : r + rows[i]], want) < (5e-5 if dtype == torch.float32 else 1e-2), (rows, i)
                r += rows[i]
        for i in live:
            at[i] += rows[i]
    assert bool((state[1] == 0).all()) and bool((top[1] == 0).all())


def test_matrix_memory_of_a_long_prompt_in_segments(kn):
    H, d, P, n = 2, 32, 48, 1100
    q, k, v = (dev(rnd(n, H * w, seed=s)) for s, w in ((1, d), (2, d), (3, P)))
    take, decay = dev(torch.rand(n, H, generator=torch.Generator().manual_seed(4))), dev(1 - 0.02 * torch.rand(n, H))
    need = kn.ssd_scan_workspace(1, H, P + 1, d, n)
    assert need > 0
    res = []
    for more in ({}, dict(max_rows=n, workspace=torch.zeros(need, device=DEV))):
        state = dev(rnd(2, H, P + 1, d, seed=9))
        y = torch.zeros(n, H * (P + 1), device=DEV)
        kn.ssd_scan(v, k, q, take, None, None, None, state, y, H, P + 1, d, H, i32([1]), i32([0, n]), 1, decay=decay, ones=True, **more)
        res.append((y.cpu(), state.cpu()))
    assert pc.err(res[1][0], res[0][0]) < 1e-5 and pc.err(res[1][1], res[0][1]) < 1e-5


@pytest.mark.parametrize("width", [48, 80, 2048, 4096, 51, 8200])
def test_normed_branches_norm_and_residual_in_one_pass(kn, width):
    rows, eps, beps = 19, 1e-5, 1e-3
    x, stack = rnd(rows, width, seed=1), rnd(2, rows, width, seed=2)
    stack[0, 3] *= 1e-3  # (a branch that is nearly nothing: its eps counts)
    ws, b, w = [rnd(width, seed=s, mean=1.0, std=0.3) for s in (3, 4)], rnd(width, seed=5), rnd(width, seed=6, mean=1.0)
    y = 0.5 * (pp.rms(stack[0].double() + b.double(), beps) * ws[0].double() + pp.rms(stack[1].double(), beps) * ws[1].double())
    want = x.double() + pp.rms(y, eps) * w.double()
    mean = torch.zeros(rows, width, device=DEV)
    kn.rmsnorm_mean(dev(stack), [dev(t) for t in ws], beps, mean, biases=[dev(b), None])
    assert pc.err(mean, y) < 3e-6
    for dtype in (torch.bfloat16, None):
        got, rounded = dev(x), None if dtype is None else torch.zeros((rows, width), dtype=dtype, device=DEV)
        kn.rmsnorm_residual(got, mean, dev(w), eps, rounded)
        assert pc.err(got, want) < 3e-6
        if rounded is not None:
            assert torch.equal(rounded, got.to(dtype))
        if not kn.mean_residual_takes(width):
            assert width in (51, 8200)
            continue
        got = dev(x)
        kn.mean_residual(got, dev(stack), [dev(t) for t in ws], [dev(b), None], beps, dev(w), eps, rounded)
        assert pc.err(got, want) < 3e-6
        if rounded is not None:
            assert torch.equal(rounded, got.to(dtype))


@pytest.mark.parametrize("width,dtype", [(48, torch.bfloat16), (51, torch.float32), (2048, torch.bfloat16), (4096, torch.float32)])
def test_lookup_with_sinusoids(kn, width, dtype):
    table = rnd(30, width, seed=1).to(dtype)
    pos = [0, 1, 2, 77, 1000, 99999]
    toks = [3, 29, 0, 7, 7, 31]  # (the last is no row of the table: zeros)
    freqs = torch.tensor([10000.0 ** (-2.0 * i / width) for i in range((width + 1) // 2)], dtype=F)
    out = torch.zeros(len(pos), width, device=DEV)
    kn.embed(dev(table, dtype), i32(toks), out, row_pos=i32(pos), freqs=freqs.to(DEV))
    want = torch.stack([table[t].double() if t < 30 else torch.zeros(width, dtype=F) for t in toks])
    for r, p in enumerate(pos):
        for c in range(width):
            a = p * 10000.0 ** (-(c - c % 2) / width)
            want[r, c] += math.cos(a) if c % 2 else math.sin(a)
    assert float((out.cpu().double() - want).abs().max()) < 1e-6
    assert float((want[3] - want[4]).abs().max()) > 0.1  # one token at two places


@pytest.mark.parametrize("rows,k,inner", [(1, 512, 64), (5, 64, 40), (16, 1024, 2048), (40, 1024, 2048), (300, 512, 2048),
                                          (130, 96, 24), (700, 2048, 2816), (2048, 1024, 4096)])
def test_gated_unit_with_the_tanh_gelu_in_the_products_epilogue(kn, rows, k, inner):
    """Every way the product can take (few rows, some rows, prompts, a remainder of columns in a launch of its own), dense
    and packed weights; the other activation of that epilogue is another function."""
    x, gate, up = rnd(rows, k, seed=1).to(torch.bfloat16), rnd(inner, k, seed=2, std=2 / k ** 0.5), rnd(inner, k, seed=3, std=k ** -0.5)
    gate, up = gate.to(torch.bfloat16), up.to(torch.bfloat16)
    g, u = x.float() @ gate.float().T, x.float() @ up.float().T
    want = pp.gelu_tanh(g.double()) * u.double()
    assert kn.linear_swiglu_supported(torch.bfloat16, 2 * inner, k)
    w = kn.interleave_gate_up(dev(gate, torch.bfloat16), dev(up, torch.bfloat16))
    for weight in (w, kn.pack_weight(w)):
        out = torch.zeros((rows, inner), dtype=torch.bfloat16, device=DEV)
        kn.linear_swiglu(dev(x, torch.bfloat16), weight, out, activation="gelu_tanh")
        assert pc.err(out, want) < 6e-3
    small = want.abs() < 0.1 * want.abs().max()  # (the far tail of the negative gates included)
    assert float((out.cpu().double() - want)[small].abs().max() / want.abs().max()) < 2e-3
    kn.linear_swiglu(dev(x, torch.bfloat16), w, out)
    assert pc.err(out, want) > 2e-2


@pytest.mark.parametrize("rows,n,k", [(1, 40, 2048), (8, 288, 8192), (16, 17, 4096), (3, 160, 2112), (5, 1000, 6144)])
def test_few_rows_of_a_narrow_weight_share_a_long_k_over_blocks(kn, rows, n, k):
    x, w = rnd(rows, k, seed=1).to(torch.bfloat16), rnd(n, k, seed=2, std=k ** -0.5).to(torch.bfloat16)
    pieces = kn.linear_narrow_pieces(torch.bfloat16, rows, n, k)
    assert pieces > 1 or k == 2112
    if pieces == 1:
        return
    parts, out = torch.zeros((pieces, rows, n), device=DEV), torch.zeros((rows, n), device=DEV)
    kn.linear(dev(x, torch.bfloat16), dev(w, torch.bfloat16), parts)
    kn.sum_pieces(parts, out)
    assert pc.err(out, x.double() @ w.double().T) < 2e-6
    assert all(float(p.abs().max()) > 0 for p in parts)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_pieces_of_a_product_added_up(kn, dtype):
    pieces = rnd(5, 37, 21, seed=1)
    out = torch.full((37, 30), 9.0, dtype=dtype, device=DEV)
    kn.sum_pieces(dev(pieces), out[:, :21])
    assert pc.err(out[:, :21], pieces.double().sum(0)) < (1e-6 if dtype == torch.float32 else 5e-3)
    assert bool((out[:, 21:] == 9.0).all())


def test_short_convolution_of_many_rows(kn):
    """Rows enough for several a thread: two long sequences and a short one, whose rows meet inside a thread's run, from
    states that an earlier step left; the same bits as row by row."""
    C, taps, lens = 136, 4, (301, 3, 290)
    w, b = dev(rnd(C, taps, seed=1)), dev(rnd(C, seed=2))
    for dtype in (torch.float32, torch.bfloat16):
        x, n = dev(rnd(sum(lens), C, seed=3), dtype), sum(lens)
        before = rnd(3, taps - 1, C, seed=4)
        start = [7, 0, 2]
        before[1] = 0  # (the second sequence is at its start)
        cu = i32([0] + np.cumsum(lens).tolist())
        pos = [s + i for s, l in zip(start, lens) for i in range(l)]
        seq = [i for i, l in enumerate(lens) for _ in range(l)]
        out, state = torch.zeros((n, C), dtype=dtype, device=DEV), dev(before)
        kn.causal_conv(x, w, b, state, out, i32(pos), i32(seq), i32([0, 1, 2]), i32(start),
                       i32([s + l for s, l in zip(start, lens)]), cu, 3)
        at = 0
        for i, l in enumerate(lens):
            hist = torch.cat([before[i].double(), x[at : at + l].cpu().double()])
            want = pp.short_conv(hist, w.cpu().double(), b.cpu().double())[taps - 1 :]
            assert pc.err(out[at : at + l], want) < (2e-6 if dtype == torch.float32 else 1e-2)
            assert pc.err(state[i], hist[-(taps - 1) :]) == 0
            at += l
        single = dev(before)
        for t in range(3):  # single tokens of all three: the same bits
            rows = [0 + t, 301 + t, 304 + t]
            one = torch.zeros((3, C), dtype=dtype, device=DEV)
            kn.causal_conv(x[rows].contiguous(), w, b, single, one, i32([7 + t, t, 2 + t]), i32(range(3)), i32([0, 1, 2]),
                           i32([7 + t, t, 2 + t]), i32([8 + t, 1 + t, 3 + t]), i32(range(4)), 3)
            assert torch.equal(one, out[rows])


def test_shaped_sizes_that_do_not_fit_are_refused(kn):
    from longbow_quarrel_amd.kernels.hip import KernelLibraryError
    cache = Paged(4, 1, 16, 16, torch.float32)
    q, out = torch.zeros(4, 32, device=DEV), torch.zeros(4, 32, device=DEV)
    args = (q, out, 2, 1, 16, 16, i32(range(4)), i32([0] * 4), i32([0]), cache.table, cache.k, cache.v, 64, 1.0)
    for more in (dict(temp=torch.zeros(3, device=DEV)), dict(distance_bias=torch.zeros(3, 5, device=DEV)),
                 dict(wide_gate=torch.zeros(4, 16, device=DEV)), dict(log_bias=(torch.zeros(2, device=DEV), None)),
                 dict(softcap=-1.0)):
        with pytest.raises(KernelLibraryError):
            kn.sink_attention(*args, sink=False, **more)
    with pytest.raises(KernelLibraryError):
        kn.qkv_norm_store(torch.zeros(4, 64, device=DEV), q, 2, 1, 16, 16, 0.0, q_weight=torch.zeros(16, device=DEV))


# ---- the engine ------------------------------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    made = {}

    def get(name, dtype="float32", **kw):
        key = (name, dtype, tuple(sorted((k, str(v)) for k, v in kw.items())))
        if key not in made:
            made[key] = pc.Case(tmp_path_factory.mktemp("puzonex"), name, load, dtype=dtype,
                                rounding=dtype == "bfloat16", **kw)
        return made[key]

    return get


@pytest.mark.parametrize("name", ["log", "table", "memory", "scan", "dense"])
def test_a_mechanism_alone(cases, name):
    case = cases(name)
    pc.whole_and_token_by_token(case, TOL_F32, lengths=(1, 2, 9, 70))
    pc.portions(case, TOL_F32, n=140)


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_float32_under_every_cutting_and_batching(cases, name):
    case = cases(name)
    pc.whole_and_token_by_token(case, TOL_F32)
    pc.portions(case, TOL_F32)
    pc.unequal_batches(case, TOL_F32)
    pc.slots_and_blocks_used_again(case, TOL_F32)


@pytest.mark.parametrize("seed", range(1, 13))
def test_configurations_drawn_from_a_seed(cases, seed):
    """Other sizes, head counts, windows, caps, tables, states, layer orders and constants, in both dtypes."""
    case = cases(seed)
    t, u = pc.tokens(200, case.vocab, seed), pc.tokens(9, case.vocab, seed + 50)
    assert pc.err(case.run_cut(t, [150, 2, 1, 20]), case.want(t)) < TOL_F32
    eng = case.eng
    sa, sb = eng.new_sequence(), eng.new_sequence()
    out = eng.step([StepEntry(sa, u[:8], range(8)), StepEntry(sb, t[:130], range(130))])
    assert pc.err(out, torch.cat([case.want(u)[:8], case.want(t)[:130]])) < TOL_F32
    out = eng.step([StepEntry(sa, u[8:], [0]), StepEntry(sb, t[130:131], [0])])
    assert pc.err(out, torch.stack([case.want(u)[8], case.want(t)[130]])) < TOL_F32
    eng.release(sa)
    eng.release(sb)
    case.assert_idle()
    case16 = cases(seed, "bfloat16")
    pc.assert_close_bf16(case16.run_cut(t, [150, 2]), case16.want(t), case16.noise(t))


def test_the_residual_stream_after_every_layer(cases):
    case = cases("a")
    got, want = case.layers(pc.tokens(37, case.vocab, 8))
    assert len(got) == len(want) == 6
    for i, (g, w) in enumerate(zip(got, want)):
        assert pc.err(g, w) < TOL_F32, f"after layer {i}"


@pytest.mark.parametrize("kind", ["log", "table"])
@pytest.mark.parametrize("window", [1, 2, 63, 64, 65, 130])
def test_keys_just_inside_and_just_outside_the_window(cases, kind, window):
    """Peaked attention under windows of one token, of a cache block less one, a block, a block and one, and two
    blocks and two: the last key a row sees and the first it does not, in a prompt, across portions and in
    decoding.  The plain implementation with a window one token off differs by much at these rows."""
    case = cases(f"{kind}-window-{window}", cfg=pc.windowed(kind, window), sharp=6.0)
    n = max(2 * window + 10, 80)
    t = pc.tokens(n, case.vocab, 40 + window)
    pc.a_window_off_by_one_would_show(case, t, list(range(window, n)))
    want = case.want(t)
    assert pc.err(case.run_cut(t, [n]), want) < TOL_F32
    assert pc.err(case.run_cut(t, [window, 1, 1, 2, window - 1 or 1, 3]), want) < TOL_F32
    assert pc.err(case.run_cut(t, [max(1, window - 1)]), want) < TOL_F32  # decoding across the window's edge
    case.assert_idle()
    case16 = cases(f"{kind}-window-{window}", "bfloat16", cfg=pc.windowed(kind, window), sharp=6.0)
    pc.assert_close_bf16(case16.run_cut(t, [max(1, window - 1)]), case16.want(t), case16.noise(t))


@pytest.mark.parametrize("name", ["log", "table"])
def test_attention_without_a_window_over_hundreds_of_tokens(cases, name):
    """The cap binds, the logarithm keeps falling, the table's last row serves every far distance."""
    cfg = copy.deepcopy(pc.CONFIGS[name])
    del pc.attention_of(cfg)["mask"]
    case = cases(f"{name}-open", cfg=cfg, sharp=3.0)
    t = pc.tokens(400, case.vocab, 6)
    assert pc.err(case.run_cut(t, [330, 3]), case.want(t)) < TOL_F32


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_bfloat16_whole_in_portions_and_in_batches(cases, name):
    case = cases(name, "bfloat16")
    t = pc.tokens(150, case.vocab, 3)
    want, noise = case.want(t), case.noise(t)
    pc.assert_close_bf16(case.run_cut(t, [150]), want, noise)
    pc.assert_close_bf16(case.run_cut(t, [64, 1, 63, 2, 3]), want, noise)
    u = pc.tokens(70, case.vocab, 4)
    eng = case.eng
    sa, sb = eng.new_sequence(), eng.new_sequence()
    out = eng.step([StepEntry(sa, t[:100], range(100)), StepEntry(sb, u[:3], range(3))])
    pc.assert_close_bf16(out, torch.cat([want[:100], case.want(u)[:3]]), noise)
    got = []
    for i in range(20):
        got.append(eng.step([StepEntry(sb, [u[3 + i]], [0]), StepEntry(sa, [t[100 + i]], [0])]).clone())
    got = torch.cat(got)
    pc.assert_close_bf16(torch.cat([got[0::2], got[1::2]]), torch.cat([case.want(u)[3:23], want[100:120]]), noise)
    eng.release(sa)
    eng.release(sb)
    case.assert_idle()


def test_bfloat16_decoding_over_long_contexts(cases):
    """Single tokens over several hundred positions (the windows long since full, their first blocks given back)
    against the same rows as parts of a prompt and against the plain implementation."""
    case = cases("c", "bfloat16")
    t, u = pc.tokens(640, case.vocab, 61), pc.tokens(330, case.vocab, 62)
    eng = case.eng
    sa, sb = eng.new_sequence(), eng.new_sequence()
    whole = eng.step([StepEntry(sa, t, range(600, 640)), StepEntry(sb, u, range(290, 330))]).clone()
    eng.release(sa)
    eng.release(sb)
    sa, sb = eng.new_sequence(), eng.new_sequence()
    eng.step([StepEntry(sa, t[:600], []), StepEntry(sb, u[:290], [])])
    got = torch.cat([eng.step([StepEntry(sa, [t[600 + i]], [0]), StepEntry(sb, [u[290 + i]], [0])]).clone() for i in range(40)])
    eng.release(sa)
    eng.release(sb)
    case.assert_idle()
    got = torch.cat([got[0::2], got[1::2]])
    want = torch.cat([case.want(t)[600:], case.want(u)[290:]])
    noise = max(case.noise(t), case.noise(u))
    pc.assert_close_bf16(got, want, noise)
    pc.assert_close_bf16(got, whole.double(), noise)


@pytest.mark.parametrize("name", ["scan", "memory"])
def test_a_slow_decay_keeps_old_tokens_in_the_state(cases, name):
    """Also over a prompt long enough for the scans in segments."""
    case = cases(f"{name}-slow", cfg=pc.long_memory(name), memory=5.0)
    t = pc.tokens(700, case.vocab, 31)
    want = case.want(t)
    other = case.want([(t[0] + 1) % case.vocab] + t[1:260])
    assert pc.err(other[-1], want[259]) > 1e-3  # the first token still matters, far beyond the window
    assert pc.err(case.run_cut(t, [700]), want) < TOL_F32
    assert pc.err(case.run_cut(t[:260], [3, 64, 1, 2, 130]), want[:260]) < TOL_F32
    assert pc.err(case.run_cut(t, [100, 560, 2]), want) < TOL_F32


def test_a_narrow_product_that_shares_its_channels_over_blocks(cases):
    """Channels enough that the product of step sizes, B and C leaves pieces (and is added up) in a long prompt and not in a
    short one."""
    cfg = copy.deepcopy(pc.CFG_SCAN)
    cfg["layers"][0]["mixer"].update(inner=2048, state=16, dt_rank=8)
    case = cases("scan-wide", "bfloat16", cfg=cfg)
    assert case.eng.kernels.linear_pieces(torch.bfloat16, 300, 40, 2048) > 1
    t = pc.tokens(300, case.vocab, 3)
    pc.assert_close_bf16(case.run_cut(t, [300]), case.want(t), case.noise(t))
    pc.assert_close_bf16(case.run_cut(t, [9, 270, 2]), case.want(t), case.noise(t))


def test_the_first_tokens_see_zeros_ahead_of_the_sequence(cases):
    case = cases("a")
    eng = case.eng
    a, b = pc.tokens(150, case.vocab, 1), pc.tokens(6, case.vocab, 2)
    sa = eng.new_sequence()
    eng.step([StepEntry(sa, a, [])])
    eng.release(sa)
    for first in (1, 2, 3, 6):
        s = eng.new_sequence()
        assert s == sa
        out = eng.step([StepEntry(s, b[:first], range(first))])
        assert pc.err(out, case.want(b)[:first]) < TOL_F32
        if first < 6:
            out = eng.step([StepEntry(s, b[first:], range(6 - first))])
            assert pc.err(out, case.want(b)[first:]) < TOL_F32
        eng.release(s)
    case.assert_idle()


@pytest.mark.parametrize("name", ["a", "c"])
def test_long_decoding(cases, name):
    pc.long_decoding(cases(name), TOL_F32)


def test_float32_logits_do_not_depend_on_the_cutting_or_the_batch_by_more_than_rounding(cases):
    case = cases("c")
    t, u = pc.tokens(140, case.vocab, 7), pc.tokens(30, case.vocab, 8)
    whole = case.run_cut(t, [140]).double()
    assert pc.err(case.run_cut(t, [64, 1, 2, 70]), whole) < 1e-5 and pc.err(case.run_cut(t, [100]), whole) < 1e-5
    eng = case.eng
    sa, sb = eng.new_sequence(), eng.new_sequence()
    out = eng.step([StepEntry(sb, u, []), StepEntry(sa, t[:90], range(90))])
    assert pc.err(out, whole[:90]) < 1e-5
    out = eng.step([StepEntry(sa, [t[90]], [0]), StepEntry(sb, [5], [])])
    assert pc.err(out[0], whole[90]) < 1e-5
    eng.release(sa)
    eng.release(sb)


@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation_through_the_entry_point(cases, graphs):
    case = cases("a")
    reqs, wants = pc.greedy(case, n_new=12, prompts=5)
    res = lq.generate(case.eng, reqs, max_new_tokens=12, max_batch=3, stop_ids=[], use_graphs=graphs)
    assert res.tokens == wants
    case.assert_idle()


def test_generation_in_bfloat16_captured_and_direct_steps_agree_and_stop_ids_end_requests(cases):
    case = cases("c", "bfloat16")
    assert case.eng.graph_safe
    reqs = [pc.tokens(n, case.vocab, 40 + n) for n in (3, 70, 9, 1, 130, 20)]
    direct = lq.generate(case.eng, reqs, max_new_tokens=40, max_batch=4, stop_ids=[], use_graphs=False)
    stop = direct.tokens[1][7]
    a = lq.generate(case.eng, reqs, max_new_tokens=40, max_batch=4, stop_ids=[stop], use_graphs=False)
    b = lq.generate(case.eng, reqs, max_new_tokens=40, max_batch=4, stop_ids=[stop], use_graphs=True)
    assert a.tokens == b.tokens and a.finish == b.finish and "stop" in a.finish
    case.assert_idle()


def test_command_line_and_trace_replay(cases, tmp_path):
    case = cases("b")
    reqs, wants = pc.greedy(case, n_new=5, prompts=1)
    out = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "quarrel"), "-model", case.folder, "-dtype", "float32",
                          "-prompt", " ".join(map(str, reqs[0])), "-n", "5", "-temp", "0", "-penalty", "1"],
                         capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    assert "Architecture: Puzonex" in out.stdout
    assert out.stdout.strip().splitlines()[-1].split() == [str(t) for t in wants[0]]
    a, b = pc.tokens(70, case.vocab, 1), pc.tokens(9, case.vocab, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:66], "want": [0, 65]}, {"id": "b", "tokens": b[:7], "want": [6]}],
              "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [a[66]], "want": [0]}, {"id": "b", "tokens": [b[7]], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": [a[67]], "want": []}, {"id": "b", "tokens": [b[8]], "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[68:], "want": [1]}], "end": ["a"]}]
    for dtype, check in (("float32", lambda g, w: pc.err(g, w) < TOL_F32), ("bfloat16", lambda g, w: pc.err(g, w) < 0.1)):
        folder = tmp_path / dtype
        folder.mkdir()
        proc = subprocess.Popen([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", case.folder, "--dtype", dtype,
                                 "--out", str(folder), "--max-tokens", "79"], stdin=subprocess.PIPE, stdout=subprocess.PIPE,
                                stderr=subprocess.PIPE, text=True)
        try:
            for st in steps:
                proc.stdin.write(json.dumps(st) + "\n")
                proc.stdin.flush()
                assert proc.stdout.readline().strip() == f"done {st['step']}", proc.stderr.read()[-3000:]
            proc.stdin.close()
            assert proc.wait(timeout=120) == 0
        finally:
            if proc.poll() is None:
                proc.kill()
        read = lambda n: torch.from_numpy(np.fromfile(os.path.join(str(folder), f"{n}.f32"), dtype="<f4").reshape(-1, case.vocab).copy())
        wa, wb = case.want(a), case.want(b)
        assert check(read(0), torch.stack([wa[0], wa[65], wb[6]]))
        assert check(read(1), wa[66:67]) and check(read(2), wb[8:9]) and check(read(3), wa[69:70])
