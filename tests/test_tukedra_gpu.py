"""The Tukedra design on the GPU.  First every kernel that the design brought, or widened, alone against the plain
implementation's function of the same mechanism (float64), with inputs made so that a fault shows; then the engine
in float32 and in bfloat16 under every cutting and batching; then generation through the entry point, with captured
steps and direct ones, the command line and the trace replay."""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import longbow_quarrel_amd as lq
import plain_tukedra as pt
import tukedra_cases as tc
from longbow_quarrel_amd.engine import StepEntry
from longbow_quarrel_amd.parts.linear_attention import decay_powers

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEV = "cuda:0"
TOL_F32 = 5e-5
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


# ---- the kernels alone -------------------------------------------------------------------------------------------
SCANS = [
    # heads, key size, value size, activation, rotated entries, interleaved, key scale
    (4, 32, 80, "silu", 0, False, 1.0), (3, 64, 40, None, 64, False, 0.2), (2, 24, 40, None, 16, False, 0.5),
    (1, 7, 9, "silu", 0, False, 1.0), (5, 6, 1, None, 2, True, 2.0), (2, 128, 128, None, 128, False, 0.1),
    (1, 256, 160, "silu", 100, True, 0.3), (2, 130, 70, "silu", 130, False, 1.0), (3, 20, 300, None, 6, True, 1.0),
    (1, 300, 24, None, 40, False, 0.2), (1, 600, 5, "silu", 0, False, 1.0), (16, 16, 16, "silu", 4, False, 1.0),
    (2, 48, 130, None, 48, True, 0.7), (1, 1, 3, "silu", 0, False, 1.0), (1, 1024, 16, None, 1000, False, 0.05),
    (2, 301, 6, None, 0, False, 1.0),
]


def taken_in(x, heads, act, freqs, interleaved, scale=1.0):
    x = x.double().reshape(x.shape[0], heads, -1)
    x = pt.silu(x) if act else x
    return (pt.rotate(x, freqs, 1.3, interleaved) if freqs else x) * scale


@pytest.mark.parametrize("sizes", SCANS)
def test_linear_attention_with_a_fixed_decay(kn, sizes):
    """Two sequences in unequal portions, in slots out of order, as runs of columns of one product: portions of one and a few
    tokens (walked one by one) and long ones (in chunks; lengths on and beside a chunk's edge), each way from the states
    that the other left.  Decays from one that forgets at once to one that forgets nothing."""
    H, N, P, act, dims, inter, scale = sizes
    decay = [0.9, 1.0, 0.5, 0.999, 0.0][:H] + [0.97] * max(0, H - 5)
    freqs = pt.frequencies(dims, 100.0) if dims else []
    lens = (290, 197)
    full = []
    for i, n in enumerate(lens):
        q, k, v = rnd(n, H * N, seed=10 + i), rnd(n, H * N, seed=20 + i), rnd(n, H * P, seed=30 + i)
        Q, K, V = taken_in(q, H, act, freqs, inter), taken_in(k, H, act, freqs, inter, scale), taken_in(v, H, act, [], inter)
        o = torch.stack([pt.decayed_memory(Q[:, h], K[:, h], V[:, h], decay[h]) for h in range(H)], dim=1).reshape(n, -1)
        full.append((q, k, v, o))
    powers = decay_powers(decay, 64).to(DEV)
    for cuts in (((1, 3), (64, 129), (1, 1), (65, 1), (159, 63)), ((150, 2), (2, 130), (138, 65))):
        state = torch.zeros(4, H, P, N, device=DEV)
        at = [0, 0]
        for rows in cuts:
            q, k, v = (torch.cat([full[i][j][at[i] : at[i] + rows[i]] for i in (0, 1)]) for j in range(3))
            u = dev(torch.cat([rnd(sum(rows), 4, seed=1), q, k, v, rnd(sum(rows), 4, seed=2)], 1))
            cols = [u[:, a : a + n] for a, n in ((4, H * N), (4 + H * N, H * N), (4 + 2 * H * N, H * P))]
            more = {}
            if dims:
                pos = i32(list(range(at[0], at[0] + rows[0])) + list(range(at[1], at[1] + rows[1])))
                table = torch.zeros(sum(rows), dims // 2, 2, device=DEV)
                kn.rope_table(torch.tensor(freqs, dtype=F, device=DEV), pos, table)
                more = dict(cos_sin=table, interleaved=inter, magnitude=1.3)
            need = kn.decay_scan_workspace(sum(rows), 2, H, N, P, max(rows))
            assert (need > 0) == (max(rows) >= 24 and N <= 256)
            if need:
                more.update(max_rows=max(rows), workspace=torch.full((need,), float("nan"), device=DEV))
            out = torch.zeros(sum(rows), H * P, device=DEV)
            kn.decay_scan(*cols, powers, state, out, H, N, P, scale, i32([2, 0]), i32([0, rows[0], sum(rows)]), 2, activation=act,
                          **more)
            r = 0
            for i, n in enumerate(rows):
                want = full[i][3]
                got = out[r : r + n].cpu().double() - want[at[i] : at[i] + n]
                assert float(got.abs().max() / want.abs().max()) < 3e-6, (cuts, rows, i)
                at[i] += n
                r += n
        assert at == list(lens)
        assert bool((state[1] == 0).all()) and bool((state[3] == 0).all())  # nobody's slots


@pytest.mark.parametrize("N,P", [(32, 48), (7, 9), (256, 16)])
def test_single_tokens_give_the_bits_of_a_short_portion(kn, N, P):
    H = 3
    powers = decay_powers([0.9, 0.99, 0.5], 64).to(DEV)
    q, k, v = (dev(rnd(12, H * w, seed=s)) for s, w in ((1, N), (2, N), (3, P)))
    start = rnd(4, H, P, N, seed=4)
    whole, state = torch.zeros(12, H * P, device=DEV), dev(start)
    kn.decay_scan(q, k, v, powers, state, whole, H, N, P, 1.0, i32([3, 1]), i32([0, 6, 12]), 2, activation="silu")
    single = dev(start)
    for t in range(6):
        rows = [t, 6 + t]
        one = torch.zeros(2, H * P, device=DEV)
        kn.decay_scan(*(x[rows].contiguous() for x in (q, k, v)), powers, single, one, H, N, P, 1.0, i32([3, 1]), i32([0, 1, 2]), 2,
                      activation="silu")
        assert torch.equal(one, whole[rows]), t
    assert torch.equal(single, state)


def test_chunks_of_many_unequal_sequences(kn):
    """Portions of every length around a chunk's, in one launch, from states that are not zero."""
    H, N, P = 2, 16, 24
    lens = [1, 64, 63, 65, 2, 128, 129, 1, 200, 127, 30]
    rows = sum(lens)
    decay = [0.95, 0.999]
    q, k, v = rnd(rows, H * N, seed=1), rnd(rows, H * N, seed=2), rnd(rows, H * P, seed=3)
    start = rnd(len(lens), H, P, N, seed=4)
    slots = torch.randperm(len(lens), generator=torch.Generator().manual_seed(5)).tolist()
    cu = np.cumsum([0] + lens).tolist()
    state, out = dev(start), torch.zeros(rows, H * P, device=DEV)
    need = kn.decay_scan_workspace(rows, len(lens), H, N, P, max(lens))
    kn.decay_scan(dev(q), dev(k), dev(v), decay_powers(decay, 64).to(DEV), state, out, H, N, P, 1.0, i32(slots), i32(cu), len(lens),
                  max_rows=max(lens), workspace=torch.full((need,), float("nan"), device=DEV))
    for b, n in enumerate(lens):
        for h in range(H):
            S = start[slots[b], h].double()  # [P, N]
            for t in range(n):
                r = cu[b] + t
                S = decay[h] * S + torch.outer(v[r, h * P : (h + 1) * P].double(), k[r, h * N : (h + 1) * N].double())
                o = S @ q[r, h * N : (h + 1) * N].double()
                assert float((out[r, h * P : (h + 1) * P].cpu().double() - o).abs().max()) < 1e-4, (b, t)
            assert tc.err(state[slots[b], h], S) < 3e-6


@pytest.mark.parametrize("streams", [1, 2, 3, 4, 5, 16])
@pytest.mark.parametrize("width", [48, 336, 2048, 4096, 8192, 51, 8196])
def test_streams_written_and_read_in_one_pass(kn, streams, width):
    rows, eps = 7, 1e-3
    X, Y = rnd(streams, rows, width, seed=1), rnd(3, rows, width, seed=2)
    X[:, 3] *= 1e-3  # (a row that is nearly nothing: its eps counts)
    Y[:, 3] *= 1e-3
    mix, out_w, read, w = (rnd(*s, seed=9 + i) for i, s in enumerate(((streams, streams), (streams,), (streams,), (width,))))
    D = lambda t: t.double()
    for y in (Y[0], Y[:1], Y):
        whole = D(y) if y.dim() == 2 else D(y).sum(0)
        for src in (X, X[0]):
            old = D(src).expand(streams, rows, width)
            new = pt.write_streams(old, whole, D(mix), D(out_w))
            for dtype in (torch.float32, torch.bfloat16):
                for weights in (read, None):
                    u = pt.read_streams(new, D(weights) if weights is not None else torch.ones(streams, dtype=F))
                    h = torch.zeros((rows, width), dtype=dtype, device=DEV)
                    given = dev(src)
                    at = given if src.dim() == 3 else torch.zeros(streams, rows, width, device=DEV)  # in place, or from the one
                    kn.streams_step(given, streams, y=dev(y), mix=dev(mix), out_weights=dev(out_w), out=at,
                                    read=None if weights is None else dev(weights), norm_weight=dev(w), eps=eps, h=h)
                    assert tc.err(at, new) < 2e-6
                    assert tc.err(h, pt.rms(u, eps) * D(w)) < (4e-6 if dtype == torch.float32 else 6e-3)
            at = torch.zeros(streams, rows, width, device=DEV)
            kn.streams_step(dev(src), streams, y=dev(y), mix=dev(mix), out_weights=dev(out_w), out=at)  # nothing reads them yet
            assert tc.err(at, new) < 2e-6
    for src in (X, X[0]):  # only read
        h = torch.zeros((rows, width), device=DEV)
        kn.streams_step(dev(src), streams, read=dev(read), norm_weight=dev(w), eps=eps, h=h)
        assert tc.err(h, pt.rms(pt.read_streams(D(src).expand(streams, rows, width), D(read)), eps) * D(w)) < 4e-6


def test_cap_on_logits(kn):
    x = rnd(5, 997, seed=1, std=20.0)
    got = dev(x)
    kn.softcap(got, 7.0, 0.3)
    assert tc.err(got, 7.0 * torch.tanh(x.double() * 0.3 / 7.0)) < 1e-6
    kn.softcap(got, 1e9, 1.0)


SHAPES = [
    # query heads, key heads, size, chunk, generic kernel
    (4, 2, 32, 20, False), (8, 2, 64, 64, False), (6, 2, 48, 65, False), (3, 1, 16, 63, False), (1, 1, 128, 1, False),
    (16, 1, 32, 130, False), (5, 5, 10, 40, False), (2, 2, 24, 100, False), (8, 4, 64, 7, True), (4, 2, 64, 64, True),
]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", SHAPES)
def test_attention_within_chunks(kn, sizes, dtype):
    """Every row's query is aimed at one key (its score stands out): the first of its chunk and, in the rows between, the last
    of the chunk before, in turn; the chunk's edges lie on, just beside and far from a cache block's."""
    H, G, D, chunk, generic = sizes
    T = 300
    q, k, v = rnd(T, H, D, seed=1), rnd(T, G, D, seed=2), rnd(T, G, D, seed=3)
    for i in range(T):
        j = i // chunk * chunk - (i % 2)
        if j >= 0:
            for h in range(H):
                q[i, h] = k[j, h // (H // G)] * 6.0 / k[j, h // (H // G)].norm()
    q, k, v = (t.to(dtype).double() for t in (q, k, v))
    scale = 1.3 / math.sqrt(D)

    def plain(size):
        seen = pt.chunk_mask(T, size)
        return torch.stack([pt.softmax_rows(q[:, h] @ k[:, h // (H // G)].T * scale, seen) @ v[:, h // (H // G)] for h in range(H)],
                           dim=1).reshape(T, -1)

    want = plain(chunk)
    assert tc.err(plain(chunk + 1)[chunk:], want[chunk:]) > 1e-2 and (chunk == 1 or tc.err(plain(chunk - 1), want) > 1e-2)
    cache = Paged(T, G, D, D, dtype, seed=5)
    pos, seq, slot = i32(range(T)), i32([0] * T), i32([0])
    kn.force_generic = generic
    try:
        kn.kv_store(dev(k.reshape(T, -1), dtype), dev(v.reshape(T, -1), dtype), G, D, D, pos, seq, slot, cache.table, cache.k, cache.v, 64)
        qd = dev(q.reshape(T, -1), dtype)
        out = torch.zeros((T, H * D), device=DEV)
        kn.sink_attention(qd, out, H, G, D, D, pos, seq, slot, cache.table, cache.k, cache.v, 64, scale, sink=False, chunk=chunk)
        assert tc.err(out, want) < 4e-5
        some = [0, 1, chunk - 1, chunk, chunk + 1, 2 * chunk - 1, 2 * chunk, 63, 64, 127, 128, 129, 255, 256, T - 1]
        need = kn.sink_attention_workspace(dtype, 1, 1, H, G, D, D, 64, 0, 0, T, chunk=chunk)
        more = dict(max_len=T, workspace=torch.zeros(need, device=DEV)) if need else {}
        for r in sorted({r for r in some if r < T}):  # single tokens
            one = torch.zeros((1, H * D), device=DEV)
            kn.sink_attention(qd[r : r + 1], one, H, G, D, D, i32([r]), i32([0]), slot, cache.table, cache.k, cache.v, 64, scale,
                              sink=False, decode=True, chunk=chunk, **more)
            assert tc.err(one[0], want[r]) < 4e-5, r
        lo, hi = 90, 260  # a portion of the rows
        part = torch.zeros((hi - lo, H * D), device=DEV)
        kn.sink_attention(qd[lo:hi], part, H, G, D, D, i32(range(lo, hi)), i32([0] * (hi - lo)), slot, cache.table, cache.k, cache.v,
                          64, scale, sink=False, chunk=chunk)
        assert tc.err(part, want[lo:hi]) < 4e-5
    finally:
        kn.force_generic = False


def test_single_tokens_in_large_chunks_share_their_keys_out_over_workgroups(kn):
    H, G, D, T, chunk, dtype = 4, 1, 64, 1500, 1100, torch.bfloat16
    q, k, v = (rnd(T, n, D, seed=s).to(dtype).double() for s, n in ((1, H), (2, G), (3, G)))
    scale = 1.0 / math.sqrt(D)
    seen = pt.chunk_mask(T, chunk)
    cache = Paged(T, G, D, D, dtype, seed=5)
    kn.kv_store(dev(k.reshape(T, -1), dtype), dev(v.reshape(T, -1), dtype), G, D, D, i32(range(T)), i32([0] * T), i32([0]), cache.table,
                cache.k, cache.v, 64)
    need = kn.sink_attention_workspace(dtype, 1, 1, H, G, D, D, 64, 0, 0, T, chunk=chunk)
    assert need > 0
    for r in (T - 1, 1099, 1100, 1101, 800, 1180):
        want = torch.cat([pt.softmax_rows((q[r : r + 1, h] @ k[:, 0].T) * scale, seen[r : r + 1]) @ v[:, 0] for h in range(H)], dim=1)
        one = torch.zeros((1, H * D), device=DEV)
        kn.sink_attention(dev(q[r : r + 1].reshape(1, -1), dtype), one, H, G, D, D, i32([r]), i32([0]), i32([0]), cache.table, cache.k,
                          cache.v, 64, scale, sink=False, decode=True, chunk=chunk, max_len=T, workspace=torch.zeros(need, device=DEV))
        assert tc.err(one, want) < 4e-5, r


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [
    # heads, kv heads, size, value size (0: the keys), rotated entries, interleaved, norm of q and k, weighted
    (4, 2, 32, 0, 12, True, "head", False), (6, 2, 24, 0, 24, True, "head", False), (3, 1, 7, 0, 4, True, "head", False),
    (8, 2, 64, 64, 64, False, "head", True), (5, 5, 10, 6, 6, False, None, False), (8, 4, 128, 0, 100, False, "head", False),
    (2, 1, 600, 0, 300, True, "head", False), (16, 4, 128, 0, 64, True, "head", False), (2, 2, 16, 0, 2, True, None, False),
])
def test_biases_rotation_norm_and_the_store_of_q_k_and_v(kn, sizes, dtype):
    H, G, D, P, dims, inter, norm, weighted = sizes
    T, eps, mag = 75, 1e-2, 1.2
    tied = P == 0
    P = P or D
    qw, kw, vw = H * D, G * D, 0 if tied else G * P
    src, bias = rnd(T, qw + kw + vw, seed=1), rnd(qw + kw + vw, seed=2)
    wq, wk = (rnd(D, seed=3, mean=1.0, std=0.3), rnd(D, seed=4, mean=1.0, std=0.3)) if weighted else (None, None)
    freqs = pt.frequencies(dims, 50.0)
    t = src.double() + bias.double()
    v = t[:, qw : qw + kw] if tied else t[:, qw + kw :]

    def ready(x, n, w):
        x = pt.rotate(x.reshape(T, n, D), freqs, mag, inter)
        x = pt.rms(x, eps) if norm else x
        return (x if w is None else x * w.double()).reshape(T, -1)

    q, k = ready(t[:, :qw], H, wq), ready(t[:, qw : qw + kw], G, wk)
    wide = dev(torch.cat([rnd(T, 4, seed=5), src, rnd(T, 4, seed=6)], 1))[:, 4 : 4 + qw + kw + vw]
    cache = Paged(T, G, D, P, dtype, seed=7)
    out = torch.zeros((T, qw), dtype=dtype, device=DEV)
    args = dict(bias=dev(bias), q_weight=None if wq is None else dev(wq), k_weight=None if wk is None else dev(wk), norm_qk=norm,
                v_from_k=tied, interleaved=inter, magnitude=mag)
    tol = 3e-6 if dtype == torch.float32 else 1e-2
    for lo, hi in ((0, 70), (70, T)):
        table = torch.zeros(hi - lo, dims // 2, 2, device=DEV)
        kn.rope_table(torch.tensor(freqs, dtype=F, device=DEV), i32(range(lo, hi)), table)
        place = dict(row_pos=i32(range(lo, hi)), row_seq=i32([0] * (hi - lo)), seq_slot=i32([0]), block_table=cache.table,
                     kcache=cache.k, vcache=cache.v, block_size=64)
        kn.qkv_norm_store(wide[lo:hi], out[lo:hi], H, G, D, P, eps, cos_sin=table, **args)  # q alone
        assert tc.err(out[lo:hi], q[lo:hi]) < tol
        out[lo:hi] = 0
        kn.qkv_norm_store(wide[lo:hi], out[lo:hi], H, G, D, P, eps, cos_sin=table, **args, **place)
    assert tc.err(out, q) < tol
    gk, gv = cache.read(T)
    assert tc.err(gk.reshape(T, -1), k) < tol and tc.err(gv.reshape(T, -1), v) < tol


@pytest.mark.parametrize("experts,top", [(11, 4), (2, 1), (7, 7), (64, 8), (1, 1), (5, 3)])
def test_router_with_a_softmax_over_the_chosen_logits(kn, experts, top):
    rows = 130
    z = rnd(rows, experts, seed=1, std=3.0)
    z[3] = 0.5  # a tie of all: the lower indices win
    z[5] *= 60.0  # far apart: weights that vanish beside one, none of them lost
    z[7, :] -= 200.0
    wide = dev(torch.cat([z, rnd(rows, 3, seed=2)], 1))[:, :experts]
    route = torch.zeros(rows, experts, device=DEV)
    kn.moe_route(wide, route, top, scoring="softmax_chosen")
    got, want = route.cpu().double(), pt.route(z.double(), top)
    assert bool(((got >= 0).sum(1) == top).all())
    assert float((got.clamp(min=0) - want).abs().max()) < 1e-6
    assert (got[3] >= 0).nonzero().flatten().tolist() == list(range(top))
    for r in range(rows):
        assert set((got[r] >= 0).nonzero().flatten().tolist()) == set(sorted(range(experts), key=lambda e: (-float(z[r, e]), e))[:top])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,ff,shared", [(6, 24, 16), (3, 13, 0), (2, 7, 5), (1, 128, 0), (8, 80, 112), (4, 512, 1024)])
def test_activations_of_experts_without_a_gate(kn, experts, ff, shared, dtype):
    rows = 19
    u, z = rnd(rows, experts * ff + shared, seed=1), rnd(rows, experts, seed=2)
    route = pt.route(z.double(), max(1, experts // 2)).float()
    route[route == 0] = -1.0
    w = torch.cat([route.clamp(min=0).repeat_interleave(ff, 1), torch.ones(rows, shared)], 1)
    want = pt.relu_squared(u.double()) * w.double()
    out = torch.full((rows, experts * ff + shared), 9.0, dtype=dtype, device=DEV)
    kn.moe_act(dev(u), dev(route), out, experts, ff, "relu2", shared=shared)
    assert tc.err(out, want) < (1e-6 if dtype == torch.float32 else 5e-3)
    assert bool((out.cpu()[want == 0] == 0).all())
    plain = torch.zeros_like(out)
    kn.activation(dev(u), plain, "relu2")
    assert tc.err(plain, pt.relu_squared(u.double())) < (1e-6 if dtype == torch.float32 else 5e-3)


@pytest.mark.parametrize("gate", ["silu", "sigmoid"])
@pytest.mark.parametrize("n,group,weighted", [(256, 256, True), (192, 32, False), (2048, 2048, True), (63, 9, False), (1040, 1040, True),
                                              (2048, 256, False), (51, 51, True), (4096, 4096, True), (24, 1, False), (640, 640, False)])
def test_norm_and_gate_of_the_heads(kn, n, group, weighted, gate):
    rows, eps = 33, 1e-3
    y, z, w = rnd(rows, n, seed=1), rnd(rows, n, seed=2), rnd(n, seed=3, mean=1.0, std=0.3) if weighted else None
    y[4] *= 1e-3
    act = pt.silu if gate == "silu" else pt.sigmoid
    want = pt.rms(y.double().reshape(rows, -1, group), eps).reshape(rows, n) * (1.0 if w is None else w.double()) * act(z.double())
    wide = dev(torch.cat([rnd(rows, 4, seed=5), z], 1))[:, 4:]
    for dtype in (torch.float32, torch.bfloat16):
        out = torch.zeros((rows, n), dtype=dtype, device=DEV)
        kn.gated_rmsnorm(dev(y), wide, None if w is None else dev(w), eps, group, out, gate_first=False, gate=gate)
        assert tc.err(out, want) < (3e-6 if dtype == torch.float32 else 6e-3)


def test_sizes_that_do_not_fit_are_refused(kn):
    from longbow_quarrel_amd.kernels.hip import KernelLibraryError
    z = lambda *s: torch.zeros(*s, device=DEV)
    powers, state = z(2, 65), z(2, 2, 4, 8)
    args = lambda **kw: {**dict(q=z(3, 16), k=z(3, 16), v=z(3, 8), powers=powers, state=state, out=z(3, 8), heads=2, key_dim=8, value_dim=4,
                                k_scale=1.0, seq_slot=i32([0]), cu_rows=i32([0, 3]), batch=1), **kw}
    for more in (dict(k=z(3, 8)), dict(powers=z(2, 64)), dict(state=z(2, 2, 8, 4)), dict(activation="relu"), dict(out=z(2, 8)),
                 dict(cos_sin=z(3, 5, 2)), dict(batch=4), dict(state=z(2, 2, 4, 8).to(torch.bfloat16)),
                 dict(workspace=z(4), max_rows=64)):
        with pytest.raises(KernelLibraryError):
            kn.decay_scan(**args(**more))
    X, h, w = z(2, 3, 8), z(3, 8), z(8)
    for more in (dict(read=z(3), norm_weight=w, h=h), dict(norm_weight=z(7), h=h), dict(y=z(3, 8), mix=z(2, 2), out_weights=z(3), out=z(2, 3, 8)),
                 dict(y=z(3, 8), mix=z(3, 2), out_weights=z(2), out=z(2, 3, 8)), dict(), dict(norm_weight=w, h=z(3, 4))):
        with pytest.raises(KernelLibraryError):
            kn.streams_step(X, 2, **more)
    with pytest.raises(KernelLibraryError):
        kn.streams_step(z(17, 1, 8), 17, norm_weight=w, h=z(1, 8))
    cache = Paged(4, 1, 16, 16, torch.float32)
    with pytest.raises(KernelLibraryError):
        kn.sink_attention(z(4, 32), z(4, 32), 2, 1, 16, 16, i32(range(4)), i32([0] * 4), i32([0]), cache.table, cache.k, cache.v, 64, 1.0,
                          sink=False, chunk=5, keep_first=2)
    with pytest.raises(KernelLibraryError):
        kn.qkv_norm_store(z(4, 48), z(4, 32), 2, 1, 16, 16, 0.0, v_from_k=True, norm_qk="row", cos_sin=z(4, 4, 2))
    with pytest.raises(KernelLibraryError):
        kn.moe_route(z(3, 4), z(3, 4), 2, scoring="softmax_chosen", correction=z(4))
    with pytest.raises(KernelLibraryError):
        kn.moe_act(z(3, 9), z(3, 2), z(3, 9), 2, 4, "relu2")


# ---- the engine ------------------------------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    made = {}

    def get(name, dtype="float32", **kw):
        key = (name, dtype, tuple(sorted((k, str(v)) for k, v in kw.items())))
        if key not in made:
            made[key] = tc.Case(tmp_path_factory.mktemp("tukedra"), name, load, dtype=dtype,
                                rounding=dtype == "bfloat16", **kw)
        return made[key]

    return get


@pytest.mark.parametrize("name", tc.ALONE)
def test_a_mechanism_alone(cases, name):
    case = cases(name)
    tc.whole_and_token_by_token(case, TOL_F32, lengths=(1, 2, 9, 70))
    tc.portions(case, TOL_F32, n=140)


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_float32_under_every_cutting_and_batching(cases, name):
    case = cases(name)
    tc.whole_and_token_by_token(case, TOL_F32)
    tc.portions(case, TOL_F32)
    tc.unequal_batches(case, TOL_F32)
    tc.slots_and_blocks_used_again(case, TOL_F32)


@pytest.mark.parametrize("seed", range(1, 13))
def test_configurations_drawn_from_a_seed(cases, seed):
    """Other sizes, head counts, decays, chunks, rotations, streams, experts, layer orders and constants, in both dtypes."""
    case = cases(seed)
    t, u = tc.tokens(200, case.vocab, seed), tc.tokens(9, case.vocab, seed + 50)
    assert tc.err(case.run_cut(t, [150, 2, 1, 20]), case.want(t)) < TOL_F32
    eng = case.eng
    sa, sb = eng.new_sequence(), eng.new_sequence()
    out = eng.step([StepEntry(sa, u[:8], range(8)), StepEntry(sb, t[:130], range(130))])
    assert tc.err(out, torch.cat([case.want(u)[:8], case.want(t)[:130]])) < TOL_F32
    out = eng.step([StepEntry(sa, u[8:], [0]), StepEntry(sb, t[130:131], [0])])
    assert tc.err(out, torch.stack([case.want(u)[8], case.want(t)[130]])) < TOL_F32
    eng.release(sa)
    eng.release(sb)
    case.assert_idle()
    case16 = cases(seed, "bfloat16")
    tc.assert_close_bf16(case16.run_cut(t, [150, 2]), case16.want(t), case16.noise(t))


def test_prompts_sorted_by_expert(cases):
    """Prompts of 256 rows and more, alone and in a batch, go through the way that sorts a step's rows by expert."""
    for name in ("experts", "c"):
        case = cases(name)
        t = tc.tokens(320, case.vocab, 17)
        assert tc.err(case.run_cut(t, [310, 2]), case.want(t)) < TOL_F32
        assert tc.err(case.run_cut(t, [20, 290]), case.want(t)) < TOL_F32


def test_the_residual_stream_after_every_layer(cases):
    for name in ("a", "streams"):
        case = cases(name)
        got, want = case.layers(tc.tokens(37, case.vocab, 8))
        assert len(got) == len(want) == len(case.cfg["layers"])
        for i, (g, w) in enumerate(zip(got, want)):
            assert tc.err(g, w) < TOL_F32, f"after layer {i}"


@pytest.mark.parametrize("size", [1, 2, 63, 64, 65, 130])
def test_keys_just_inside_and_just_outside_the_chunk(cases, size):
    """Peaked attention within chunks of one token, of a cache block less one, a block, a block and one, and two blocks
    and two: the rows on either side of a chunk's edge, in a prompt, across portions and in decoding.  The plain
    implementation with chunks a token off differs by much from the first edge on."""
    case = cases(f"chunk-{size}", cfg=tc.chunked(size), sharp=4.0)
    n = max(2 * size + 10, 80)
    t = tc.tokens(n, case.vocab, 40 + size)
    tc.a_chunk_off_by_one_would_show(case, t)
    want = case.want(t)
    assert tc.err(case.run_cut(t, [n]), want) < TOL_F32
    assert tc.err(case.run_cut(t, [size, 1, 1, 2, size - 1 or 1, 3]), want) < TOL_F32
    assert tc.err(case.run_cut(t, [max(1, size - 1)]), want) < TOL_F32  # decoding across the chunk's edge
    case.assert_idle()
    case16 = cases(f"chunk-{size}", "bfloat16", cfg=tc.chunked(size), sharp=4.0)
    tc.assert_close_bf16(case16.run_cut(t, [max(1, size - 1)]), case16.want(t), case16.noise(t))


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_bfloat16_whole_in_portions_and_in_batches(cases, name):
    case = cases(name, "bfloat16")
    t = tc.tokens(150, case.vocab, 3)
    want, noise = case.want(t), case.noise(t)
    tc.assert_close_bf16(case.run_cut(t, [150]), want, noise)
    tc.assert_close_bf16(case.run_cut(t, [64, 1, 63, 2, 3]), want, noise)
    u = tc.tokens(70, case.vocab, 4)
    eng = case.eng
    sa, sb = eng.new_sequence(), eng.new_sequence()
    out = eng.step([StepEntry(sa, t[:100], range(100)), StepEntry(sb, u[:3], range(3))])
    tc.assert_close_bf16(out, torch.cat([want[:100], case.want(u)[:3]]), noise)
    got = []
    for i in range(20):
        got.append(eng.step([StepEntry(sb, [u[3 + i]], [0]), StepEntry(sa, [t[100 + i]], [0])]).clone())
    got = torch.cat(got)
    tc.assert_close_bf16(torch.cat([got[0::2], got[1::2]]), torch.cat([case.want(u)[3:23], want[100:120]]), noise)
    eng.release(sa)
    eng.release(sb)
    case.assert_idle()


def test_bfloat16_decoding_over_long_contexts(cases):
    """Single tokens over several hundred positions (chunks that are over, their blocks given back) against the same rows as
    parts of a prompt and against the plain implementation."""
    case = cases("c", "bfloat16")
    t, u = tc.tokens(640, case.vocab, 61), tc.tokens(330, case.vocab, 62)
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
    tc.assert_close_bf16(got, want, noise)
    tc.assert_close_bf16(got, whole.double(), noise)


@pytest.mark.parametrize("name", ["lightning", "retention"])
def test_a_slow_decay_keeps_old_tokens_in_the_state(cases, name):
    case = cases(f"{name}-slow", cfg=tc.slow(name))
    t = tc.tokens(700, case.vocab, 31)
    want = case.want(t)
    other = case.want([(t[0] + 1) % case.vocab] + t[1:260])
    assert tc.err(other[-1], want[259]) > 1e-3  # the first token still matters, chunks later
    assert tc.err(case.run_cut(t, [700]), want) < TOL_F32
    assert tc.err(case.run_cut(t[:260], [3, 64, 1, 2, 130]), want[:260]) < TOL_F32
    assert tc.err(case.run_cut(t, [100, 560, 2]), want) < TOL_F32


def test_the_first_tokens_start_from_nothing(cases):
    case = cases("a")
    eng = case.eng
    a, b = tc.tokens(150, case.vocab, 1), tc.tokens(6, case.vocab, 2)
    sa = eng.new_sequence()
    eng.step([StepEntry(sa, a, [])])
    eng.release(sa)
    for first in (1, 2, 3, 6):
        s = eng.new_sequence()
        assert s == sa
        out = eng.step([StepEntry(s, b[:first], range(first))])
        assert tc.err(out, case.want(b)[:first]) < TOL_F32
        if first < 6:
            out = eng.step([StepEntry(s, b[first:], range(6 - first))])
            assert tc.err(out, case.want(b)[first:]) < TOL_F32
        eng.release(s)
    case.assert_idle()


@pytest.mark.parametrize("name", ["a", "c"])
def test_long_decoding(cases, name):
    tc.long_decoding(cases(name), TOL_F32)


def test_float32_logits_do_not_depend_on_the_cutting_or_the_batch_by_more_than_rounding(cases):
    case = cases("c")
    t, u = tc.tokens(140, case.vocab, 7), tc.tokens(30, case.vocab, 8)
    whole = case.run_cut(t, [140]).double()
    assert tc.err(case.run_cut(t, [64, 1, 2, 70]), whole) < 1e-5 and tc.err(case.run_cut(t, [100]), whole) < 1e-5
    eng = case.eng
    sa, sb = eng.new_sequence(), eng.new_sequence()
    out = eng.step([StepEntry(sb, u, []), StepEntry(sa, t[:90], range(90))])
    assert tc.err(out, whole[:90]) < 1e-5
    out = eng.step([StepEntry(sa, [t[90]], [0]), StepEntry(sb, [5], [])])
    assert tc.err(out[0], whole[90]) < 1e-5
    eng.release(sa)
    eng.release(sb)


@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation_through_the_entry_point(cases, graphs):
    case = cases("a")
    reqs, wants = tc.greedy(case, n_new=12, prompts=5)
    res = lq.generate(case.eng, reqs, max_new_tokens=12, max_batch=3, stop_ids=[], use_graphs=graphs)
    assert res.tokens == wants
    case.assert_idle()


def test_generation_in_bfloat16_captured_and_direct_steps_agree_and_stop_ids_end_requests(cases):
    case = cases("c", "bfloat16")
    assert case.eng.graph_safe
    reqs = [tc.tokens(n, case.vocab, 40 + n) for n in (3, 70, 9, 1, 130, 20)]
    direct = lq.generate(case.eng, reqs, max_new_tokens=40, max_batch=4, stop_ids=[], use_graphs=False)
    stop = direct.tokens[1][7]
    a = lq.generate(case.eng, reqs, max_new_tokens=40, max_batch=4, stop_ids=[stop], use_graphs=False)
    b = lq.generate(case.eng, reqs, max_new_tokens=40, max_batch=4, stop_ids=[stop], use_graphs=True)
    assert a.tokens == b.tokens and a.finish == b.finish and "stop" in a.finish
    case.assert_idle()


def test_command_line_and_trace_replay(cases, tmp_path):
    case = cases("b")
    reqs, wants = tc.greedy(case, n_new=5, prompts=1)
    out = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "quarrel"), "-model", case.folder, "-dtype", "float32",
                          "-prompt", " ".join(map(str, reqs[0])), "-n", "5", "-temp", "0", "-penalty", "1"],
                         capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    assert "Architecture: Tukedra" in out.stdout
    assert out.stdout.strip().splitlines()[-1].split() == [str(t) for t in wants[0]]
    a, b = tc.tokens(70, case.vocab, 1), tc.tokens(9, case.vocab, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:66], "want": [0, 65]}, {"id": "b", "tokens": b[:7], "want": [6]}],
              "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [a[66]], "want": [0]}, {"id": "b", "tokens": [b[7]], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": [a[67]], "want": []}, {"id": "b", "tokens": [b[8]], "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[68:], "want": [1]}], "end": ["a"]}]
    for dtype, check in (("float32", lambda g, w: tc.err(g, w) < TOL_F32), ("bfloat16", lambda g, w: tc.err(g, w) < 0.1)):
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
