"""The Puzonex design through the engine's own code (registry, loader, cache groups, step function, generation
loop) on the CPU, over the torch stand-in for the kernels, against the plain implementation.  The GPU tests
repeat every scenario with the HIP kernels; these catch faults of the parts, the cache and the batching."""
import copy
import math

import pytest
import torch

import longbow_quarrel_amd as lq
import plain_puzonex as pp
import puzonex_cases as pc
from cpu_kernels import CpuKernels
from longbow_quarrel_amd.engine import StepEntry
from longbow_quarrel_amd.parts.base import KVNeed, MultiNeed, StateNeed
from longbow_quarrel_amd.parts.sink_attention import distance_rows

# A sublayer's result is normed to unit size, a memory's answer twice: where one nearly vanishes at a token, its 32-bit
# rounding is blown up with it (the plain implementation run in 32-bit is off by up to 5e-5 at single rows of these
# cases, 1e-6 at most rows).  A fault moves the rows it touches by 1e-3 and more.
TOL = 1e-4
F = torch.float64


def load(folder, dtype, max_tokens):
    return lq.load_engine(folder, dtype=dtype, max_tokens=max_tokens, device="cpu", kernels=CpuKernels(),
                          max_slots=8, max_sequence_tokens=max_tokens)


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    made = {}

    def get(name, **kw):
        key = (name, tuple(sorted((k, str(v)) for k, v in kw.items())))
        if key not in made:
            made[key] = pc.Case(tmp_path_factory.mktemp("puzonex"), name, load, **kw)
        return made[key]

    return get


# ---- configuration, registry, tensors, cache needs ----------------------------------------------------------------
def test_configuration_reads_every_size_and_writes_the_same_keys_back():
    for cfg in pc.CONFIGS.values():
        assert lq.PuzonexConfig.from_dict(cfg).to_dict() == cfg
    from longbow_quarrel_amd.model import DecoderModel
    from longbow_quarrel_amd.registry import config_from_dict, spec_from_config

    config = config_from_dict(pc.CFG_A)
    assert isinstance(config, lq.PuzonexConfig)
    model = DecoderModel(spec_from_config(config))
    assert [r.layer for r in model.spec.schedule] == list(range(6))
    specs = {s.name: s for s in model.tensor_specs()}
    shapes = {n: tuple(s.shape) for n, s in specs.items()}
    # the left side has no values of its own and no sink; the attention layer no output bias, gate or temperature
    assert {"embed", "head", "final.norm", "l0.norm1", "l0.norm2", "l0.mlp.gate"} <= set(specs)
    assert not {"l0.mix.left.v", "l0.mix.left.v.b", "l0.mix.left.sink", "l0.mix.left.r1", "l1.mix.o.b", "l1.mix.g",
                "l1.mix.temp", "l1.mix.rel"} & set(specs)
    assert shapes["l0.mix.left.q.b"] == (144,) and shapes["l0.mix.left.k.b"] == (48,) and shapes["l0.mix.left.o.b"] == (80,)
    assert shapes["l0.mix.left.q.norm"] == (144,) and shapes["l0.mix.left.k.norm"] == (48,)  # all heads together
    assert shapes["l1.mix.q.norm"] == (16,) and shapes["l1.mix.k.norm"] == (16,)  # shared by the heads
    assert shapes["l0.mix.left.rel"] == (12, 6) and shapes["l0.mix.left.g"] == (144, 80) and shapes["l0.mix.left.temp"] == (6,)
    assert shapes["l1.mix.v.b"] == (80,) and shapes["l1.mix.r2"] == (2,) and shapes["l1.mix.sink"] == (2,)
    assert shapes["l0.mix.right.norm"] == (60,) and shapes["l0.mix.right.i"] == (3, 80) and shapes["l0.mix.right.f.b"] == (3,)
    assert shapes["l2.mix.in"] == (112, 80) and shapes["l2.mix.x"] == (30, 56) and shapes["l2.mix.dt"] == (56, 6)
    assert shapes["l2.mix.A_log"] == (56, 12) and shapes["l2.mix.conv"] == (56, 4) and shapes["l2.mix.D"] == (56,)
    assert specs["l2.norm2"].optional and not specs["l1.norm2"].optional and "l2.mlp.up" not in specs
    needs = model.cache_needs()
    assert needs[1] == KVNeed(2, 16, 70, 40) and needs[3] == KVNeed(2, 40, 0, 16)
    assert needs[2] == MultiNeed((StateNeed((56, 12), torch.float32), StateNeed((3, 56), torch.float32)))
    assert needs[0] == MultiNeed((KVNeed(2, 24, 20, 24), MultiNeed((StateNeed((3, 21, 12), torch.float32),
                                                                    StateNeed((3,), torch.float32)))))


@pytest.mark.parametrize("key,value,text", [
    (("layers", 0, "type"), "delta", "layers[0].type"),
    (("layers", 0, "mixer", "left", "kv_heads"), 4, "kv_heads"),
    (("layers", 0, "mixer", "left", "scale"), None, "left.scale"),
    (("layers", 0, "mixer", "left", "softcap"), -1.0, "left.softcap"),
    (("layers", 0, "mixer", "left", "mask", "size"), 0, "mask.size"),
    (("layers", 0, "mixer", "left", "bias_max"), None, "left.bias_max"),
    (("layers", 0, "mixer", "left", "bias_max"), 6.0, "left.bias_max"),
    (("layers", 0, "mixer", "left", "vdim"), 8, "left.vdim"),
    (("layers", 0, "mixer", "right", "gate_cap"), 0.0, "right.gate_cap"),
    (("layers", 0, "mixer", "right", "heads"), None, "right.heads"),
    (("layers", 1, "mixer", "softcap"), "wide", "mixer.softcap"),
    (("layers", 2, "mixer", "state"), 0, "mixer.state"),
    (("layers", 2, "mixer", "dt_rank"), None, "mixer.dt_rank"),
    (("layers", 1, "mlp", "kind"), "moe", "mlp.kind"),
    (("layers", 1, "mlp", "ff"), None, "mlp.ff"),
    (("norm", "eps"), "tiny", "norm.eps"),
    (("width",), None, "width"),
])
def test_configuration_errors_name_their_key(key, value, text):
    cfg = copy.deepcopy(pc.CFG_A)
    d = cfg
    for k in key[:-1]:
        d = d[k]
    d[key[-1]] = value
    with pytest.raises(lq.ConfigError) as e:
        lq.PuzonexConfig.from_dict(cfg)
    assert text in str(e.value)


def test_keys_that_a_configuration_leaves_out():
    cfg = copy.deepcopy(pc.CFG_LOG)
    m = cfg["layers"][0]["mixer"]
    del m["kv_heads"], m["vdim"], m["mask"], m["softcap"]
    a = lq.PuzonexConfig.from_dict(cfg).layers[0].attention
    assert (a.kv_heads, a.vdim, a.window, a.softcap) == (4, 16, 0, 0.0)


def test_the_rows_of_the_bias_table_come_from_the_file(tmp_path):
    cfg = copy.deepcopy(pc.CFG_A)
    weights = pc.make_weights(cfg, 5)
    for layer in cfg["layers"]:
        if layer["type"] == "parallel":
            del layer["mixer"]["left"]["bias_rows"]
    eng = load(pc.write_folder(tmp_path, cfg, weights, "norows"), "float32", 256)
    assert [x.left.bias_rows for x in eng.config.layers if x.left] == [12, 8]
    t = pc.tokens(30, cfg["vocab"], 1)
    got = eng.step([StepEntry(eng.new_sequence(), t, range(30))])
    assert pc.err(got, pp.forward(cfg, weights, t)) < TOL
    with pytest.raises(lq.ConfigError) as e:
        lq.random_engine(lq.PuzonexConfig.from_dict(cfg), 1, device="cpu", kernels=CpuKernels())
    assert "bias_rows" in str(e.value)


def test_the_norm_of_an_absent_feed_forward_may_be_in_the_file(tmp_path):
    cfg = copy.deepcopy(pc.CFG_SCAN)
    weights = pc.make_weights(cfg, 5)
    weights.pop("l0.norm2", None)
    t = pc.tokens(12, cfg["vocab"], 1)
    got = []
    for name, more in (("without", {}), ("with", {"l0.norm2": torch.full((cfg["width"],), 3.0)})):
        eng = load(pc.write_folder(tmp_path, cfg, {**weights, **more}, name), "float32", 256)
        got.append(eng.step([StepEntry(eng.new_sequence(), t, range(12))]))
    assert torch.equal(got[0], got[1]) and pc.err(got[0], pp.forward(cfg, weights, t)) < TOL


def test_missing_and_unexpected_tensors_are_named(tmp_path):
    cfg = copy.deepcopy(pc.CFG_TABLE)
    weights = pc.make_weights(cfg, 5)
    weights["l0.mix.left.v"] = weights["l0.mix.left.k"].clone()  # the values are the keys
    del weights["l0.mix.left.temp"], weights["l0.mix.right.f.b"]
    with pytest.raises(lq.WeightError) as e:
        load(pc.write_folder(tmp_path, cfg, weights, "bad"), "float32", 256)
    assert e.value.missing == ["l0.mix.left.temp", "l0.mix.right.f.b"] and e.value.unexpected == ["l0.mix.left.v"]


def test_mechanisms_that_do_not_go_together_are_refused():
    from longbow_quarrel_amd.parts.sink_attention import SinkWindowAttention
    sizes = dict(width=8, heads=2, kv_heads=1, key_dim=4, value_dim=4, scale=1.0, prefix="x")
    for more in (dict(qk_norm="row", rotary={"dims": 4, "base": 10.0}),
                 dict(qkv_bias=True, qk_norm_eps=1e-6), dict(entry_gate=True, head_gate=True),
                 dict(qk_norm="rows"), dict(values_from_keys=True, key_dim=4, value_dim=8), dict(softcap=-1.0)):
        with pytest.raises(ValueError):
            SinkWindowAttention(**{**sizes, **more})
    for rows, most in ((1, 5.0), (8, 4.0), (8, 3.0)):
        with pytest.raises(ValueError):
            distance_rows(rows, most)


# ---- the plain implementation's own mechanisms against hand-made cases ---------------------------------------------
def test_plain_sinusoids_are_sine_and_cosine_of_neighbouring_entries():
    s = pp.sinusoids(4, 5)  # an odd width ends with a sine
    assert s[0].tolist() == [0.0, 1.0, 0.0, 1.0, 0.0]
    f = [1.0, 10000.0 ** -0.4, 10000.0 ** -0.8]
    assert torch.allclose(s[3], torch.tensor([math.sin(3 * f[0]), math.cos(3 * f[0]), math.sin(3 * f[1]),
                                              math.cos(3 * f[1]), math.sin(3 * f[2])], dtype=F))


def test_plain_buckets_and_the_librarys():
    # 8 rows up to 16: distances 0 to 3 one by one, then ln(n / 4) / ln 4 * 4 = 2 log2(n / 4) steps: 4 5 at 4, from
    # 4 sqrt(2) = 5.7 row 5, from 8 row 6, from 11.3 row 7, and row 7 for all beyond
    want = [0, 1, 2, 3, 4, 4, 5, 5, 6, 6, 6, 6, 7, 7, 7, 7, 7, 7, 7]
    assert [pp.bucket(n, 8, 16.0) for n in range(19)] == want
    assert pp.bucket(10 ** 6, 8, 16.0) == 7
    for rows, most in ((8, 16.0), (10, 30.0), (5, 7.5), (2, 3.0), (3, 51.0), (32, 128.0), (31, 415.0), (12, 60.0), (24, 96.0)):
        full = distance_rows(rows, most)
        assert full[-1] == rows - 1 and full[:-1].count(rows - 1) == 0  # it ends with the first distance of the last row
        assert full == [pp.bucket(n, rows, most) for n in range(len(full))]
        assert all(pp.bucket(n, rows, most) == rows - 1 for n in range(len(full), len(full) + 50))
        assert distance_rows(rows, most, 3) == full[:3]
    # an exact step counts as reached: ln 2 / ln 8 * 12 is 4
    assert pp.bucket(24, 24, 96.0) == 16 and pp.bucket(23, 24, 96.0) == 15 and pp.bucket(48, 24, 96.0) == 20


def test_plain_biases_by_distance():
    b = pp.log_bias(3, 0.5, 2.0)
    assert float(b[2, 2]) == 0.0 and float(b[2, 1]) == pytest.approx(-0.5 * math.log(3.0))
    assert float(b[2, 0]) == pytest.approx(-0.5 * math.log(5.0))
    t = pp.table_bias(5, torch.tensor([10.0, 20.0, 30.0, 40.0], dtype=F), 8.0)  # half 2: rows 0 1 2 2 3
    assert t[4].tolist() == [40.0, 30.0, 30.0, 20.0, 10.0]


def test_plain_cap_and_gelu():
    s = torch.tensor([0.01, -3.0, 100.0], dtype=F)
    assert torch.allclose(pp.soft_cap(s, 2.0), torch.tensor([2 * math.tanh(0.005), 2 * math.tanh(-1.5), 2.0], dtype=F))
    assert pp.soft_cap(s, None) is s and pp.soft_cap(s, 0.0) is s
    z = torch.tensor([1.0], dtype=F)
    tanh_form = 0.5 * (1 + math.tanh(math.sqrt(2 / math.pi) * 1.044715))
    assert float(pp.gelu_tanh(z)) == pytest.approx(tanh_form, rel=1e-14)
    assert abs(tanh_form - 0.5 * (1 + math.erf(math.sqrt(0.5)))) > 1e-4


def test_plain_softmax_with_a_sink():
    score = torch.tensor([[0.0, math.log(3.0), 50.0]], dtype=F)
    seen = torch.tensor([[True, True, False]])
    assert torch.allclose(pp.softmax_rows(score, seen, math.log(4.0)), torch.tensor([[1 / 8, 3 / 8, 0.0]], dtype=F))
    assert torch.allclose(pp.softmax_rows(score, seen), torch.tensor([[1 / 4, 3 / 4, 0.0]], dtype=F))


def test_plain_attention_norms_values_and_takes_the_bias_off_after_the_cap():
    """One head, keys of one entry, two value channels.  With one entry a normed query or key is its sign times the
    weight.  At token 1: scores 2 * 3 * 0.5 = 3 against both keys, capped to 2 tanh(1.5) for both, then 0.5 ln 3 off for
    the key one back; the sink's ln 2 joins the denominator."""
    m = {"heads": 1, "kv_heads": 1, "dim": 1, "vdim": 2, "scale": 0.5, "softcap": 2.0, "mask": {"size": 5}}
    w = {"q": [[1.0, 0, 0]], "q.b": [1.0], "k": [[1.0, 0, 0]], "k.b": [0.5], "v": [[0, 3.0, 0], [0, 0, 4.0]], "v.b": [0.0, 0.0],
         "q.norm": [2.0], "k.norm": [3.0], "r1": [0.5], "r2": [2.0], "sink": [math.log(2.0)], "o": [[1.0, 0], [0, 1.0]]}
    w = {"x." + k: torch.tensor(v, dtype=F) for k, v in w.items()}
    h = torch.tensor([[1.0, 1, 0], [1.0, 0, 1]], dtype=F)
    y = pp.attention(h, m, w, "x", 0.0, False)
    cap = 2 * math.tanh(1.5)
    e0, e1 = math.exp(cap - 0.5 * math.log(3.0)), math.exp(cap)
    root2 = math.sqrt(2.0)  # a value with one channel set, divided by its root mean square
    assert torch.allclose(y[1], torch.tensor([e0 / (e0 + e1 + 2) * root2, e1 / (e0 + e1 + 2) * root2], dtype=F))
    assert torch.allclose(y[0], torch.tensor([e1 / (e1 + 2) * root2, 0.0], dtype=F))


def test_plain_key_value_attention_reads_the_keys_before_their_norm():
    """Two heads on two key heads of one entry; the norm over both heads together keeps their sizes apart.  One token:
    every weight is one, so the result is the keys as projected, with their bias, gated, plus the output's bias."""
    m = {"heads": 2, "kv_heads": 2, "dim": 1, "vdim": 1, "scale": 1.0, "bias_max": 9.0, "mask": {"size": 4}}
    w = {"q": [[1.0], [2.0]], "q.b": [0.0, 0.0], "k": [[3.0], [5.0]], "k.b": [1.0, -1.0], "q.norm": [1.0, 1.0],
         "k.norm": [7.0, 7.0], "temp": [1.0, 1.0], "rel": [[0.0, 0.0]] * 4, "g": [[0.0], [math.log(3.0)]],
         "o": [[1.0, 0], [0, 1.0]], "o.b": [100.0, 200.0]}
    w = {"x." + k: torch.tensor(v, dtype=F) for k, v in w.items()}
    y = pp.key_value_attention(torch.ones(1, 1, dtype=F), m, w, "x", 0.0, False)
    assert torch.allclose(y, torch.tensor([[4.0 * 0.5 + 100, 4.0 * 0.75 + 200]], dtype=F))
    # two tokens, temperatures: q of head 1 normed over both heads is 2 / sqrt(2.5), k likewise; head 0's temperature of
    # zero leaves the table's bias alone
    w["x.temp"] = torch.tensor([0.0, 1.0], dtype=F)
    w["x.rel"] = torch.tensor([[math.log(3.0), 0.0], [0.0, 0.0], [0.0, 0.0], [0.0, 0.0]], dtype=F)
    w["x.g"] = torch.zeros(2, 1, dtype=F)
    h = torch.tensor([[1.0], [2.0]], dtype=F)
    y = pp.key_value_attention(h, m, w, "x", 0.0, False)
    assert float(y[1, 0]) == pytest.approx(0.5 * (1 / 4 * 4.0 + 3 / 4 * 7.0) + 100)
    k = [[4.0, 4.0], [7.0, 9.0]]
    kn = [7 * r[1] / math.sqrt((r[0] ** 2 + r[1] ** 2) / 2) for r in k]
    qn = 4 / math.sqrt((2 ** 2 + 4 ** 2) / 2)
    e = [math.exp(qn * v) for v in kn]
    assert float(y[1, 1]) == pytest.approx(0.5 * (e[0] * 4.0 + e[1] * 9.0) / sum(e) + 200)


def test_plain_selective_scan_by_hand():
    """Two channels with steps of their own and two state entries with rates of their own."""
    A = torch.tensor([[-1.0, -2.0], [-0.5, -3.0]], dtype=F)
    x, dt = torch.tensor([[1.0, 2.0], [3.0, 4.0]], dtype=F), torch.tensor([[0.1, 0.2], [0.3, 0.4]], dtype=F)
    B, C = torch.tensor([[1.0, 10.0], [2.0, 20.0]], dtype=F), torch.tensor([[1.0, 1.0], [1.0, 0.5]], dtype=F)
    D = torch.tensor([0.0, 7.0], dtype=F)
    y = pp.selective_scan(x, dt, B, C, A, D)
    assert float(y[0, 0]) == pytest.approx(0.1 * 1 * 11) and float(y[0, 1]) == pytest.approx(0.2 * 2 * 11 + 14)
    s0 = math.exp(-0.5 * 0.4) * 0.4 * 1 + 0.4 * 4 * 2
    s1 = math.exp(-3.0 * 0.4) * 0.4 * 10 + 0.4 * 4 * 20
    assert float(y[1, 1]) == pytest.approx(s0 + 0.5 * s1 + 28)


def test_plain_matrix_memory_starts_from_a_maximum_of_zero():
    """With gates far below zero the maximum stays where the forget gates leave it (from zero down) or at the input
    gate, and exp(-m) bounds the denominator."""
    q, k, v = torch.tensor([[2.0]], dtype=F), torch.tensor([[3.0]], dtype=F), torch.tensor([[5.0]], dtype=F)
    i, f = torch.tensor([-4.0], dtype=F), torch.tensor([-1.0], dtype=F)
    # m = max(-1 + 0, -4) = -1: S = e^(-3) 15, n = e^(-3) 3; the denominator is max(|6 e^-3|, e^1)
    assert float(pp.matrix_memory(q, k, v, i, f)) == pytest.approx(30 * math.exp(-3) / (math.e + 1e-6))
    i = torch.tensor([2.0], dtype=F)  # m = 2: S = 15, n = 3, max(6, e^-2)
    assert float(pp.matrix_memory(q, k, v, i, f)) == pytest.approx(30 / (6 + 1e-6))
    # against the recurrence without a maximum (its own gates, exp(-m) in the place of the bound scaled alike)
    g = torch.Generator().manual_seed(1)
    T = 12
    q, k, v = (torch.randn(T, n, generator=g, dtype=F) for n in (4, 4, 3))
    i, f = torch.randn(T, generator=g, dtype=F), pp.log_sigmoid(torch.randn(T, generator=g, dtype=F))
    S, n = torch.zeros(4, 3, dtype=F), torch.zeros(4, dtype=F)
    want = []
    for t in range(T):
        S = math.exp(f[t]) * S + math.exp(i[t]) * torch.outer(k[t], v[t])
        n = math.exp(f[t]) * n + math.exp(i[t]) * k[t]
        want.append((S.T @ q[t]) / max(abs(float(n @ q[t])), 1.0))
    assert pc.err(pp.matrix_memory(q, k, v, i, f), torch.stack(want)) < 1e-5  # (but for the 1e-6 under the bar)


def test_plain_convolution_ends_with_the_current_token():
    x = torch.tensor([[1.0], [10.0], [100.0]], dtype=F)
    y = pp.short_conv(x, torch.tensor([[2.0, 3.0]], dtype=F), torch.tensor([0.5], dtype=F))
    assert torch.allclose(y, pp.silu(torch.tensor([[3.5], [32.5], [320.5]], dtype=F)))


# ---- every mechanism alone, and all of them, through the engine ------------------------------------------------------
@pytest.mark.parametrize("name", ["log", "table", "memory", "scan", "dense"])
def test_a_mechanism_alone(cases, name):
    case = cases(name)
    pc.whole_and_token_by_token(case, TOL, lengths=(1, 2, 9, 70))
    pc.portions(case, TOL, n=140)


@pytest.mark.parametrize("name", ["a", "b"])
def test_whole_prompts_against_token_by_token_decoding(cases, name):
    pc.whole_and_token_by_token(cases(name), TOL)


@pytest.mark.parametrize("name", ["a", "b"])
def test_portions_of_several_sizes_down_to_two_tokens(cases, name):
    pc.portions(cases(name), TOL)


@pytest.mark.parametrize("name", ["a", "b"])
def test_batches_of_unequal_requests_against_each_alone(cases, name):
    pc.unequal_batches(cases(name), TOL)


@pytest.mark.parametrize("name", ["a", "scan"])
def test_slots_and_blocks_are_freed_and_used_again(cases, name):
    pc.slots_and_blocks_used_again(cases(name), TOL)


@pytest.mark.parametrize("seed", [1, 2, 3, 4, 5, 6, 7, 8])
def test_configurations_drawn_from_a_seed(cases, seed):
    case = cases(seed)
    assert lq.PuzonexConfig.from_dict(case.cfg).to_dict() == case.cfg
    t, u = pc.tokens(70, case.vocab, seed), pc.tokens(9, case.vocab, seed + 50)
    assert pc.err(case.run_cut(t, [40, 2, 1, 20]), case.want(t)) < TOL
    eng = case.eng
    sa, sb = eng.new_sequence(), eng.new_sequence()
    out = eng.step([StepEntry(sa, u[:8], range(8)), StepEntry(sb, t[:66], range(66))])
    assert pc.err(out, torch.cat([case.want(u)[:8], case.want(t)[:66]])) < TOL
    out = eng.step([StepEntry(sa, u[8:], [0]), StepEntry(sb, t[66:67], [0])])
    assert pc.err(out, torch.stack([case.want(u)[8], case.want(t)[66]])) < TOL
    eng.release(sa)
    eng.release(sb)
    case.assert_idle()


def test_the_residual_stream_after_every_layer(cases):
    case = cases("a")
    got, want = case.layers(pc.tokens(37, case.vocab, 8))
    assert len(got) == len(want) == 6
    for i, (g, w) in enumerate(zip(got, want)):
        assert pc.err(g, w) < TOL, f"after layer {i}"


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
    assert pc.err(case.run_cut(t, [n]), want) < TOL
    assert pc.err(case.run_cut(t, [window, 1, 1, 2, window - 1 or 1, 3]), want) < TOL
    assert pc.err(case.run_cut(t, [max(1, window - 1)]), want) < TOL  # decoding across the window's edge
    case.assert_idle()


@pytest.mark.parametrize("name,leaves", [
    ("log", {"sink": -30.0}), ("log", {"r1": 0.0}), ("log", {"r2": 0.0}), ("table", {"rel": 0.0}), ("table", {"temp": 1.0}),
    ("table", {"g": 0.0}), ("memory", {"i": 0.0}), ("memory", {"f": 0.0}), ("scan", {"D": 0.0}), ("scan", {"A_log": 0.0}),
])
def test_every_learned_number_matters(cases, name, leaves):
    """With one of them flattened in the oracle the result differs by much, so the comparisons here see it."""
    case = cases(name)
    t = pc.tokens(60, case.vocab, 9)
    assert pc.err(pp.forward(case.cfg, pc.flattened(case.weights, **leaves), t), case.want(t)) > 1e-3
    assert pc.err(case.run_cut(t, [50, 2]), case.want(t)) < TOL


@pytest.mark.parametrize("name", ["log", "table"])
def test_the_cap_and_the_far_end_of_a_bias(cases, name):
    """Attention without a window over hundreds of tokens: the cap binds, the logarithm keeps falling, the table's last
    row serves every far distance."""
    cfg = copy.deepcopy(pc.CONFIGS[name])
    del pc.attention_of(cfg)["mask"]
    case = cases(f"{name}-open", cfg=cfg, sharp=3.0)
    t = pc.tokens(150, case.vocab, 6)
    loose = copy.deepcopy(case.cfg)
    pc.attention_of(loose)["softcap"] = 1e9
    assert pc.err(pp.forward(loose, case.weights, t), case.want(t)) > 1e-3
    assert pc.err(case.run_cut(t, [100, 3]), case.want(t)) < TOL


@pytest.mark.parametrize("name", ["scan", "memory"])
def test_a_slow_decay_keeps_old_tokens_in_the_state(cases, name):
    """Decays close to one: the first tokens still weigh in the state after hundreds of steps, far beyond every
    window, so a state that is lost, reset or carried to the wrong slot shows far from where it happened."""
    case = cases(f"{name}-slow", cfg=pc.long_memory(name), memory=5.0)
    t = pc.tokens(260, case.vocab, 31)
    want = case.want(t)
    other = case.want([(t[0] + 1) % case.vocab] + t[1:])
    assert pc.err(other[-1], want[-1]) > 1e-3  # the first token still matters at the end
    assert pc.err(case.run_cut(t, [260]), want) < TOL
    assert pc.err(case.run_cut(t, [3, 64, 1, 2, 130]), want) < TOL


def test_the_first_tokens_see_zeros_ahead_of_the_sequence(cases):
    """The short convolutions read zeros before the first token, the states and the running maximum start at zero and the
    windows are not yet full, also in a slot that another sequence has left, and whether the first step brings one
    token or several."""
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
        assert pc.err(out, case.want(b)[:first]) < TOL
        if first < 6:
            out = eng.step([StepEntry(s, b[first:], range(6 - first))])
            assert pc.err(out, case.want(b)[first:]) < TOL
        eng.release(s)
    case.assert_idle()


def test_windowed_groups_give_their_blocks_back(cases):
    case = cases("log")  # one layer, a window of 40: never more than two blocks a sequence
    eng = case.eng
    s = eng.new_sequence()
    t = pc.tokens(400, case.vocab, 3)
    eng.step([StepEntry(s, t[:300], [])])
    for i in range(300, 400):
        eng.step([StepEntry(s, t[i : i + 1], [])])
    assert all(g.blocks.taken_count <= 2 for g in eng.cache.kv_groups)
    out = eng.step([StepEntry(s, [5], [0])])
    assert pc.err(out[0], case.want(t + [5])[-1]) < TOL
    eng.release(s)
    case.assert_idle()


def test_the_branches_of_mixers_side_by_side_with_and_without_the_kernel_that_joins_them(cases, monkeypatch):
    """A kernel object that does not take the joined pass gives the same logits through the mean and the norm apart."""
    case = cases("table")
    t = pc.tokens(40, case.vocab, 2)
    joined = case.run_cut(t, [30, 2])
    monkeypatch.setattr(CpuKernels, "mean_residual_takes", lambda self, width: False)
    assert pc.err(case.run_cut(t, [30, 2]), joined) < 1e-6


def test_long_decoding(cases):
    pc.long_decoding(cases("a"), TOL)


def test_greedy_generation_through_the_generation_loop(cases):
    case = cases("a")
    reqs, wants = pc.greedy(case)
    result = lq.generate(case.eng, reqs, max_new_tokens=10)
    assert result.tokens == wants
    case.assert_idle()


def test_bfloat16_run_rounds_where_the_plain_implementation_does(tmp_path_factory):
    case = pc.Case(tmp_path_factory.mktemp("puzonex16"), "a", load, dtype="bfloat16", rounding=True)
    t = pc.tokens(80, case.vocab, 3)
    pc.assert_close_bf16(case.run_cut(t, [50, 2]), case.want(t), case.noise(t))
