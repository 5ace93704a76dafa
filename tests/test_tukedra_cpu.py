"""The Tukedra design through the engine's own code (registry, loader, cache groups, step function, generation
loop) on the CPU, over the torch stand-in for the kernels, against the plain implementation.  The GPU tests
repeat every scenario with the HIP kernels; these catch faults of the parts, the cache and the batching."""
import copy
import math

import pytest
import torch

import longbow_quarrel_amd as lq
import plain_tukedra as pt
import tukedra_cases as tc
from cpu_kernels import CpuKernels
from longbow_quarrel_amd.engine import StepEntry
from longbow_quarrel_amd.parts.base import KVNeed, PartSpec, StateNeed, build_part, BLOCKS, MIXERS, FEED_FORWARDS

TOL = 5e-5
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
            made[key] = tc.Case(tmp_path_factory.mktemp("tukedra"), name, load, **kw)
        return made[key]

    return get


# ---- configuration, registry, tensors, cache needs ----------------------------------------------------------------
def test_configuration_reads_every_size_and_writes_the_same_keys_back():
    for cfg in tc.CONFIGS.values():
        assert lq.TukedraConfig.from_dict(cfg).to_dict() == cfg
    from longbow_quarrel_amd.model import DecoderModel
    from longbow_quarrel_amd.registry import config_from_dict, spec_from_config

    config = config_from_dict(tc.CFG_A)
    assert isinstance(config, lq.TukedraConfig)
    model = DecoderModel(spec_from_config(config))
    assert model.graph_safe and [r.layer for r in model.spec.schedule] == list(range(6))
    specs = {s.name: s for s in model.tensor_specs()}
    shapes = {n: tuple(s.shape) for n, s in specs.items()}
    assert {"embed", "head", "final.norm", "l0.norm1", "l0.norm2", "l0.mlp.gate", "l0.hc1.in", "l0.hc2.mix"} <= set(specs)
    # retention norms without a weight, attention has no values of its own and no biases but those of q and k
    assert not {"l0.mix.norm", "l1.mix.v", "l1.mix.v.b", "l1.mix.o.b", "l1.mix.q.norm", "l0.mix.q.b", "l3.mlp.shared.up",
                "l1.mlp.e0.gate", "l1.mlp.shared.gate"} & set(specs)
    assert shapes["l0.hc1.in"] == shapes["l0.hc2.out"] == (3,) and shapes["l0.hc1.mix"] == (3, 3)
    assert shapes["l0.mix.q"] == (72, 80) and shapes["l0.mix.v"] == shapes["l0.mix.g"] == (120, 80) and shapes["l0.mix.o"] == (80, 120)
    assert shapes["l1.mix.q"] == (144, 80) and shapes["l1.mix.k.b"] == (48,) and shapes["l1.mix.o"] == (80, 144)
    assert shapes["l2.mix.norm"] == (48,) and shapes["l4.mix.norm"] == (96,)
    assert shapes["l1.mlp.e4.up"] == (24, 80) and shapes["l1.mlp.shared.down"] == (80, 40) and shapes["l1.mlp.router"] == (5, 80)
    assert "l2.mlp.up" not in specs and all(specs[n].optional for n in ("l2.norm2", "l2.hc2.in", "l2.hc2.mix", "l2.hc2.out"))
    assert not any(specs[n].optional for n in ("l1.norm2", "l1.hc2.in", "l2.hc1.in"))
    needs = model.cache_needs()
    assert needs[0] == StateNeed((3, 40, 24), torch.float32) and needs[2] == StateNeed((4, 12, 20), torch.float32)
    assert needs[1] == KVNeed(2, 24, 0, 24, 0, 20) and needs[3] == KVNeed(3, 40, 0, 40, 0, 70) and needs[5] == KVNeed(1, 16, 0, 16)


@pytest.mark.parametrize("key,value,text", [
    (("layers", 0, "type"), "delta", "layers[0].type"),
    (("layers", 0, "mixer"), None, "layers[0].mixer"),
    (("layers", 0, "mixer", "decay"), [0.5, 0.5], "mixer.decay"),
    (("layers", 0, "mixer", "decay"), [0.5, 0.5, 1.5], "mixer.decay"),
    (("layers", 0, "mixer", "rot"), None, "mixer.rot"),
    (("layers", 0, "mixer", "rot", "dims"), 26, "rot.dims"),
    (("layers", 0, "mixer", "rot", "dims"), 7, "rot.dims"),
    (("layers", 1, "mixer", "kv_heads"), 4, "kv_heads"),
    (("layers", 1, "mixer", "vdim"), 8, "mixer.vdim"),
    (("layers", 1, "mixer", "scale"), None, "mixer.scale"),
    (("layers", 1, "mixer", "mask", "size"), 0, "mask.size"),
    (("layers", 1, "mixer", "rot", "scaling", "factor"), None, "scaling.factor"),
    (("layers", 1, "mlp", "kind"), "sparse", "mlp.kind"),
    (("layers", 1, "mlp", "router", "top"), 6, "router.top"),
    (("layers", 1, "mlp", "expert", "ff"), None, "expert.ff"),
    (("layers", 1, "mlp", "shared", "ff"), 0, "shared.ff"),
    (("layers", 2, "mixer", "heads"), None, "mixer.heads"),
    (("streams",), 0, "streams"),
    (("streams",), None, "streams"),
    (("logit_softcap",), -1.0, "logit_softcap"),
    (("embedding", "scale"), "large", "embedding.scale"),
    (("norm", "eps"), None, "norm.eps"),
    (("width",), None, "width"),
])
def test_configuration_errors_name_their_key(key, value, text):
    cfg = copy.deepcopy(tc.CFG_A)
    d = cfg
    for k in key[:-1]:
        d = d[k]
    d[key[-1]] = value
    with pytest.raises(lq.ConfigError) as e:
        lq.TukedraConfig.from_dict(cfg)
    assert text in str(e.value)


def test_keys_that_a_configuration_leaves_out():
    cfg = copy.deepcopy(tc.CFG_CHUNKED)
    for key in ("embedding", "logit_scale"):
        del cfg[key]
    m = cfg["layers"][0]["mixer"]
    del m["kv_heads"], m["vdim"], m["mask"], m["rot"]["dims"], m["rot"]["scaling"]
    c = lq.TukedraConfig.from_dict(cfg)
    a = c.layers[0].attention
    assert (a.kv_heads, a.chunk, a.rot.dims, a.rot.scaling) == (4, 0, 16, None)
    assert (c.embedding_scale, c.logit_scale, c.logit_softcap) == (1.0, 1.0, 0.0)


def test_what_belongs_to_an_absent_feed_forward_may_be_in_the_file(tmp_path):
    cfg = copy.deepcopy(tc.CFG_LIGHTNING)
    weights = tc.make_weights(cfg, 5)
    t = tc.tokens(12, cfg["vocab"], 1)
    idle = {"l0.norm2": torch.full((48,), 3.0), "l0.hc2.in": torch.ones(1), "l0.hc2.mix": torch.ones(1, 1), "l0.hc2.out": torch.ones(1)}
    got = []
    for name, more in (("without", {}), ("with", idle)):
        eng = load(tc.write_folder(tmp_path, cfg, {**weights, **more}, name), "float32", 256)
        got.append(eng.step([StepEntry(eng.new_sequence(), t, range(12))]))
    assert torch.equal(got[0], got[1]) and tc.err(got[0], pt.forward(cfg, weights, t)) < TOL


def test_missing_and_unexpected_tensors_are_named(tmp_path):
    cfg = copy.deepcopy(tc.CFG_CHUNKED)
    weights = tc.make_weights(cfg, 5)
    weights["l0.mix.v"] = weights["l0.mix.k"].clone()  # the values are the keys
    del weights["l0.hc1.mix"], weights["l0.mix.q.b"]
    with pytest.raises(lq.WeightError) as e:
        load(tc.write_folder(tmp_path, cfg, weights, "bad"), "float32", 256)
    assert e.value.missing == ["l0.hc1.mix", "l0.mix.q.b"] and e.value.unexpected == ["l0.mix.v"]


def test_mechanisms_that_do_not_go_together_are_refused():
    attention = dict(width=8, heads=2, kv_heads=1, key_dim=4, value_dim=4, scale=1.0, prefix="x")
    for more in (dict(chunk=-1), dict(chunk=4, keep_first=2), dict(qk_norm="row", rotary={"dims": 4, "base": 10.0})):
        with pytest.raises(ValueError):
            build_part(MIXERS, PartSpec("sink_window_attention", {**attention, **more}))
    linear = dict(width=8, heads=2, key_dim=4, value_dim=4, decay=[0.5, 0.5], eps=0.0, prefix="x", norm="row", gate="silu")
    for more in (dict(decay=[0.5]), dict(norm="column"), dict(gate="relu"), dict(activation="relu"),
                 dict(rotary={"dims": 6, "base": 10.0})):
        with pytest.raises(ValueError):
            build_part(MIXERS, PartSpec("decayed_linear_attention", {**linear, **more}))
    moe = dict(width=8, experts=4, top=2, inner=8, prefix="x", weight_input=False, scoring="softmax_chosen", activation="relu2")
    for more in (dict(weight_input=True), dict(correction=True), dict(groups=2, keep=1), dict(identity=1),
                 dict(shared_inner=8, shared_gate=True)):
        with pytest.raises(ValueError):
            build_part(FEED_FORWARDS, PartSpec("moe", {**moe, **more}))
    mixer = PartSpec("decayed_linear_attention", linear)
    norm = PartSpec("rmsnorm", {"width": 8, "eps": 0.0, "name": "n"})
    squash = PartSpec("dynamic_tanh", {"width": 8, "name": "n"})
    block = dict(streams=2, mixer=mixer, mixer_norm=norm, mixer_links="l")
    for more in (dict(streams=0), dict(mixer_norm=squash), dict(feed_forward=PartSpec("moe", moe))):
        with pytest.raises(ValueError):
            build_part(BLOCKS, PartSpec("hyper_connected", {**block, **more}))


# ---- the plain implementation's own mechanisms against hand-made cases ---------------------------------------------
def test_plain_rotation_pairs_and_magnitude():
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 5.0]]] * 3, dtype=F)  # three positions
    f = [0.5, 0.1]
    half, inter = pt.rotate(x, f, 1.0, False), pt.rotate(x, f, 2.0, True)
    assert torch.equal(half[0, 0], x[0, 0]) and inter[0, 0].tolist() == [2.0, 4.0, 6.0, 8.0, 5.0]
    c, s, c1, s1 = math.cos(1.0), math.sin(1.0), math.cos(0.2), math.sin(0.2)  # position 2
    assert torch.allclose(half[2, 0], torch.tensor([1 * c - 3 * s, 2 * c1 - 4 * s1, 3 * c + 1 * s, 4 * c1 + 2 * s1, 5.0], dtype=F))
    assert torch.allclose(inter[2, 0], torch.tensor([2 * (1 * c - 2 * s), 2 * (2 * c + 1 * s), 2 * (3 * c1 - 4 * s1),
                                                     2 * (4 * c1 + 3 * s1), 5.0], dtype=F))


def test_plain_yarn_frequencies_by_hand():
    # dims 8, base 10: one turn within 2 pi 10 positions lies at 8 ln(10) / (2 ln 10) = 4 pairs, ten turns at 0
    sc = {"factor": 5.0, "original": 2 * math.pi * 10.0, "fast": 10.0, "slow": 1.0}
    f = [10.0 ** (-i / 4) for i in range(4)]
    want = [f[i] / 5.0 * (i / 4) + f[i] * (1 - i / 4) for i in range(4)]
    assert pt.yarn_frequencies(8, 10.0, sc) == pytest.approx(want, rel=1e-12)
    assert pt.yarn_magnitude(5.0) == pytest.approx(0.1 * math.log(5.0) + 1) and pt.yarn_magnitude(1.0) == 1.0
    # bounds: fast beyond the first pair is clamped to 0, slow beyond the last to dims - 1; equal bounds make a step
    assert pt.yarn_frequencies(8, 10.0, {**sc, "fast": 1e6}) == pytest.approx(want, rel=1e-12)
    far = pt.yarn_frequencies(8, 10.0, {**sc, "slow": 1e-6})
    assert far == pytest.approx([f[i] / 5.0 * (i / 7) + f[i] * (1 - i / 7) for i in range(4)], rel=1e-12)
    step = pt.yarn_frequencies(8, 10.0, {**sc, "fast": 1.0})
    assert step == pytest.approx(f, rel=1e-12)  # (lo = hi = 4: no pair is beyond it)


def test_plain_decayed_memory_by_hand():
    q = torch.tensor([[1.0, 0.0], [2.0, 1.0], [1.0, 1.0]], dtype=F)
    k = torch.tensor([[1.0, 3.0], [0.0, 1.0], [2.0, 0.0]], dtype=F)
    v = torch.tensor([[10.0], [100.0], [1000.0]], dtype=F)
    o = pt.decayed_memory(q, k, v, 0.5)
    # q1.k0 = 5, q1.k1 = 1; q2.k0 = 4, q2.k1 = 1, q2.k2 = 2
    assert o[:, 0].tolist() == [10.0, 0.5 * 5 * 10 + 100, 0.25 * 4 * 10 + 0.5 * 100 + 2000]
    assert pt.decayed_memory(q, k, v, 1.0)[2, 0] == 40 + 100 + 2000 and pt.decayed_memory(q, k, v, 0.0)[2, 0] == 2000


def test_plain_mixers_norm_and_gate():
    """One token: the memory answers (q . k) v, whose norm is a sign."""
    one = lambda *rows: torch.tensor(rows, dtype=F)
    h = one([1.0, 0.0])
    w = {"x.q": one([1.0, 0], [-2.0, 0]), "x.k": one([1.0, 0], [3.0, 0]), "x.v": one([1.0, 0], [2.0, 0]),
         "x.g": one([0.0, 0], [math.log(3.0), 0]), "x.o": one([1.0, 0], [0, 1.0]), "x.norm": torch.tensor([1.0, 5.0], dtype=F)}
    m = {"heads": 2, "dim": 1, "vdim": 1, "decay": [0.5, 0.5]}
    silu = lambda z: z / (1 + math.exp(-z))
    a, b = silu(1) ** 3, silu(-2) * silu(3) * silu(2)
    r = math.sqrt((a * a + b * b) / 2)  # both heads together
    y = pt.lightning(h, m, w, "x", 0.0, False)
    assert y[0].tolist() == pytest.approx([a / r * 0.5, b / r * 5.0 * 0.75], rel=1e-12)
    m = {"heads": 2, "dim": 1, "vdim": 1, "decay": [0.5, 0.5], "rot": {"base": 10.0, "dims": 0}}
    y = pt.retention(h, m, w, "x", 0.0, False)  # every head alone: +1 and -1, silu(0) = 0 and silu(ln 3)
    assert y[0].tolist() == pytest.approx([0.0, -math.log(3.0) * 0.75], rel=1e-12)
    # the eps sees the scaled keys: dim^(-1/2) = 1/2 for four entries
    w4 = {"x.q": torch.eye(4, dtype=F), "x.k": torch.eye(4, dtype=F), "x.v": one([1.0, 0, 0, 0]), "x.g": one([1.0, 0, 0, 0]), "x.o": one([1.0])}
    y = pt.retention(one([1.0, 1, 1, 1]), {"heads": 1, "dim": 4, "vdim": 1, "decay": [0.5], "rot": {"base": 10.0, "dims": 2}}, w4, "x",
                     5.0, False)
    assert float(y) == pytest.approx(2.0 / math.sqrt(4.0 + 5.0) * silu(1), rel=1e-12)


def test_plain_chunks_count_from_the_start_of_the_sequence():
    seen = pt.chunk_mask(7, 3)
    assert [row.nonzero().flatten().tolist() for row in seen] == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]
    assert pt.chunk_mask(3, None).sum() == 6


def test_plain_attention_reads_the_keys_before_rotation_and_norm():
    """One head of two entries, no positions to speak of (a base so large that position 1 turns by nearly nothing in the
    second pair; here one pair, angle p).  The first token sees itself: its key with the bias, as projected."""
    m = {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 0.7, "rot": {"base": 10.0, "dims": 2}}
    eye = torch.eye(2, dtype=F)
    w = {"x.q": eye, "x.k": 2 * eye, "x.q.b": torch.tensor([0.5, 0.0], dtype=F), "x.k.b": torch.tensor([0.0, 1.0], dtype=F), "x.o": eye}
    h = torch.tensor([[1.0, 2.0], [3.0, -1.0]], dtype=F)
    y = pt.attention(h, m, w, "x", 0.0, False)
    assert y[0].tolist() == [2.0, 5.0]
    k = [(2.0, 5.0), (6.0, -1.0)]
    q1 = (3.5, -1.0)
    turn = lambda v, a: (v[0] * math.cos(a) - v[1] * math.sin(a), v[1] * math.cos(a) + v[0] * math.sin(a))
    unit = lambda v: tuple(x / math.sqrt((v[0] ** 2 + v[1] ** 2) / 2) for x in v)
    q = unit(turn(q1, 1.0))
    e = [math.exp(0.7 * sum(a * b for a, b in zip(q, unit(turn(kk, float(p)))))) for p, kk in enumerate(k)]
    want = [sum(e[p] * k[p][i] for p in (0, 1)) / sum(e) for i in (0, 1)]
    assert y[1].tolist() == pytest.approx(want, rel=1e-12)
    assert pt.attention(h, {**m, "mask": {"size": 1}}, w, "x", 0.0, False)[1].tolist() == [6.0, -1.0]


def test_plain_router_and_experts_by_hand():
    z = torch.tensor([[1.0, 3.0, 3.0, 2.0], [0.0, 0.0, 0.0, 0.0]], dtype=F)
    r = pt.route(z, 3)
    e = math.exp(-1.0)
    assert r[0].tolist() == pytest.approx([0.0, 1 / (2 + e), 1 / (2 + e), e / (2 + e)]) and r[1].tolist() == pytest.approx([1 / 3] * 3 + [0.0])
    assert pt.route(z, 1)[0].tolist() == [0.0, 1.0, 0.0, 0.0]
    h = torch.tensor([[2.0, -1.0]], dtype=F)
    w = {"x.router": torch.tensor([[1.0, 0], [0, 1.0]], dtype=F)}
    for name, up in (("e0", [1.0, 0.0]), ("e1", [1.0, 1.0]), ("shared", [0.0, 1.0])):
        w[f"x.{name}.up"], w[f"x.{name}.down"] = torch.tensor([up], dtype=F), torch.tensor([[1.0], [10.0]], dtype=F)
    m = {"router": {"experts": 2, "top": 2}, "shared": {"ff": 1}}
    a, b = 1 / (1 + math.exp(-3.0)), 1 / (1 + math.exp(3.0))
    y = a * 4.0 + b * 1.0 + 0.0  # relu(2)^2, relu(1)^2, and the shared expert's relu(-1)
    assert pt.mixture(h, m, w, "x", False)[0].tolist() == pytest.approx([y, 10 * y], rel=1e-12)


def test_plain_streams_by_hand():
    X = torch.tensor([[[1.0]], [[10.0]]], dtype=F)
    mix = torch.tensor([[2.0, 3.0], [5.0, 7.0]], dtype=F)  # [from, to]
    Y = pt.write_streams(X, torch.tensor([[100.0]], dtype=F), mix, torch.tensor([1.0, -1.0], dtype=F))
    assert Y.flatten().tolist() == [2 + 50 + 100, 3 + 70 - 100]
    assert float(pt.read_streams(X, torch.tensor([0.5, 2.0], dtype=F))) == 20.5


def test_plain_model_scales_and_caps_its_ends():
    cfg, w = tc.CFG_CAPPED, tc.make_weights(copy.deepcopy(tc.CFG_CAPPED), 2)
    none = {n: torch.zeros_like(t) if n.endswith(".mix.o") else t for n, t in w.items()}  # the layer adds nothing
    t = [5, 9]
    x = 3.0 * w["embed"][t].double()
    u = torch.einsum("s,rw->rw", w["l0.hc1.mix"].double().sum(1), x)  # both streams mixed, then added up
    u = u / torch.sqrt((u * u).mean(-1, keepdim=True) + 1e-6) * w["final.norm"].double()
    assert torch.allclose(pt.forward(cfg, none, t), 1.5 * torch.tanh(u @ w["head"].double().T * 1.7 / 1.5))


# ---- every mechanism alone, and all of them, through the engine ------------------------------------------------------
@pytest.mark.parametrize("name", tc.ALONE)
def test_a_mechanism_alone(cases, name):
    case = cases(name)
    tc.whole_and_token_by_token(case, TOL, lengths=(1, 2, 9, 70))
    tc.portions(case, TOL, n=140)


@pytest.mark.parametrize("name", ["a", "b"])
def test_whole_prompts_against_token_by_token_decoding(cases, name):
    tc.whole_and_token_by_token(cases(name), TOL)


@pytest.mark.parametrize("name", ["a", "b"])
def test_portions_of_several_sizes_down_to_two_tokens(cases, name):
    tc.portions(cases(name), TOL)


@pytest.mark.parametrize("name", ["a", "b"])
def test_batches_of_unequal_requests_against_each_alone(cases, name):
    tc.unequal_batches(cases(name), TOL)


@pytest.mark.parametrize("name", ["a", "retention"])
def test_slots_and_blocks_are_freed_and_used_again(cases, name):
    tc.slots_and_blocks_used_again(cases(name), TOL)


@pytest.mark.parametrize("seed", [1, 2, 3, 4, 5, 6, 7, 8])
def test_configurations_drawn_from_a_seed(cases, seed):
    case = cases(seed)
    assert lq.TukedraConfig.from_dict(case.cfg).to_dict() == case.cfg
    t, u = tc.tokens(70, case.vocab, seed), tc.tokens(9, case.vocab, seed + 50)
    assert tc.err(case.run_cut(t, [40, 2, 1, 20]), case.want(t)) < TOL
    eng = case.eng
    sa, sb = eng.new_sequence(), eng.new_sequence()
    out = eng.step([StepEntry(sa, u[:8], range(8)), StepEntry(sb, t[:66], range(66))])
    assert tc.err(out, torch.cat([case.want(u)[:8], case.want(t)[:66]])) < TOL
    out = eng.step([StepEntry(sa, u[8:], [0]), StepEntry(sb, t[66:67], [0])])
    assert tc.err(out, torch.stack([case.want(u)[8], case.want(t)[66]])) < TOL
    eng.release(sa)
    eng.release(sb)
    case.assert_idle()


@pytest.mark.parametrize("name", ["a", "streams"])
def test_the_residual_stream_after_every_layer(cases, name):
    case = cases(name)
    got, want = case.layers(tc.tokens(37, case.vocab, 8))
    assert len(got) == len(want) == len(case.cfg["layers"])
    for i, (g, w) in enumerate(zip(got, want)):
        assert tc.err(g, w) < TOL, f"after layer {i}"


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
    assert tc.err(case.run_cut(t, [n]), want) < TOL
    assert tc.err(case.run_cut(t, [size, 1, 1, 2, size - 1 or 1, 3]), want) < TOL
    assert tc.err(case.run_cut(t, [max(1, size - 1)]), want) < TOL  # decoding across the chunk's edge
    case.assert_idle()


@pytest.mark.parametrize("name,leaves", [
    ("lightning", {"norm": 1.0}), ("lightning", {"g": 0.0}), ("retention", {"g": 0.5}), ("chunked", {"b": 0.0}),
    ("experts", {"router": 0.0}), ("streams", {"mix": 0.0}), ("streams", {"in": 1.0}), ("streams", {"out": 1.0}),
])
def test_every_learned_number_matters(cases, name, leaves):
    """With one of them flattened in the oracle the result differs by much, so the comparisons here see it."""
    case = cases(name)
    t = tc.tokens(60, case.vocab, 9)
    assert tc.err(pt.forward(case.cfg, tc.flattened(case.weights, **leaves), t), case.want(t)) > 1e-3
    assert tc.err(case.run_cut(t, [50, 2]), case.want(t)) < TOL


@pytest.mark.parametrize("name,change", [
    ("lightning", lambda c: c["layers"][0]["mixer"].update(decay=[0.6, 0.95, 0.999])),
    ("retention", lambda c: c["layers"][0]["mixer"]["rot"].update(base=101.0)),
    ("retention", lambda c: c["layers"][0]["mixer"]["rot"].update(dims=14)),
    ("chunked", lambda c: c["layers"][0]["mixer"].update(scale=0.31)),
    ("chunked", lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=6.0)),
    ("chunked", lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(original=256)),
    ("experts", lambda c: c["layers"][0]["mlp"]["router"].update(top=3)),
    ("capped", lambda c: c["embedding"].update(scale=2.5)), ("capped", lambda c: c.update(logit_scale=1.75)),
    ("capped", lambda c: c.update(logit_softcap=1.6)),
])
def test_every_constant_matters(cases, name, change):
    case = cases(name)
    cfg = copy.deepcopy(case.cfg)
    change(cfg)
    if name == "capped" and cfg["embedding"] != case.cfg["embedding"]:
        cfg["norm"]["eps"] = case.cfg["norm"]["eps"] = 1.0  # (a norm follows: the scale shows through its eps alone)
        wrong, right = (pt.forward(c, case.weights, [1, 2, 3]) for c in (cfg, case.cfg))
        case.cfg["norm"]["eps"] = 1e-6
        assert tc.err(wrong, right) > 1e-3
        return
    t = tc.tokens(60, case.vocab, 9)
    assert tc.err(pt.forward(cfg, case.weights, t), case.want(t)) > 1e-4


@pytest.mark.parametrize("name", ["lightning", "retention"])
def test_a_slow_decay_keeps_old_tokens_in_the_state(cases, name):
    """Decays close to one: the first tokens still weigh in the state after hundreds of steps, so a state that is lost,
    reset or carried to the wrong slot shows far from where it happened."""
    case = cases(f"{name}-slow", cfg=tc.slow(name))
    t = tc.tokens(260, case.vocab, 31)
    want = case.want(t)
    other = case.want([(t[0] + 1) % case.vocab] + t[1:])
    assert tc.err(other[-1], want[-1]) > 1e-3  # the first token still matters at the end
    assert tc.err(case.run_cut(t, [260]), want) < TOL
    assert tc.err(case.run_cut(t, [3, 64, 1, 2, 130]), want) < TOL


def test_the_first_tokens_start_from_nothing(cases):
    """States start at zero and chunks at the sequence's first token, also in a slot that another sequence has left, and
    whether the first step brings one token or several."""
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
        assert tc.err(out, case.want(b)[:first]) < TOL
        if first < 6:
            out = eng.step([StepEntry(s, b[first:], range(6 - first))])
            assert tc.err(out, case.want(b)[first:]) < TOL
        eng.release(s)
    case.assert_idle()


def test_chunked_groups_give_their_blocks_back(cases):
    case = cases("chunked")  # one layer, chunks of 40: never more than two blocks a sequence, and one right after an edge
    eng = case.eng
    s = eng.new_sequence()
    t = tc.tokens(400, case.vocab, 3)
    eng.step([StepEntry(s, t[:300], [])])
    held = []
    for i in range(300, 400):
        eng.step([StepEntry(s, t[i : i + 1], [])])
        held.append(max(g.blocks.taken_count for g in eng.cache.kv_groups))
    assert max(held) <= 2 and held[319 - 300] == 0  # (320 tokens end a chunk and a block: nothing is needed any more)
    out = eng.step([StepEntry(s, [5], [0])])
    assert tc.err(out[0], case.want(t + [5])[-1]) < TOL
    eng.release(s)
    case.assert_idle()


@pytest.mark.parametrize("name", ["experts", "a"])
def test_prompts_sorted_by_expert(cases, name, monkeypatch):
    """Rows enough for the way that sorts a step's rows by expert."""
    from longbow_quarrel_amd.parts.feedforward import MixtureOfExperts
    case = cases(name)
    monkeypatch.setattr(MixtureOfExperts, "sort_from_rows", 16)
    t = tc.tokens(60, case.vocab, 12)
    assert tc.err(case.run_cut(t, [60]), case.want(t)) < TOL
    assert tc.err(case.run_cut(t, [15, 30]), case.want(t)) < TOL


def test_streams_between_blocks_of_other_kinds():
    """A block that knows nothing of the streams gets their sum, and the copies start again, equal, behind it."""
    from longbow_quarrel_amd.model import DecoderModel, ModelSpec, Run, token_table
    from longbow_quarrel_amd.parts.base import BuildEnv
    from longbow_quarrel_amd.engine.step import Engine

    norm = lambda n: PartSpec("rmsnorm", {"width": 8, "eps": 1e-6, "name": n})
    dense = lambda p: PartSpec("swiglu", {"width": 8, "inner": 8, "prefix": p, "names": {"gate": "g", "up": "u", "down": "d"}})
    linear = lambda p: PartSpec("decayed_linear_attention", {"width": 8, "heads": 1, "key_dim": 4, "value_dim": 4, "decay": [0.5],
                                                             "eps": 1e-6, "prefix": p, "norm": "row", "gate": "silu"})
    hyper = lambda i: PartSpec("hyper_connected", {"streams": 3, "mixer": linear(f"m{i}"), "mixer_norm": norm(f"n{i}"), "mixer_links": f"c{i}"})
    spec = ModelSpec(20, 8, token_table("e", 20, 8), (hyper(0), hyper(1), PartSpec("prenorm", {
        "mixer": linear("p"), "feed_forward": dense("f"), "mixer_norm": norm("pn"), "ffn_norm": norm("fn")}), hyper(2)),
        tuple(Run(i) for i in range(4)), norm("z"), "head", False)
    model = DecoderModel(spec)
    g = torch.Generator().manual_seed(1)
    w = {s.name: torch.randn(s.shape, generator=g) for s in model.tensor_specs()}
    model.bind(dict(w), BuildEnv(torch.float32, torch.device("cpu"), CpuKernels()))
    eng = Engine(model, model.env, 256, 4)
    t = [3, 7, 1, 1, 19]
    got = eng.step([StepEntry(eng.new_sequence(), t, range(5))])
    d = {n: v.double() for n, v in w.items()}

    def lin(h, p):
        m = {"heads": 1, "decay": [0.5]}
        q, k, v = (h @ d[f"{p}.{n}"].T for n in "qkv")
        o = pt.rms(pt.decayed_memory(q, k, v, 0.5), 1e-6) * d[p + ".norm"]
        return o * pt.silu(h @ d[p + ".g"].T) @ d[p + ".o"].T

    def stage(X, i):
        u = pt.rms(pt.read_streams(X, d[f"c{i}.in"]), 1e-6) * d[f"n{i}"]
        return pt.write_streams(X, lin(u, f"m{i}"), d[f"c{i}.mix"], d[f"c{i}.out"])

    x = d["e"][t]
    x = stage(stage(torch.stack([x] * 3), 0), 1).sum(0)
    x = x + lin(pt.rms(x, 1e-6) * d["pn"], "p")
    h = pt.rms(x, 1e-6) * d["fn"]
    x = x + (pt.silu(h @ d["f.g"].T) * (h @ d["f.u"].T)) @ d["f.d"].T
    x = stage(torch.stack([x] * 3), 2).sum(0)
    assert tc.err(got, (pt.rms(x, 1e-6) * d["z"]) @ d["head"].T) < TOL


def test_long_decoding(cases):
    tc.long_decoding(cases("a"), TOL)


def test_greedy_generation_through_the_generation_loop(cases):
    case = cases("a")
    reqs, wants = tc.greedy(case)
    result = lq.generate(case.eng, reqs, max_new_tokens=10)
    assert result.tokens == wants
    case.assert_idle()


def test_bfloat16_run_rounds_where_the_plain_implementation_does(tmp_path_factory):
    case = tc.Case(tmp_path_factory.mktemp("tukedra16"), "a", load, dtype="bfloat16", rounding=True)
    t = tc.tokens(80, case.vocab, 3)
    tc.assert_close_bf16(case.run_cut(t, [50, 2]), case.want(t), case.noise(t))


def test_random_weights_give_an_engine_that_steps():
    eng = lq.random_engine(lq.TukedraConfig.from_dict(tc.CFG_A), 1, dtype="float32", device="cpu", kernels=CpuKernels(),
                           max_tokens=256, max_slots=2)
    out = eng.step([StepEntry(eng.new_sequence(), [1, 2, 3], [2])])
    assert bool(torch.isfinite(out).all()) and float(out.abs().max()) > 0
    mix = eng.model.blocks[0].links[0][1]
    assert float((mix.diagonal() - 1).abs().max()) < 0.6 and float((mix - torch.diag(mix.diagonal())).abs().max()) < 0.6
