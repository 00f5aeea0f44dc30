"""The Zisedra design without a GPU: the configuration reader, the model's description (tensors, runs, cache
units), the plain implementation's mechanisms against numbers worked by hand, and random models written and read
back."""
import copy
import importlib
import math

import numpy as np
import pytest

import plain_zisedra as pz
import zisedra_configs as zc

L = importlib.import_module("daisi-llogos_amd")
registry = importlib.import_module("daisi-llogos_amd.config.registry")
model_mod = importlib.import_module("daisi-llogos_amd.models.model")
config_mod = importlib.import_module("daisi-llogos_amd.config.model_config")
kernels = importlib.import_module("daisi-llogos_amd.ops.kernels")
parts = importlib.import_module("daisi-llogos_amd.parts")


def _model(cfg, shapes=None):
    arch = registry.architecture_of(cfg)
    typed = arch.read_config(cfg, shapes=shapes)
    return typed, model_mod.Model(arch.model_spec(typed))


def test_the_reader_takes_every_size_and_constant_from_the_file():
    typed, _ = _model(zc.ZIS_A)
    assert (typed.vocab, typed.width, typed.norm_eps, typed.residual_mult) == (131, 96, 1e-5, 0.45)
    assert (typed.loop.start, typed.loop.stop, typed.loop.times) == (1, 3, 2)
    assert [l.type for l in typed.layers] == ["delta", "parallel", "delta", "parallel"]
    m = typed.layers[0].mixer
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.conv, m.decay_rank, m.gate_rank) == (4, 2, 24, 40, 4, 0, 0)
    a, r = typed.layers[1].left, typed.layers[1].right
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.window, a.rot_dims, a.rot_base) == (3, 1, 24, 40, 0.4, 37, 12, 500.0)
    assert (a.scaling.factor, a.scaling.low, a.scaling.high, a.scaling.original) == (4.0, 1.0, 4.0, 64.0)
    assert (r.heads, r.kv_heads, r.dim, r.vdim, r.conv, r.decay_rank, r.gate_rank) == (3, 3, 16, 24, 3, 12, 20)
    assert typed.layers[3].left.scaling is None
    f = typed.layers[0].mlp
    assert (f.ff, f.limit, f.experts, f.top, f.groups, f.keep, f.shared_ff, f.shared_limit) == (40, 1.0, 6, 2, 3, 2, 56, 0.6)
    f = typed.layers[1].mlp
    assert (f.experts, f.groups, f.keep, f.shared_ff) == (4, 1, 1, 0)
    assert typed.layers[2].mlp is None and not typed.layers[2].second_norm
    typed, _ = _model(zc.ZIS_B)
    assert typed.residual_mult == 1.0 and typed.layers[0].left.rot_dims == 0
    typed, _ = _model(zc.ZIS_E)
    assert typed.loop is None and typed.layers[1].left.window == 0


@pytest.mark.parametrize("path,value,word", [
    (("layers", 0, "type"), "delta_9", "delta_9"), (("layers", 0, "mixer", "heads"), None, "heads"), (("layers", 0, "mixer", "heads"), 3, "kv_heads"),
    (("layers", 0, "mixer", "dim"), 0, "dim"), (("layers", 0, "mixer", "conv"), 0, "conv"), (("layers", 0, "mixer", "conv"), None, "conv"),
    (("layers", 1, "mixer", "left"), None, "left"), (("layers", 1, "mixer", "right"), None, "right"), (("layers", 1, "mixer", "left", "scale"), None, "scale"),
    (("layers", 1, "mixer", "left", "rot", "dims"), 7, "dims"), (("layers", 1, "mixer", "left", "rot", "dims"), 26, "dims"),
    (("layers", 1, "mixer", "left", "rot", "base"), None, "base"), (("layers", 1, "mixer", "left", "mask", "size"), 0, "size"),
    (("layers", 1, "mixer", "left", "rot", "scaling", "high"), 1.0, "low"), (("layers", 1, "mixer", "left", "rot", "scaling", "factor"), None, "factor"),
    (("layers", 1, "mixer", "right", "decay_rank"), 0, "decay_rank"), (("layers", 0, "mlp", "kind"), "sparse", "sparse"), (("layers", 0, "mlp", "router", "top"), 5, "top"),
    (("layers", 0, "mlp", "router", "groups", "count"), 4, "count"), (("layers", 0, "mlp", "router", "groups", "keep"), 4, "keep"),
    (("layers", 0, "mlp", "expert", "limit"), None, "limit"), (("layers", 0, "mlp", "shared", "limit"), None, "limit"), (("layers", 0, "mlp", "expert"), None, "expert"),
    (("loop", "stop"), 5, "loop"), (("loop", "start"), 3, "loop"), (("loop", "times"), 0, "times"), (("norm",), None, "norm"), (("width",), "wide", "width"),
    (("vocab",), 0, "vocab"), (("layers",), [], "layers")])
def test_a_wrong_or_missing_key_is_named(path, value, word):
    cfg = copy.deepcopy(zc.ZIS_A)
    at = cfg
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    with pytest.raises(config_mod.ConfigError) as e:
        _model(cfg)
    assert word in str(e.value)


def test_the_description_runs_a_loop_with_units_of_its_own_for_every_pass():
    _, model = _model(zc.ZIS_A)
    assert [(e.layer, e.enter) for e in model.schedule] == [(0, None), (1, (0, 0)), (2, None), (1, (0, 1)), (2, None), (3, None)]
    needs = model.cache_needs()
    assert len(needs) == 9 and model.cache_reads() == [None] * 9         # a pair of mixers asks for two units
    size = lambda h, g, d, v, taps: h * d * v + taps * (2 * g * d + h * v)
    alone, beside, last = size(2, 1, 32, 16, 2), size(3, 3, 16, 24, 3), size(2, 1, 24, 56, 5)
    assert [n[1].shape[0] if n[1] else None for n in needs] == [size(4, 2, 24, 40, 4), None, beside, alone, None, beside, alone, None, last]
    kv = needs[1][0]
    assert needs[4][0] == kv and (kv.n_kv_heads, kv.head_dim, kv.value_dim, kv.window, kv.sinks) == (1, 32, 48, 37, 0)
    names = {s.name: tuple(s.shape) for s in model.tensor_specs()}
    assert names["embed"] == (131, 96) and names["loop.in"] == (96, 192) and "loop.step" not in names and "head" not in names
    assert names["l0.mix.q"] == (48, 96) and names["l0.mix.v"] == (160, 96) and names["l0.mix.v.conv"] == (160, 4) and names["l0.mix.a"] == (4, 96)
    assert names["l0.mix.A_log"] == (4,) and names["l0.mix.dt_bias"] == (4,) and names["l0.mix.norm"] == (40,) and names["l0.mix.g"] == (160, 96)
    assert names["l0.mix.o"] == (96, 160) and names["l0.mix.b"] == (4, 96)
    assert names["l1.mix.left.q"] == (72, 96) and names["l1.mix.left.q.b"] == (72,) and names["l1.mix.left.v.b"] == (40,) and "l1.mix.left.o.b" not in names
    assert names["l1.mix.right.a1"] == (12, 96) and names["l1.mix.right.a2"] == (48, 12) and names["l1.mix.right.dt_bias"] == (48,)
    assert names["l1.mix.right.g1"] == (20, 96) and names["l1.mix.right.g2"] == (72, 20) and "l1.mix.right.a" not in names and "l1.mix.right.low" not in names
    assert names["l1.mix.left.out"] == (96,) and names["l1.mix.right.out"] == (96,)
    assert names["l0.mlp.router"] == (6, 96) and names["l0.mlp.e5.down"] == (96, 40) and names["l0.mlp.shared.up"] == (56, 96) and "l0.mlp.correction" not in names
    assert "l1.mlp.shared.up" not in names and "l2.norm2" not in names and names["l3.norm2"] == (96,) and names["final.norm"] == (96,)
    assert model.graph_safe and model.spec.tie_head
    _, model = _model(zc.ZIS_B)
    assert [e.layer for e in model.schedule] == [0, 1] * 3 and [e.enter for e in model.schedule][::2] == [(0, 0), (0, 1), (0, 2)]
    _, model = _model(zc.ZIS_D)
    assert [(e.layer, e.enter) for e in model.schedule] == [(0, None), (1, (0, 0))]
    assert not any(s.name.startswith("loop") for s in _model(zc.ZIS_E)[1].tensor_specs())


def test_sizes_that_only_the_tensors_give():
    cfg = copy.deepcopy(zc.ZIS_A)
    for k in ("decay_rank", "gate_rank"):
        del cfg["layers"][1]["mixer"]["right"][k]
    typed, model = _model(cfg, shapes={"l1.mix.right.a1": (9, 96), "l1.mix.right.g1": (31, 96), "l2.norm2": (96,)})
    assert (typed.layers[1].right.decay_rank, typed.layers[1].right.gate_rank) == (9, 31) and typed.layers[2].second_norm
    names = {s.name: tuple(s.shape) for s in model.tensor_specs()}
    assert names["l1.mix.right.a2"] == (48, 9) and names["l1.mix.right.g2"] == (72, 31) and names["l2.norm2"] == (96,)       # a norm that nothing reads may be there


def test_random_models_are_written_and_read_back(tmp_path):
    for name, cfg in zc.ALL.items():
        path = L.write_random_model(str(tmp_path / name), cfg, seed=3)
        got_cfg, tensors = pz.load(path)
        assert got_cfg == cfg
        _, model = _model(cfg)
        assert {s.name: tuple(s.shape) for s in model.tensor_specs()} == {k: v.shape for k, v in tensors.items()}
        logits = pz.forward(got_cfg, tensors, [1, 2, 3, 4, 5])
        assert logits.shape == (5, cfg["vocab"]) and np.isfinite(logits).all()


def test_what_the_parts_refuse():
    rec = dict(prefix="m.", hidden=8, n_heads=2, n_kv_heads=1, head_dim=8, v_dim=8, conv_taps=2, eps=1e-5)
    for bad in (dict(n_kv_heads=3), dict(head_dim=kernels.DELTA_MAX_DIM + 1), dict(v_dim=kernels.DELTA_MAX_V + 1), dict(conv_taps=0), dict(conv_taps=17), dict(gate="tanh")):
        with pytest.raises(ValueError):
            parts.Delta(**dict(rec, **bad))
    moe = dict(prefix="f.", hidden=8, n_experts=4, top=1, intermediate=8)
    for bad in (dict(group_score="mean"), dict(out_scale=2.0, weigh="input"), dict(groups=3), dict(groups=4, keep=1, top=2)):
        with pytest.raises(ValueError):
            parts.RoutedMoE(**dict(moe, **bad))
    pair = dict(hidden=8, left=("delta", dict(rec, prefix="l.")), left_norm="a", right_norm="b", eps=1e-5)
    with pytest.raises(ValueError):
        parts.SideBySide(right=("wkv", dict(prefix="r.", hidden=8, n_heads=1, head_dim=8, decay_rank=2, eps=1e-5)), **pair)
    nested = parts.SideBySide(right=("side_by_side", dict(pair, left=("delta", dict(rec, prefix="x.")), right=("delta", dict(rec, prefix="r.")))), **pair)
    assert [p.prefix for p in nested.cache_parts()] == ["l.", "x.", "r."]


# ---------------------------------------------------------------------------
# the plain implementation's mechanisms against numbers worked by hand
# ---------------------------------------------------------------------------
def test_the_norms_and_the_activations():
    x = np.array([[3.0, -4.0]])
    rms = math.sqrt(12.5 + 0.5)
    assert np.allclose(pz.norm(x, np.array([0.5, -0.25]), 0.5), [[1.5 / rms, 1.0 / rms]])
    assert np.allclose(pz.length_one(x), x / math.sqrt(25.0 + 1e-6))
    assert np.allclose(pz.silu(np.array([1.0, -2.0])), [1.0 / (1.0 + math.exp(-1.0)), -2.0 / (1.0 + math.exp(2.0))])
    assert np.allclose(pz.softplus(np.array([0.0, 50.0, -50.0])), [math.log(2.0), 50.0, math.exp(-50.0)])


def test_the_convolutions_last_tap_is_the_tokens_own():
    x = np.array([[1.0, 10.0], [2.0, 20.0], [3.0, 30.0]])
    taps = np.array([[0.5, 0.25, 1.0], [0.0, 2.0, 1.0]])
    assert np.allclose(pz.short_conv(x, taps), [[1.0, 10.0], [2.25, 40.0], [0.5 + 0.5 + 3.0, 70.0]])
    assert np.allclose(pz.short_conv(x, np.array([[2.0], [3.0]])), x * [2.0, 3.0])


def test_the_delta_rule_by_hand():
    q, k = np.array([[[1.0, 2.0]], [[3.0, -1.0]]]), np.array([[[0.6, 0.8]], [[1.0, 0.0]]])
    v, beta, g = np.array([[[10.0]], [[4.0]]]), np.array([[0.5], [0.25]]), np.array([[[0.5, 0.5]], [[0.1, 0.2]]])
    o, S = pz.delta_recurrence(q, k, v, beta, g)
    s0 = np.array([0.6, 0.8]) * 5.0                            # u = 0.5 * (10 - 0)
    assert np.allclose(o[0, 0, 0], s0 @ [1.0, 2.0])            # a token reads its own write
    d = s0 * [0.1, 0.2]                                        # each key channel by its own decay, ahead of everything else
    u = 0.25 * (4.0 - d[0])
    s1 = d + np.array([1.0, 0.0]) * u
    assert np.allclose(S[0, :, 0], s1) and np.allclose(o[1, 0, 0], s1 @ [3.0, -1.0])
    o2, _ = pz.delta_recurrence(q[1:], k[1:], v[1:], beta[1:], g[1:], s0.reshape(1, 2, 1))
    assert np.allclose(o2[0], o[1])


def test_what_enters_the_recurrence_by_hand():
    rng = np.random.default_rng(0)
    h, m = rng.standard_normal((2, 4)), {"heads": 4, "kv_heads": 2, "dim": 2, "vdim": 1}
    t = {"q": rng.standard_normal((4, 4)), "k": rng.standard_normal((4, 4)), "v": rng.standard_normal((4, 4)), "b": rng.standard_normal((4, 4)),
         "q.conv": np.ones((4, 1)), "k.conv": np.ones((4, 1)), "v.conv": np.ones((4, 1)), "A_log": np.log([1.0, 2.0, 3.0, 4.0]), "a": rng.standard_normal((4, 4)),
         "dt_bias": np.array([0.1, 0.2, 0.3, 0.4])}
    q, k, v, beta, g = pz.delta_inputs(h, t, m)
    raw = pz.silu(t["q"] @ h[1])
    assert np.allclose(q[1, 1], q[1, 0]) and np.allclose(q[1, 3], raw[2:] / np.sqrt((raw[2:] ** 2).sum() + 1e-6) / math.sqrt(2.0))      # two heads a key head
    assert np.allclose((k ** 2).sum(-1), 1.0, atol=1e-3) and np.allclose(v[1, 2], pz.silu(t["v"][2] @ h[1]))
    assert np.allclose(beta[1, 3], 1.0 / (1.0 + math.exp(-(t["b"][3] @ h[1]))))
    assert np.allclose(g[1, 2], math.exp(-3.0 * math.log1p(math.exp(t["a"][2] @ h[1] + 0.3))))
    del t["a"]
    t.update(a1=rng.standard_normal((3, 4)), a2=rng.standard_normal((8, 3)), dt_bias=np.arange(8) * 0.1)
    g = pz.delta_inputs(h, t, m)[4]
    z = t["a2"] @ (t["a1"] @ h[1]) + t["dt_bias"]
    assert np.allclose(g[1, 2, 1], math.exp(-3.0 * math.log1p(math.exp(z[5]))))


def test_the_rotation_pairs_neighbours_and_leaves_the_rest():
    x = np.arange(1.0, 7.0).reshape(1, 1, 6)
    f = pz.frequencies(4, 100.0)
    assert np.allclose(f, [1.0, 0.1])
    got = pz.rotate(np.repeat(x, 2, axis=0), [0, 1], f)
    c, s, c2, s2 = math.cos(1.0), math.sin(1.0), math.cos(0.1), math.sin(0.1)
    assert np.allclose(got[0, 0], x[0, 0])
    assert np.allclose(got[1, 0], [c - 2.0 * s, 2.0 * c + s, 3.0 * c2 - 4.0 * s2, 4.0 * c2 + 3.0 * s2, 5.0, 6.0])


def test_long_wavelengths_are_slowed_and_those_between_mixed():
    sc = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 100.0}
    f = pz.frequencies(8, 10.0 ** 4, sc)
    plain = [10.0 ** -i for i in range(4)]                     # wavelengths 6.3, 62.8, 628, 6283
    s = (100.0 / (2 * math.pi / plain[1]) - 1.0) / 3.0
    assert np.allclose(f, [plain[0], (1 - s) * plain[1] / 4.0 + s * plain[1], plain[2] / 4.0, plain[3] / 4.0])
    made = parts.Rotary(8, 8, 10.0 ** 4, pairing="interleaved", scaling={"type": "llama3", "factor": 4.0, "low_freq_factor": 1.0, "high_freq_factor": 4.0,
                                                                         "original_max_position_embeddings": 100.0}).freqs
    assert np.allclose(made, f, rtol=1e-12)


def test_the_window_counts_the_query_itself():
    p = pz.window_softmax(np.zeros((4, 4)), 2)
    assert np.allclose(p, [[1, 0, 0, 0], [0.5, 0.5, 0, 0], [0, 0.5, 0.5, 0], [0, 0, 0.5, 0.5]])
    assert np.allclose(pz.window_softmax(np.zeros((3, 3)), 1), np.eye(3))


def test_the_bounds_of_an_expert_by_hand():
    t = {"gate": np.array([[1.0], [1.0], [1.0]]), "up": np.array([[1.0], [-9.0], [9.0]]), "down": np.array([[1.0, 10.0, 100.0]])}
    got = pz.clamped_ff(np.array([[0.5], [4.0], [-4.0]]), t, 2.0)
    act = lambda g: g / (1.0 + math.exp(-1.702 * g))
    assert np.allclose(got[0, 0], act(0.5) * (1.5 - 10.0 + 300.0))
    assert np.allclose(got[1, 0], act(2.0) * (3.0 - 10.0 + 300.0))               # the gate is bounded from above ...
    assert np.allclose(got[2, 0], act(-4.0) * (-1.0 + 30.0 - 100.0))             # ... and from above alone, up on both sides


def test_the_choice_within_the_best_groups_by_hand():
    s = np.array([0.9, 0.1, 0.6, 0.55, 0.5, 0.5])              # groups: 1.0, 1.15, 1.0
    assert pz.choose(s, 2, 3, 1).tolist() == [2, 3]            # (the largest score is in a group that is not kept)
    assert pz.choose(s, 3, 3, 2).tolist() == [0, 2, 3] and pz.choose(s, 3, 1, 1).tolist() == [0, 2, 3]
    assert pz.choose(s, 2, 6, 2).tolist() == [0, 2]            # groups of one
    h = np.array([[1.0]])
    t = {"router": np.log(s / (1 - s))[:, None]}
    for e in range(6):
        t.update({f"e{e}.gate": np.array([[1.0]]), f"e{e}.up": np.array([[0.0]]), f"e{e}.down": np.array([[10.0 ** e]])})
    a = 1.0 / (1.0 + math.exp(-1.702))
    entry = zc.moe(6, 2, 1, 7.0, (3, 1))
    assert np.allclose(pz.mixture(h, t, entry), a * (0.6 * 100.0 + 0.55 * 1000.0))           # the scores as they are
    t.update({"shared.gate": np.array([[1.0]]), "shared.up": np.array([[5.0]]), "shared.down": np.array([[1.0]])})
    assert np.allclose(pz.mixture(h, t, zc.moe(6, 2, 1, 7.0, (3, 1), (1, 2.0))), a * (0.6 * 100.0 + 0.55 * 1000.0 + 3.0))


def test_a_pass_begins_with_the_stream_and_the_embedding_output_through_a_matrix():
    assert pz.runs(zc.ZIS_A) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    cfg = copy.deepcopy(zc.ZIS_D)
    cfg["loop"]["times"] = 2
    _, model = _model(cfg)
    rng = np.random.default_rng(2)
    t = {s.name: rng.standard_normal(s.shape) for s in model.tensor_specs()}
    for k in t:                                                # layers that add nothing: what is left are the entries
        if k.endswith((".mix.o", ".down", ".out")):
            t[k] = np.zeros_like(t[k])
    streams = []
    pz.forward(cfg, t, [7], streams)
    x0, A, B = t["embed"][7], t["loop.in"][:, :48], t["loop.in"][:, 48:]
    once = A @ x0 + B @ x0
    assert np.allclose(streams[0][0], x0) and np.allclose(streams[1][0], once) and np.allclose(streams[2][0], A @ once + B @ x0)


def test_the_factor_is_on_what_a_sublayer_adds():
    cfg = copy.deepcopy(zc.ZIS_D)
    del cfg["loop"]
    _, model = _model(cfg)
    rng = np.random.default_rng(3)
    t = {s.name: rng.standard_normal(s.shape) * 0.3 for s in model.tensor_specs()}
    x = rng.standard_normal((4, 48))
    one = pz.layer(x, pz.part(t, "l0."), cfg["layers"][0], 1e-5, 1.0)
    assert np.allclose(pz.layer(x, pz.part(t, "l0."), cfg["layers"][0], 1e-5, 0.25), x + 0.25 * (one - x))
