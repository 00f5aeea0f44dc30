"""The Peponex design without a GPU: the configuration reader, the model's description (tensors, runs, cache
units), the plain implementation's mechanisms against numbers worked by hand, and random models written and read
back."""
import copy
import importlib
import math

import numpy as np
import pytest

import peponex_configs as pc
import plain_peponex as pp

L = importlib.import_module("daisi-llogos_amd")
registry = importlib.import_module("daisi-llogos_amd.config.registry")
model_mod = importlib.import_module("daisi-llogos_amd.models.model")
config_mod = importlib.import_module("daisi-llogos_amd.config.model_config")
kernels = importlib.import_module("daisi-llogos_amd.ops.kernels")


def _model(cfg, shapes=None):
    arch = registry.architecture_of(cfg)
    typed = arch.read_config(cfg, shapes=shapes)
    return typed, model_mod.Model(arch.model_spec(typed))


def test_the_reader_takes_every_size_and_constant_from_the_file():
    typed, _ = _model(pc.PEP_A)
    assert (typed.vocab, typed.width, typed.norm_eps, typed.logit_softcap, typed.side_dim) == (131, 96, 1e-5, 6.0, 20)
    assert (typed.loop.start, typed.loop.stop, typed.loop.times) == (1, 3, 2)
    assert [l.type for l in typed.layers] == ["wkv", "lightning", "latent_attention", "wkv"]
    m = typed.layers[0].mixer
    assert (m.heads, m.dim, m.decay_rank) == (3, 16, 12)
    m = typed.layers[1].mixer
    assert (m.heads, m.dim, m.vdim, m.decay) == (2, 24, 40, (0.5, 0.97))
    m = typed.layers[2].mixer
    assert (m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.scale, m.rot_dims, m.rot_base, m.window) == (3, 24, 8, 40, 40, 0.3, 8, 10000.0, 37)
    f = typed.layers[0].mlp
    assert (f.kind, f.ff) == ("dense", 136)
    f = typed.layers[1].mlp
    assert (f.kind, f.ff, f.experts, f.top) == ("moe", 40, 5, 2)
    assert typed.layers[3].mlp is None and not typed.layers[3].second_norm
    typed, _ = _model(pc.PEP_B)
    assert typed.side_dim == 0 and typed.logit_softcap == 0.0
    assert _model(pc.PEP_E)[0].loop is None


@pytest.mark.parametrize("path,value,word", [
    (("layers", 0, "type"), "wkv_9", "wkv_9"), (("layers", 1, "mixer", "decay"), [0.5], "decay"), (("layers", 1, "mixer", "decay"), "fast", "decay"),
    (("layers", 1, "mixer", "decay"), None, "decay"), (("layers", 0, "mixer", "heads"), None, "heads"), (("layers", 0, "mixer", "dim"), 0, "dim"),
    (("layers", 2, "mixer", "kv_rank"), None, "kv_rank"), (("layers", 2, "mixer", "scale"), None, "scale"), (("layers", 2, "mixer", "rot", "dims"), 7, "dims"),
    (("layers", 2, "mixer", "rot", "dims"), 10, "dims"), (("layers", 2, "mixer", "rot", "base"), None, "base"), (("layers", 2, "mixer", "mask", "size"), 0, "size"),
    (("layers", 2, "mixer", "mask", "size"), None, "size"), (("layers", 0, "mlp", "kind"), "sparse", "sparse"), (("layers", 1, "mlp", "router", "top"), 6, "top"),
    (("layers", 1, "mlp", "expert"), None, "expert"), (("layers", 0, "mlp", "ff"), 0, "ff"), (("loop", "stop"), 5, "loop"), (("loop", "start"), 3, "loop"),
    (("loop", "times"), 0, "times"), (("token_side", "dim"), None, "dim"), (("norm",), None, "norm"), (("width",), "wide", "width"), (("vocab",), 0, "vocab")])
def test_a_wrong_or_missing_key_is_named(path, value, word):
    cfg = copy.deepcopy(pc.PEP_A)
    at = cfg
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    with pytest.raises(config_mod.ConfigError) as e:
        _model(cfg)
    assert word in str(e.value)


def test_the_description_runs_a_loop_with_units_of_its_own_for_every_pass():
    _, model = _model(pc.PEP_A)
    assert [(e.layer, e.enter) for e in model.schedule] == [(0, None), (1, (0, 0)), (2, None), (1, (0, 1)), (2, None), (3, None)]
    needs = model.cache_needs()
    assert model.cache_reads() == [None] * 6
    assert [n[1].shape if n[1] else None for n in needs] == [(3 * 16 * 16 + 96,), (2 * 24 * 40,), None, (2 * 24 * 40,), None, (2 * 32 * 32 + 96,)]
    kv = needs[2][0]
    assert needs[4][0] == kv and (kv.n_kv_heads, kv.head_dim, kv.window, kv.sinks) == (1, 48, 37, 0)
    names = {s.name: tuple(s.shape) for s in model.tensor_specs()}
    assert len(names) == len(model.tensor_specs())             # the table that every layer reads is listed once
    assert names["side.embed"] == (131, 80) and names["loop.step"] == (2, 96) and names["l2.side.gate"] == (20, 96)
    assert names["l2.side.proj"] == (96, 20) and names["l2.side.norm"] == (96,)
    assert names["l1.mix.q"] == (48, 96) and names["l1.mix.v"] == (80, 96) and names["l1.mix.g"] == (80, 96) and names["l1.mix.norm"] == (80,)
    assert names["l2.mix.q"] == (96, 96) and names["l2.mix.dkv"] == (48, 96) and names["l2.mix.uk"] == (72, 40) and names["l2.mix.uv"] == (120, 40)
    assert "l2.mix.sink" not in names and "l2.mix.g" not in names
    assert names["l1.mlp.router"] == (5, 96) and names["l1.mlp.e4.down"] == (96, 40) and "l1.mlp.correction" not in names and "l1.mlp.e5.up" not in names
    assert "l3.norm2" not in names and names["l2.norm2"] == (96,) and names["head"] == (131, 96) and names["final.norm"] == (96,)
    assert model.graph_safe and model.spec.logit_softcap == 6.0
    _, model = _model(pc.PEP_B)
    assert [e.layer for e in model.schedule] == [0, 1, 2] * 3 and [e.enter for e in model.schedule][::3] == [(0, 0), (0, 1), (0, 2)]
    assert not any("side" in s.name for s in model.tensor_specs())
    _, model = _model(pc.PEP_D)
    assert [(e.layer, e.enter) for e in model.schedule] == [(0, None), (1, (0, 0))]
    assert not any(s.name == "loop.step" for s in _model(pc.PEP_E)[1].tensor_specs())


def test_sizes_that_only_the_tensors_give():
    cfg = copy.deepcopy(pc.PEP_A)
    del cfg["layers"][0]["mixer"]["decay_rank"]
    typed, model = _model(cfg, shapes={"l0.mix.w1": (9, 96), "l3.mix.w1": (20, 96), "l3.norm2": (96,)})
    assert typed.layers[0].mixer.decay_rank == 9 and typed.layers[3].second_norm
    names = {s.name: tuple(s.shape) for s in model.tensor_specs()}
    assert names["l0.mix.w2"] == (48, 9) and names["l3.norm2"] == (96,)       # a norm that nothing reads may be there


def test_two_parts_that_describe_a_tensor_differently_are_refused():
    _, model = _model(pc.PEP_A)
    model.layers[1].tail.count = 3
    with pytest.raises(ValueError) as e:
        model.tensor_specs()
    assert "side.embed" in str(e.value)


def test_random_models_are_written_and_read_back(tmp_path):
    for name, cfg in pc.ALL.items():
        path = L.write_random_model(str(tmp_path / name), cfg, seed=3)
        got_cfg, tensors = pp.load(path)
        assert got_cfg == cfg
        _, model = _model(cfg)
        assert {s.name: tuple(s.shape) for s in model.tensor_specs()} == {k: v.shape for k, v in tensors.items()}
        logits = pp.forward(got_cfg, tensors, [1, 2, 3, 4, 5])
        assert logits.shape == (5, cfg["vocab"]) and np.isfinite(logits).all()


def test_the_recurrences_segments_cover_every_sequence_in_whole_chunks():
    for lens in ([1], [31], [33, 2], [128], [2048], [2047, 5], [100000]):
        for heads in (1, 4, 32, 400):
            n, length = kernels.decay_segments(lens, heads, 1, n_cus=256)
            assert length % kernels.DECAY_CHUNK == 0 and n * length >= max(lens) > (n - 1) * length
    assert kernels.decay_segments([2048], 400, 2, n_cus=256)[0] == 1 and kernels.decay_segments([2048], 32, 1, n_cus=256)[0] == 16
    p = kernels.decay_powers((0.5, 1.0, 0.999), "cpu")
    assert p.shape == (3, 33) and p[0, 3] == 0.125 and (p[1] == 1.0).all() and abs(float(p[2, 32]) - 0.999 ** 32) < 1e-7


# ---------------------------------------------------------------------------
# the plain implementation's mechanisms against numbers worked by hand
# ---------------------------------------------------------------------------
def test_the_norm_and_the_activations():
    x = np.array([[3.0, -4.0]])
    rms = math.sqrt(12.5 + 0.5)
    assert np.allclose(pp.norm(x, np.array([0.5, -0.25]), 0.5), [[1.5 / rms, 1.0 / rms]])
    assert np.allclose(pp.silu(np.array([1.0, -2.0])), [1.0 / (1.0 + math.exp(-1.0)), -2.0 / (1.0 + math.exp(2.0))])
    z = 0.7
    assert np.allclose(pp.gelu_tanh(np.array([z, 0.0])), [0.5 * z * (1.0 + math.tanh(0.7978845608028654 * (z + 0.044715 * z ** 3))), 0.0])
    assert np.allclose(pp.softcap(np.array([2.0]), 4.0), [4.0 * math.tanh(0.5)]) and np.allclose(pp.softcap(np.array([2.0]), None), [2.0])


def test_the_recurrence_with_a_bonus_by_hand():
    r = np.array([[[1.0, 2.0]], [[3.0, 1.0]]])
    k = np.array([[[1.0, -1.0]], [[2.0, 0.5]]])
    v = np.array([[[10.0, 1.0]], [[20.0, 2.0]]])
    w = np.array([[[0.5, 0.25]], [[0.1, 0.2]]])
    u = np.array([[2.0, 3.0]])
    o, S = pp.wkv_recurrence(r, k, v, w, u)
    assert np.allclose(o[0, 0], (1.0 * 2.0 * 1.0 + 2.0 * 3.0 * -1.0) * v[0, 0])            # from nothing: the bonus alone
    # the state behind token 0 is k v^T as it is (its decay met a state of zero)
    assert np.allclose(o[1, 0], (3.0 * 1.0 + 1.0 * -1.0) * v[0, 0] + (3.0 * 2.0 * 2.0 + 1.0 * 3.0 * 0.5) * v[1, 0])
    assert np.allclose(S[0, 0], 0.1 * 1.0 * v[0, 0] + 2.0 * v[1, 0]) and np.allclose(S[0, 1], 0.2 * -1.0 * v[0, 0] + 0.5 * v[1, 0])


def test_the_recurrence_with_a_fixed_decay_by_hand():
    q = np.array([[[1.0, 2.0]], [[3.0, -1.0]]])
    k = np.array([[[1.0, 0.5]], [[2.0, 1.0]]])
    v = np.array([[[10.0]], [[4.0]]])
    o, S = pp.decay_recurrence(q, k, v, [0.25])
    assert np.allclose(o[:, 0, 0], [(1.0 + 1.0) * 10.0, (3.0 - 0.5) * 0.25 * 10.0 + (6.0 - 1.0) * 4.0])       # a token reads its own product
    assert np.allclose(S[0, :, 0], [0.25 * 10.0 + 8.0, 0.25 * 5.0 + 4.0])
    o2, _ = pp.decay_recurrence(q[1:], k[1:], v[1:], [0.25], np.array([[[10.0], [5.0]]]))
    assert np.allclose(o2[0], o[1])


def test_the_mixes_take_zeros_before_the_first_token():
    h = np.array([[1.0, 2.0], [3.0, 5.0]])
    assert np.allclose(pp.before(h), [[0.0, 0.0], [1.0, 2.0]])


def test_the_rotation_pairs_a_dimension_with_the_one_half_the_rotated_width_on():
    x = np.arange(1.0, 5.0).reshape(1, 1, 4)
    got = pp.rotate(np.repeat(x, 2, axis=0), [0, 1], 4, 100.0)
    assert np.allclose(got[0, 0], [1.0, 2.0, 3.0, 4.0])
    c, s, c2, s2 = math.cos(1.0), math.sin(1.0), math.cos(0.1), math.sin(0.1)
    assert np.allclose(got[1, 0], [c - 3.0 * s, 2.0 * c2 - 4.0 * s2, 3.0 * c + s, 4.0 * c2 + 2.0 * s2])


def test_the_window_counts_the_query_itself():
    p = pp.window_softmax(np.zeros((4, 4)), 2)
    assert np.allclose(p, [[1, 0, 0, 0], [0.5, 0.5, 0, 0], [0, 0.5, 0.5, 0], [0, 0, 0.5, 0.5]])
    assert np.allclose(pp.window_softmax(np.zeros((3, 3)), 1), np.eye(3))
    assert np.allclose(pp.window_softmax(np.log(np.array([[1.0, 1.0], [1.0, 3.0]])), 9), [[1.0, 0.0], [0.25, 0.75]])


def test_the_router_and_the_weight_on_the_input_by_hand():
    h = np.array([[1.0, 2.0]])
    w = np.array([[1.0, 0.0], [0.0, 1.0], [-1.0, 0.0]])
    chosen, weights = pp.route(h, w, 2)
    sg = lambda z: 1.0 / (1.0 + math.exp(-z))
    assert chosen.tolist() == [[1, 0]] and np.allclose(weights, [[sg(2.0), sg(1.0)]])           # not renormed
    t = {"router": w, **{f"e{e}.{n}": np.array([[float(e + 1), 0.5]]) for e in range(3) for n in ("gate", "up")},
         **{f"e{e}.down": np.array([[1.0], [float(e)]]) for e in range(3)}}
    got = pp.mixture(h, t, {"router": {"experts": 3, "top": 2}})
    want = np.zeros(2)
    for e, wt in ((1, sg(2.0)), (0, sg(1.0))):
        a = wt * (float(e + 1) + 1.0)
        want += a * sg(a) * a * np.array([1.0, float(e)])
    assert np.allclose(got, [want])


def test_a_layers_part_of_the_second_embedding_is_its_own_columns_in_every_pass():
    cfg = copy.deepcopy(pc.PEP_D)
    _, model = _model(cfg)
    rng = np.random.default_rng(1)
    t = {s.name: rng.standard_normal(s.shape) * 0.3 for s in model.tensor_specs()}
    one = pp.forward(cfg, t, [3, 4, 5])
    t2 = dict(t, **{"side.embed": t["side.embed"].copy()})
    t2["side.embed"][4, 8:16] += 1.0                           # layer 1's columns of token 4
    two = pp.forward(cfg, t2, [3, 4, 5])
    assert np.allclose(one[0], two[0]) and not np.allclose(one[1], two[1])
    x = rng.standard_normal((2, 48))
    got = pp.token_side(x, np.ones((2, 8)) * 2.0, pp.part(t, "l1.side."), 1e-5)
    y = (pp.gelu_tanh(x @ t["l1.side.gate"].T) * 2.0) @ t["l1.side.proj"].T
    assert np.allclose(got, y / np.sqrt((y ** 2).mean(1, keepdims=True) + 1e-5) * t["l1.side.norm"])


def test_a_pass_gets_its_vector_and_from_the_second_on_the_embedding_output():
    cfg = copy.deepcopy(pc.PEP_B)
    assert pp.runs(cfg) == [(0, 0), (1, None), (2, None), (0, 1), (1, None), (2, None), (0, 2), (1, None), (2, None)]
    assert pp.runs(pc.PEP_A) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    # layers that add nothing (all of their closing matrices zero): what is left are the sums
    _, model = _model(cfg)
    rng = np.random.default_rng(2)
    t = {s.name: rng.standard_normal(s.shape) for s in model.tensor_specs()}
    for k in t:
        if k.endswith((".mix.o", ".down")):
            t[k] = np.zeros_like(t[k])
    streams = []
    pp.forward(cfg, t, [7], streams)
    x0, st = t["embed"][7], t["loop.step"]
    assert np.allclose(streams[2][0], x0 + st[0]) and np.allclose(streams[5][0], 2 * x0 + st[0] + st[1])
    assert np.allclose(streams[8][0], 3 * x0 + st[0] + st[1] + st[2])
