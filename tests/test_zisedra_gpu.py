"""The Zisedra design on the GPU against the plain implementation: every mechanism alone, whole prompts,
prompts cut into portions, token-by-token decoding, unequal batches with slots and pages used again, long
decoding over page borders, windows' edges, states carried over hundreds of tokens, what every part of the design
adds shown to decide, greedy generation through the library's entry point, and the trace runner and the command
line as programs."""
import importlib
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_zisedra as pz
import zisedra_configs as zc
import zisedra_helpers as H

pytestmark = pytest.mark.gpu
L = H.llogos
P = importlib.import_module("daisi-llogos_amd.parts")
K = importlib.import_module("daisi-llogos_amd.ops.kernels")
base = importlib.import_module("daisi-llogos_amd.parts.base")
DEV = torch.device("cuda:0")
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
PART_TOL = {"float32": 3e-5, "bfloat16": 3e-2}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _np(t):
    return t.detach().cpu().double().numpy()


def _f32(a):
    return torch.tensor(np.asarray(a), dtype=torch.float32, device=DEV)


def _i32(a):
    return torch.tensor(np.asarray(a), dtype=torch.int32, device=DEV)


def _rounded(a, dtype):
    """Random inputs as the engine's type holds them, as float64."""
    return np.asarray(torch.tensor(a).to(DT[dtype]).double())


def _ctx(rt, lens, new, slots, ids=None):
    """A step that brings new[i] tokens to sequence i, which is lens[i] long afterwards."""
    B, T = len(lens), sum(new)
    tok_seq = np.repeat(np.arange(B), new).astype(np.int32)
    tok_pos = np.concatenate([np.arange(l - n, l) for l, n in zip(lens, new)]).astype(np.int32)
    cu = np.concatenate([[0], np.cumsum(new)])
    return P.StepContext(runtime=rt, n_tokens=T, batch=B, ids=_i32(np.zeros(T) if ids is None else ids), tok_seq=_i32(tok_seq),
                         tok_pos=_i32(tok_pos), slots=_i32(slots), cu_seqlens=cu.tolist(), starts=[l - n for l, n in zip(lens, new)],
                         slot_ids=list(slots), is_decode=max(new) == 1, max_context=max(lens),
                         cu_dev=None if max(new) == 1 else _i32(cu))


def _steps(lengths, cuts):
    """Cut sequences of `lengths` into steps: cuts[s][i] tokens of sequence i in step s (0: not in the step)."""
    done = [0] * len(lengths)
    for cut in cuts:
        seqs = [i for i, c in enumerate(cut) if c]
        lo = [done[i] for i in seqs]
        for i in seqs:
            done[i] += cut[i]
        yield seqs, lo, [done[i] for i in seqs]
    assert done == list(lengths), "the cuts do not cover the sequences"


def _bind(part, rng, dtype, scale=0.3, scaled=None):
    """Random tensors for a part (stored in bfloat16, as a model folder holds them); returns them as float64."""
    tensors, plain = {}, {}
    lim = {"norm": (0.7, 1.3), "router": (-0.4, 0.4), "a_log": (-2.0, 1.5), "dt_bias": (-4.0, 1.0), "taps": (-0.6, 0.6)}
    for spec in part.tensor_specs():
        if spec.kind in lim:
            t = torch.tensor(rng.uniform(*lim[spec.kind], size=spec.shape), dtype=torch.bfloat16)
        else:
            t = torch.tensor(rng.standard_normal(spec.shape) * scale * (scaled or {}).get(spec.name, 1.0), dtype=torch.bfloat16)
        tensors[spec.name], plain[spec.name] = t, t.double().numpy()
    part.bind(tensors.get, P.Runtime(DEV, DT[dtype]))
    return plain


def _run(eng, slot, toks, lo, hi):
    return eng.step([(slot, list(toks[lo:hi]))], want="all")


PIECES = [(60, 9, 1), (1, 1, 1), (1, 1, 1), (3, 58, 0), (1, 1, 0), (2, 0, 0), (64, 0, 0), (1, 0, 0), (17, 0, 0)]     # of 150, 70 and 3 tokens
WHOLE = [(148, 68, 3), (1, 1, 0), (1, 1, 0)]


def _close(got, want, tol, what=""):
    assert np.isfinite(got).all(), what
    err = np.abs(got - want).max()
    assert err <= tol * max(1.0, np.abs(want).max()), f"{what}: {err:.3e} of {np.abs(want).max():.3e}"


# ---------------------------------------------------------------------------
# mechanisms alone
# ---------------------------------------------------------------------------
# (heads, key heads, key channels, value channels, taps)
RULES = [(4, 2, 24, 40, 4), (3, 3, 10, 18, 1), (1, 1, 16, 16, 2), (2, 1, 64, 128, 4), (3, 1, 128, 64, 3), (1, 1, 256, 200, 4), (5, 1, 3, 7, 6), (2, 2, 33, 5, 4),
         (1, 1, 96, 300, 4), (4, 2, 128, 128, 4), (2, 1, 192, 48, 16), (1, 1, 256, 300, 2), (2, 2, 48, 127, 4)]


def _rule_inputs(shape, channelwise, rng, lengths, parallel_keys=False, fast=True):
    """Projected rows, decays' and gates' inputs of some sequences, and what the plain recurrence makes of them."""
    heads, G, D, V, taps = shape
    W, n_decay = 2 * G * D + heads * V, heads * D if channelwise else heads
    f32 = lambda a: np.asarray(torch.tensor(a, dtype=torch.float32).double())
    conv = f32(rng.uniform(-0.6, 0.6, size=(W, taps)))
    conv[:, -1] += 0.8
    a_log, dt_bias = f32(rng.uniform(-2.0, 1.5, heads)), f32(rng.uniform(-5.0, 1.0, n_decay))
    if fast:                                                    # some decays that leave nothing, some that leave all
        dt_bias[::3] += 40.0
        dt_bias[1::3] -= 20.0
    rows, z, gates, want, ends = [], [], [], [], []
    lean = rng.standard_normal(G * D) * 3.0
    for n in lengths:
        r, zz, g = f32(rng.standard_normal((n, W + heads))), f32(rng.standard_normal((n, n_decay))), f32(rng.standard_normal((n, heads * V)))
        r[:, W:] *= 3.0
        if parallel_keys:
            r[:, G * D:2 * G * D] = f32(r[:, G * D:2 * G * D] * 0.05 + lean)
            r[:, W:] += 6.0
        y = pz.silu(pz.short_conv(r[:, :W], conv))
        of = np.arange(heads) // (heads // G)
        q = (pz.length_one(y[:, :G * D].reshape(n, G, D)) / np.sqrt(D))[:, of]
        k = pz.length_one(y[:, G * D:2 * G * D].reshape(n, G, D))[:, of]
        v = y[:, 2 * G * D:].reshape(n, heads, V)
        dec = np.exp(-np.exp(a_log)[:, None] * pz.softplus(zz + dt_bias).reshape(n, heads, -1)) * np.ones((n, heads, D))
        o, S = pz.delta_recurrence(q, k, v, pz.sigmoid(r[:, W:]), dec)
        rows.append(r); z.append(zz); gates.append(g); want.append(o.reshape(n, -1)); ends.append(S)
    sh = K.DeltaShape(H=heads, G=G, D=D, V=V, taps=taps, channelwise=channelwise, b_col=W)
    return sh, rows, z, gates, conv, a_log, dt_bias, want, ends


def _split(a, rng, parts):
    """A product in `parts` partial sums (float32 views of wider rows), or in one."""
    wide = torch.zeros((parts,) + a.shape[:-1] + (a.shape[-1] + 4,), dtype=torch.float32, device=DEV)
    noise = [_f32(rng.standard_normal(a.shape)) for _ in range(parts - 1)]
    for i, nz in enumerate(noise):
        wide[i, ..., :a.shape[-1]] = nz
    wide[parts - 1, ..., :a.shape[-1]] = _f32(a) - sum(noise, torch.zeros(a.shape, device=DEV))
    wide = wide[..., :a.shape[-1]]
    return wide if parts > 1 else wide[0]


@pytest.mark.parametrize("channelwise", [False, True])
@pytest.mark.parametrize("single", ["step", "chunks"])
@pytest.mark.parametrize("cuts", [PIECES, WHOLE])
@pytest.mark.parametrize("shape", RULES)
def test_the_delta_rule_alone_in_pieces(shape, cuts, single, channelwise):
    """Whole prompts, portions and single tokens (by their own kernel, and by the one for longer steps) against the plain
    recurrence, rows of products in one part and in several; decays of about one and about zero between them; the state and
    the convolution's rows at the end too."""
    heads, G, D, V, taps = shape
    if single == "step" and not K.delta_step_threads(D, V):
        pytest.skip("a head too large for the kernel of single tokens: the other one serves")
    rng = np.random.default_rng(heads * 1000 + D + V + taps)
    lengths, slots = (150, 70, 3), [2, 0, 3]
    sh, rows, z, gates, conv, a_log, dt_bias, want, ends = _rule_inputs(shape, channelwise, rng, lengths)
    state = torch.zeros((5, sh.state_floats), dtype=torch.float32, device=DEV)
    state[[1, 4]] = float("nan")                               # nobody's
    rt = P.Runtime(DEV, torch.float32)
    norm_w, taps_t, eps = rng.uniform(0.5, 1.5, V), _f32(conv.T.copy()), 1e-3
    for silu in (True, False):
        state[slots] = 0.0
        state[slots, heads * D * V:] = float("nan")            # (rows of positions before the first are not read)
        got = [np.zeros((n, heads * V)) for n in lengths]
        for step, (seqs, lo, hi) in enumerate(_steps(lengths, cuts)):
            ctx = _ctx(rt, hi, [b - a for a, b in zip(lo, hi)], [slots[i] for i in seqs])
            cat = lambda arrays: np.concatenate([arrays[i][a:b] for i, a, b in zip(seqs, lo, hi)])
            parts = (1, 3, 6)[step % 3]
            rt_, zt, gt = _split(cat(rows), rng, parts), _split(cat(z), rng, (1, 2)[step % 2]), _split(cat(gates), rng, (2, 1, 5)[step % 3])
            args = (ctx, sh, rt_, taps_t, zt, _f32(dt_bias), _f32(a_log))
            if ctx.is_decode and single == "step":
                y = _np(K.delta_step(*args, gt, silu, _f32(norm_w), eps, state, torch.float32))
            else:
                act, logd, beta = K.delta_prepare(*args, state)
                o = K.delta_scan(ctx, sh, act, logd, beta, state)
                y = _np(K.delta_out(o, gt, silu, _f32(norm_w), eps, heads, torch.float32))
            at = 0
            for i, a, b in zip(seqs, lo, hi):
                got[i][a:b] = y[at:at + b - a]
                at += b - a
        for i, n in enumerate(lengths):
            act_g = pz.silu(gates[i]) if silu else pz.sigmoid(gates[i])
            full = pz.norm(want[i].reshape(n, heads, V), norm_w, eps).reshape(n, -1) * act_g
            _close(got[i], full, 1e-4, f"sequence {i}, silu {silu}")
            S = _np(state[slots[i]])
            _close(S[:heads * D * V].reshape(heads, D, V), ends[i], 2e-5, f"state {i}")
            ring = S[heads * D * V:].reshape(taps, -1)
            for p in range(max(0, n - taps + 1), n):            # (a further row may hold anything)
                assert np.abs(ring[p % taps] - rows[i][p, :sh.width]).max() <= 1e-5


@pytest.mark.parametrize("channelwise", [False, True])
def test_the_delta_rule_with_keys_that_repeat(channelwise):
    """Keys that hardly differ and a strength of almost one: every token must take back what the last one wrote, so a
    recurrence that only added would be another by far, and a chunk's triangular system is at its hardest."""
    rng = np.random.default_rng(5)
    for shape in ((2, 1, 32, 48, 4), (2, 2, 128, 64, 4)):
        heads, G, D, V, taps = shape
        sh, rows, z, gates, conv, a_log, dt_bias, want, ends = _rule_inputs(shape, channelwise, rng, (200,), parallel_keys=True, fast=False)
        dt_bias -= 4.0
        conv[:, :-1] *= 0.2
        y = pz.silu(pz.short_conv(rows[0][:, :sh.width], conv))
        of = np.arange(heads) // (heads // G)
        q = (pz.length_one(y[:, :G * D].reshape(-1, G, D)) / np.sqrt(D))[:, of]
        k = pz.length_one(y[:, G * D:2 * G * D].reshape(-1, G, D))[:, of]
        assert (np.einsum("thd,thd->th", k[1:], k[:-1]) > 0.95).mean() > 0.9
        dec = np.exp(-np.exp(a_log)[:, None] * pz.softplus(z[0] + dt_bias).reshape(200, heads, -1)) * np.ones((200, heads, D))
        o, S = pz.delta_recurrence(q, k, y[:, 2 * G * D:].reshape(-1, heads, V), pz.sigmoid(rows[0][:, sh.width:]), dec)
        for cuts in ([200], [33, 1, 1, 64, 101]):
            state, at, got = torch.zeros((1, sh.state_floats), dtype=torch.float32, device=DEV), 0, []
            for c in cuts:
                ctx = _ctx(P.Runtime(DEV, torch.float32), [at + c], [c], [0])
                pre = K.delta_prepare(ctx, sh, _f32(rows[0][at:at + c]), _f32(conv.T.copy()), _f32(z[0][at:at + c]), _f32(dt_bias), _f32(a_log), state)
                got.append(_np(K.delta_scan(ctx, sh, *pre, state)))
                at += c
            got = np.concatenate(got).reshape(o.shape)
            assert np.abs(got - o).max() <= 1e-4 * np.abs(o).max() and np.abs(_np(state[0, :S.size]).reshape(S.shape) - S).max() <= 1e-4 * np.abs(S).max()


def test_the_delta_rule_carries_a_loud_token_over_hundreds():
    """One token's value is large; 600 tokens later, whose keys leave some of it, it still decides, whatever the cut; without
    it, or with a decay a hundredth off, the result is another by far."""
    rng = np.random.default_rng(8)
    heads, D, V, n = 2, 64, 48, 640
    W = 2 * heads * D + heads * V
    conv = np.zeros((W, 2)); conv[:, 1] = 1.0
    f32 = lambda a: np.asarray(torch.tensor(a, dtype=torch.float32).double())
    rows = f32(rng.standard_normal((n, W + heads)))
    rows[:, :2 * heads * D] += 2.0                             # (silu of these is about the value itself)
    rows[:, W:] = -4.5                                         # weak writes
    rows[20, 2 * heads * D:W] = 400.0
    rows[20, W:] = 6.0
    a_log, dt_bias, z = np.array([-6.0, -7.0]), np.zeros(heads), np.zeros((n, heads))

    def plain(r, dt):
        y = pz.silu(pz.short_conv(r[:, :W], conv))
        q = pz.length_one(y[:, :heads * D].reshape(n, heads, D)) / np.sqrt(D)
        k = pz.length_one(y[:, heads * D:2 * heads * D].reshape(n, heads, D))
        dec = np.exp(-np.exp(a_log)[:, None] * pz.softplus(z + dt).reshape(n, heads, 1)) * np.ones((n, heads, D))
        return pz.delta_recurrence(q, k, y[:, 2 * heads * D:].reshape(n, heads, V), pz.sigmoid(r[:, W:]), dec)[0].reshape(n, -1)

    want = plain(rows, dt_bias)
    size = np.abs(want[600:]).max()
    quiet = rows.copy(); quiet[20, 2 * heads * D:W] = 0.0
    assert np.abs(plain(quiet, dt_bias)[600:] - want[600:]).max() > 0.1 * size
    assert np.abs(plain(rows, dt_bias + 0.05)[600:] - want[600:]).max() > 0.002 * size
    sh = K.DeltaShape(H=heads, G=heads, D=D, V=V, taps=2, channelwise=False, b_col=W)
    gate, ones = torch.full((n, heads * V), 40.0, device=DEV), torch.ones(V, device=DEV)
    for cuts in ([640], [31, 1, 33, 2, 500] + [1] * 73, [600] + [1] * 40):
        state, at, got = torch.zeros((1, sh.state_floats), dtype=torch.float32, device=DEV), 0, []
        for c in cuts:
            ctx = _ctx(P.Runtime(DEV, torch.float32), [at + c], [c], [0])
            args = (ctx, sh, _f32(rows[at:at + c]), _f32(conv.T.copy()), _f32(z[at:at + c]), _f32(dt_bias), _f32(a_log))
            if c == 1:
                got.append(_np(K.delta_step(*args, gate[:1], False, ones, 1e-12, state, torch.float32)))
            else:
                got.append(_np(K.delta_out(K.delta_scan(ctx, sh, *K.delta_prepare(*args, state), state), gate[:c], False, ones, 1e-12, heads, torch.float32)))
            at += c
        normed = pz.unit_rows(want.reshape(n, heads, V), 1e-12).reshape(n, -1)
        assert np.abs(np.concatenate(got)[600:] - normed[600:]).max() <= 6e-4


def test_the_delta_rule_refuses_what_does_not_fit():
    rt = P.Runtime(DEV, torch.float32)
    sh = K.DeltaShape(H=2, G=1, D=8, V=8, taps=3, channelwise=False, b_col=32)
    ctx = _ctx(rt, [4], [4], [0])
    z2 = lambda *s: torch.zeros(s, device=DEV)
    ok = dict(rows=z2(4, 34), conv=z2(3, 32), z=z2(4, 2), dt_bias=z2(2), a_log=z2(2), state=z2(1, sh.state_floats))
    pre = K.delta_prepare(ctx, sh, **ok)
    K.delta_scan(ctx, sh, *pre, ok["state"])
    for name, bad in (("rows", z2(4, 33)), ("rows", z2(3, 34)), ("rows", z2(4, 34).bfloat16()), ("conv", z2(2, 32)), ("conv", z2(3, 31)), ("z", z2(4, 1)),
                      ("dt_bias", z2(3)), ("a_log", z2(1)), ("state", z2(1, sh.state_floats - 1))):
        with pytest.raises(K.KernelError):
            K.delta_prepare(ctx, sh, **dict(ok, **{name: bad}))
    for i, bad in ((0, z2(4, 31)), (1, z2(4, 3)), (2, z2(3, 2))):
        with pytest.raises(K.KernelError):
            K.delta_scan(ctx, sh, *(bad if i == j else t for j, t in enumerate(pre)), ok["state"])
    with pytest.raises(K.KernelError):
        K.delta_step(ctx, sh, *(ok[n] for n in ("rows", "conv", "z", "dt_bias", "a_log")), z2(4, 16), True, z2(8), 1e-5, ok["state"], torch.float32)


@pytest.mark.parametrize("rows", H.DTYPES)
@pytest.mark.parametrize("T,N,pa,pb", [(1, 6, 1, 1), (5, 80, 3, 1), (300, 100, 1, 2), (7, 1024, 2, 11), (2, 5001, 1, 1), (260, 4096, 1, 1)])
def test_two_normed_outputs_join_the_stream(T, N, pa, pb, rows):
    rng = np.random.default_rng(N)
    a, b, x = rng.standard_normal((pa, T, N)) * 3, rng.standard_normal((pb, T, N)) * 0.2, rng.standard_normal((T, N))
    wa, wb, wn = rng.uniform(0.5, 1.5, N), rng.uniform(-1.5, 0.5, N), rng.uniform(0.5, 1.5, N)
    v = pz.norm(a.sum(0), wa, 1e-3) + pz.norm(b.sum(0), wb, 1e-3)
    t = lambda m: _f32(m) if len(m) > 1 else _f32(m[0])
    _close(_np(K.pair_norm(t(a), t(b), _f32(wa), _f32(wb), 1e-3)), v, 1e-5)
    for nxt in (False, True):
        xt = _f32(x)
        h = K.pair_norm(t(a), t(b), _f32(wa), _f32(wb), 1e-3, x=xt, next_w=_f32(wn) if nxt else None, next_eps=0.1, out_dtype=DT[rows])
        _close(_np(xt), x + v, 1e-5)
        assert (h is None) == (not nxt)
        if nxt:
            _close(_np(h), pz.norm(x + v, wn, 0.1), 1e-5 if rows == "float32" else 1e-2)
    if pa == pb == 1:                                          # products that come in bfloat16, one or both
        ab, bb = _f32(a[0]).bfloat16(), _f32(b[0]).bfloat16()
        for one, two in ((ab, bb), (ab, _f32(b[0])), (_f32(a[0]), bb)):
            _close(_np(K.pair_norm(one, two, _f32(wa), _f32(wb), 1e-3)), pz.norm(_np(one), wa, 1e-3) + pz.norm(_np(two), wb, 1e-3), 1e-5)


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("hidden,ff,limit,T", [(48, 33, 0.5, 5), (96, 64, 1.5, 70), (64, 40, 1e9, 3), (128, 96, 0.0, 130), (64, 64, 1.2, 40), (256, 160, 0.8, 16),
                                                  (128, 96, 1.0, 1100), (64, 48, 0.0, 2)])
@pytest.mark.parametrize("fused", [True, False])
def test_the_bounded_feed_forward_alone(hidden, ff, limit, T, fused, dtype, monkeypatch):
    """The bounds in the products' epilogues (few rows, prompts of the tiled product, rows without their norm's scale) and in
    a kernel behind them."""
    monkeypatch.setattr(P.ClampedGLU, "fuse_from", 0 if fused else 1 << 30)
    if dtype == "bfloat16" and fused and ff % 16 == 0 and (T <= 64 or 1024 <= T <= 2048) and hidden % 64 == 0:
        monkeypatch.setattr(K, "clamped_glu", lambda *a, _k=K.clamped_glu: _k(*a) if a[0].shape[-1] == 10 else pytest.fail("not fused"))
    rng = np.random.default_rng(ff)
    mlp = P.ClampedGLU(prefix="f.", hidden=hidden, intermediate=ff, limit=limit)
    plain = _bind(mlp, rng, dtype)
    h = _rounded(rng.standard_normal((T, hidden)), dtype)
    want = pz.clamped_ff(h, pz.part(plain, "f."), limit)
    x = torch.zeros((T, hidden), dtype=torch.float32, device=DEV)
    ht = torch.tensor(h, dtype=DT[dtype], device=DEV)
    _close(_np(K.sum_parts(mlp.forward(None, ht), None, torch.float32)), want, PART_TOL[dtype])
    left = mlp.forward(None, ht, residual=base.Residual(x, None))
    _close(_np(x) if isinstance(left, K.RowSquares) else _np(K.sum_parts(left, None, torch.float32)), want, PART_TOL[dtype])
    if 0.0 < limit < 10.0:                                     # both bounds are met, on the gate only from above
        for other in (limit * 1.1, limit * 0.9):
            assert np.abs(pz.clamped_ff(h, pz.part(plain, "f."), other) - want).max() > 30 * PART_TOL["float32"] * np.abs(want).max()
    if dtype == "bfloat16" and T <= 16 and hidden % 8 == 0 and ff % 16 == 0:
        # behind a product that has added itself to the stream: the norm's rows come without their scale
        before = P.Linear(["w"], 64, [hidden], suffix="")
        nxt = P.RMSNorm(name="n", width=hidden, eps=1e-3, suffix="")
        w = {"w": torch.tensor(rng.standard_normal((hidden, 64)) * 0.3, dtype=torch.bfloat16), "n": torch.tensor(rng.uniform(0.5, 1.5, hidden), dtype=torch.bfloat16)}
        before.bind(w.get, mlp.rt); nxt.bind(w.get, mlp.rt)
        xt = _f32(rng.standard_normal((T, hidden)))
        left = before.add_to(torch.tensor(rng.standard_normal((T, 64)), dtype=torch.bfloat16, device=DEV), base.Residual(xt, nxt))
        rows = nxt.forward(xt, left, lazy=True)
        assert isinstance(rows, base.NormedRows)
        full = pz.clamped_ff(pz.norm(_np(xt), w["n"].double().numpy(), 1e-3), pz.part(plain, "f."), limit)
        _close(_np(K.sum_parts(mlp.forward(None, rows), None, torch.float32)), full, PART_TOL[dtype])
    z = rng.standard_normal((3, 4, 10)) * 3.0
    g, u = np.minimum(z.sum(0)[:, :5], 1.25), np.clip(z.sum(0)[:, 5:], -1.25, 1.25)
    _close(_np(K.clamped_glu(_f32(z), 1.25, DT[dtype])), g * pz.sigmoid(1.702 * g) * (u + 1.0), PART_TOL[dtype])


# (heads, key heads, key channels, value channels, taps, decay rank, gate rank, hidden)
DELTAS = [(4, 2, 24, 40, 4, 0, 0, 56), (3, 1, 10, 18, 1, 5, 3, 72), (1, 1, 16, 16, 2, 8, 0, 40), (2, 1, 64, 128, 4, 0, 12, 64), (4, 4, 128, 128, 4, 16, 16, 96),
          (5, 1, 8, 8, 6, 0, 0, 33), (2, 1, 256, 300, 3, 7, 9, 40)]


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("cuts", [PIECES, WHOLE])
@pytest.mark.parametrize("shape", DELTAS)
def test_the_delta_mixer_alone_in_pieces(shape, cuts, dtype):
    heads, G, D, V, taps, dr, gr, hidden = shape
    rng = np.random.default_rng(heads * 10 + D)
    mix = P.Delta(prefix="m.", hidden=hidden, n_heads=heads, n_kv_heads=G, head_dim=D, v_dim=V, conv_taps=taps, eps=1e-3, decay_rank=dr, gate_rank=gr,
                  gate="sigmoid" if gr else "silu", out_scale=0.4)
    plain = _bind(mix, rng, dtype)
    names = {"q", "k", "v", "q.conv", "k.conv", "v.conv", "b", "A_log", "dt_bias", "norm", "o"} | ({"a1", "a2"} if dr else {"a"}) | ({"g1", "g2"} if gr else {"g"})
    assert set(plain) == {"m." + n for n in names} and mix.kv_spec() is None
    lengths, slots = (150, 70, 3), [1, 3, 0]
    h = [_rounded(rng.standard_normal((n, hidden)), dtype) for n in lengths]
    m = {"heads": heads, "kv_heads": G, "dim": D, "vdim": V}
    want = [0.4 * pz.delta(x, pz.part(plain, "m."), m, 1e-3) for x in h]
    state = torch.zeros((4,) + mix.state_spec().shape, dtype=torch.float32, device=DEV)
    got = _in_pieces(mix, h, lengths, slots, cuts, dtype, lambda seqs: P.LayerCache(state=state))
    for g, w_ in zip(got, want):
        _close(g, w_, (3 if dtype == "bfloat16" else 2) * PART_TOL[dtype])
    with pytest.raises(RuntimeError):
        mix.forward(_ctx(mix.rt, [1], [1], [0]), torch.zeros((1, hidden), dtype=DT[dtype], device=DEV), P.LayerCache())


def _in_pieces(mix, h, lengths, slots, cuts, dtype, cache_of, f32_rows=False):
    got = [np.zeros((n, h[0].shape[1])) for n in lengths]
    for step, (seqs, lo, hi) in enumerate(_steps(lengths, cuts)):
        ctx = _ctx(mix.rt, hi, [b - a for a, b in zip(lo, hi)], [slots[i] for i in seqs])
        rows = torch.tensor(np.concatenate([h[i][a:b] for i, a, b in zip(seqs, lo, hi)]), dtype=torch.float32 if f32_rows else DT[dtype], device=DEV)
        cache = cache_of(seqs)
        if step % 2:                                           # with a stream that the mixer may add itself to
            x = torch.randn(rows.shape, dtype=torch.float32, device=DEV)
            before = x.clone()
            left = mix.forward(ctx, rows, cache, residual=base.Residual(x, None))
            o = _np(x - before) if isinstance(left, (K.RowSquares, base.NormedAhead)) else _np(K.sum_parts(left, None, torch.float32))
            assert isinstance(left, (K.RowSquares, base.NormedAhead)) or torch.equal(x, before)
        else:
            o = _np(K.sum_parts(mix.forward(ctx, rows, cache), None, torch.float32))
        at = 0
        for i, a, b in zip(seqs, lo, hi):
            got[i][a:b] = o[at:at + b - a]
            at += b - a
    return got


# (heads, key/value heads, key width, value width, rotated width, hidden)
ATTENTIONS = [(3, 1, 24, 40, 12, 56), (2, 2, 12, 20, 0, 72), (4, 2, 64, 64, 32, 64), (4, 1, 96, 128, 96, 64), (2, 1, 128, 128, 64, 96), (6, 2, 128, 64, 16, 40), (3, 3, 8, 8, 8, 33),
              (4, 4, 64, 80, 2, 48), (2, 1, 48, 48, 24, 64)]
WINDOWS = [0, 1, 2, 37, 63, 64, 65, 66, 100, 400]


def _attention(shape, window, dtype, rng, scale=None, scaling=None):
    heads, kv, d, dv, rot, hidden = shape
    scale = scale or 4.0 / (0.09 * hidden * np.sqrt(d))        # scores that spread over some units whatever the sizes
    pos = P.Rotary(d, rot, 300.0, pairing="interleaved", scaling=scaling) if rot else None
    mix = P.Attention(prefix="m.", hidden=hidden, n_heads=heads, n_kv_heads=kv, head_dim=d, v_dim=dv, position=pos, bias=True, scale=scale, window=window,
                      names=("q", "k", "v", "o"), suffix="", bias_suffix=".b")
    plain = _bind(mix, rng, dtype, scaled={f"m.{n}.b": 3.0 for n in "qkv"})
    m = {"heads": heads, "kv_heads": kv, "dim": d, "vdim": dv, "scale": scale, "mask": {"size": window or 10 ** 9}}
    if rot:
        m["rot"] = {"dims": rot, "base": 300.0}
        if scaling:
            m["rot"]["scaling"] = {"factor": scaling["factor"], "low": scaling["low_freq_factor"], "high": scaling["high_freq_factor"],
                                   "original": scaling["original_max_position_embeddings"]}
    return mix, plain, m


def _pools(mix, pages, dtype):
    spec = mix.kv_spec()
    k = torch.full((pages, spec.n_kv_heads, 64 * spec.head_dim), float("nan"), dtype=DT[dtype], device=DEV)
    v = torch.full((pages, spec.n_kv_heads, 64 * spec.value_dim), float("nan"), dtype=DT[dtype], device=DEV)
    # (a head whose size is rounded up in the pages: what lies behind it is never read)
    return k, v


class _Pages:
    """Pages of three sequences in any order; as soon as no later query can see a page its place in the table is taken
    away, as the cache does."""

    def __init__(self, window):
        self.window, self.seen, self.pages = window, [0, 0, 0], {0: [7, 2, 5], 1: [0, 8], 2: [3]}

    def table(self, seqs, new_lens):
        table = np.full((len(seqs), 3), -1, dtype=np.int32)
        for row, i in enumerate(seqs):
            for j, p in enumerate(self.pages[i]):
                if not self.window or 64 * j + 63 > self.seen[i] - self.window:
                    table[row, j] = p
        for i, n in zip(seqs, new_lens):
            self.seen[i] = n
        return _i32(table)


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("cuts", [PIECES, WHOLE])
@pytest.mark.parametrize("shape", ATTENTIONS)
@pytest.mark.parametrize("window", WINDOWS)
def test_the_window_attention_alone_in_pieces(window, shape, cuts, dtype, monkeypatch):
    """Pages in any order that start as NaN.  Head shapes that the matrix cores take must run there, prompts and single
    tokens."""
    heads, kv, d, dv, rot, hidden = shape
    rng = np.random.default_rng(heads * 10 + d + window)
    mix, plain, m = _attention(shape, window, dtype, rng, scaling=SCALING if rot > 2 else None)
    assert mix.kv_spec().window == window
    if dtype == "bfloat16" and d in (64, 96, 128) and dv in (64, 80, 128):
        monkeypatch.setattr(K, "attention_generic", lambda *a, **k: pytest.fail("the kernel for any shape ran"))
    lengths = (150, 70, 3)
    h = [_rounded(rng.standard_normal((n, hidden)), dtype) for n in lengths]
    want = [pz.window_attention(x, pz.part(plain, "m."), m) for x in h]
    k_pool, v_pool = _pools(mix, 9, dtype)
    pages = _Pages(window)
    got = [np.zeros((n, hidden)) for n in lengths]
    for seqs, lo, hi in _steps(lengths, cuts):
        ctx = _ctx(mix.rt, hi, [b - a for a, b in zip(lo, hi)], [0, 1, 2][:len(seqs)])
        rows = torch.tensor(np.concatenate([h[i][a:b] for i, a, b in zip(seqs, lo, hi)]), dtype=DT[dtype], device=DEV)
        o = _np(K.sum_parts(mix.forward(ctx, rows, P.LayerCache(k_pool=k_pool, v_pool=v_pool, table=pages.table(seqs, hi))), None, torch.float32))
        at = 0
        for i, a, b in zip(seqs, lo, hi):
            got[i][a:b] = o[at:at + b - a]
            at += b - a
    for i, (g, w_) in enumerate(zip(got, want)):
        _close(g, w_, (2 if dtype == "bfloat16" else 1) * PART_TOL[dtype], f"sequence {i}")
    for n in "qkv":                                            # every bias shows
        t = dict(pz.part(plain, "m."))
        t[n + ".b"] = np.zeros_like(t[n + ".b"])
        if not (n == "k" and not rot or window == 1 and n in "qk"):      # (without a rotation a key's bias moves all scores of a query alike)
            assert np.abs(pz.window_attention(h[0], t, m) - want[0]).max() > 30 * PART_TOL["float32"] * np.abs(want[0]).max(), n


SCALING = {"type": "llama3", "factor": 4.0, "low_freq_factor": 1.0, "high_freq_factor": 4.0, "original_max_position_embeddings": 200}


@pytest.mark.parametrize("window", [40, 64, 65, 129, 150])
@pytest.mark.parametrize("shape", [(2, 1, 64, 64, 16, 64), (2, 2, 96, 80, 16, 64), (2, 1, 24, 40, 8, 64)])
def test_a_key_at_the_windows_edge_decides(window, shape):
    """A loud token's key stands out for every query that sees it: the last one that does and the first that does not are
    told apart in a prompt, behind a portion's start and in decoding (a window one longer or shorter is another result by a
    hundred times the bound there)."""
    rng = np.random.default_rng(window)
    heads, kv, d, dv, rot, hidden = shape
    mix, plain, m = _attention(shape, window, "float32", rng, scale=0.05)
    t = dict(pz.part(plain, "m."))
    loud, n = 50, 50 + window + 20
    h = rng.standard_normal((n, hidden))
    h[loud] *= 2.0
    bias = rng.standard_normal(hidden)
    bias /= np.linalg.norm(bias)
    h += bias * 6.0
    key = (h[loud] @ t["k"].T + t["k.b"]).reshape(kv, d)
    q = t["q"].reshape(heads, d, hidden).copy()
    for hd in range(heads):                                    # every query leans towards the loud token's key where nothing is rotated
        kk = key[hd // (heads // kv)].copy()
        kk[:rot] = 0.0
        q[hd] += np.outer(kk / np.linalg.norm(kk) * 12.0, bias)
    t["q"] = q.reshape(-1, hidden)
    t = {k_: _rounded(v_, "bfloat16") for k_, v_ in t.items()}
    h = _rounded(h, "bfloat16")
    want = pz.window_attention(h, t, m)
    last = loud + window - 1                                   # the last query that sees the loud key
    size = np.abs(want).max()
    for by, row in ((-1, last), (1, last + 1)):
        other = pz.window_attention(h, t, dict(m, mask={"size": window + by}))
        assert np.abs(other[row] - want[row]).max() > 100 * PART_TOL["float32"] * size
    for dtype in H.DTYPES:
        mix.bind({"m." + k_: torch.tensor(v_, dtype=torch.bfloat16) for k_, v_ in t.items()}.get, P.Runtime(DEV, DT[dtype]))
        for first in (n, last, last + 1, last - 1, 128):       # all in the prompt; a portion or single tokens from the edge on
            for tail in ("portion", "single"):
                k_pool, v_pool = _pools(mix, 6, dtype)
                table = _i32([[4, 1, 0, 5, 2, 3]])
                cuts = [(0, first)] + ([(first, n)] if tail == "portion" else [(a, a + 1) for a in range(first, n)]) if first < n else [(0, n)]
                got = []
                for lo, hi in cuts:
                    cache = P.LayerCache(k_pool=k_pool, v_pool=v_pool, table=table)
                    got.append(_np(K.sum_parts(mix.forward(_ctx(mix.rt, [hi], [hi - lo], [0]), torch.tensor(h[lo:hi], dtype=DT[dtype], device=DEV), cache),
                                               None, torch.float32)))
                err = np.abs(np.concatenate(got) - want).max(axis=1)
                assert err.max() <= (PART_TOL[dtype] if dtype == "float32" else 0.1) * size, f"{dtype} from {first} on, {tail}: worst at {err.argmax()}"


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("kind", ["rms", "layer", "none"])
@pytest.mark.parametrize("hidden", [56, 96, 257])
def test_two_mixers_side_by_side_alone_in_pieces(hidden, kind, dtype):
    """With and without a stream to join, whatever norm reads it next."""
    rng = np.random.default_rng(hidden)
    left = dict(prefix="m.left.", hidden=hidden, n_heads=2, n_kv_heads=1, head_dim=24, v_dim=40, position=P.Rotary(24, 8, 100.0, pairing="interleaved"), bias=True,
                scale=0.05, window=50, names=("q", "k", "v", "o"), suffix="", bias_suffix=".b")
    right = dict(prefix="m.right.", hidden=hidden, n_heads=3, n_kv_heads=1, head_dim=16, v_dim=20, conv_taps=3, eps=1e-3, decay_rank=5, gate_rank=7, gate="sigmoid")
    mix = P.SideBySide(hidden=hidden, left=("attention", left), right=("delta", right), left_norm="m.left.out", right_norm="m.right.out", eps=1e-3, out_scale=0.6)
    assert mix.cache_parts() == [mix.left, mix.right] and mix.graph_safe and mix.kv_spec() is None and mix.state_spec() is None
    plain = _bind(mix, rng, dtype)
    m = {"left": {"heads": 2, "kv_heads": 1, "dim": 24, "vdim": 40, "scale": 0.05, "mask": {"size": 50}, "rot": {"base": 100.0, "dims": 8}},
         "right": {"heads": 3, "kv_heads": 1, "dim": 16, "vdim": 20}}
    lengths, slots = (150, 70, 3), [1, 3, 0]
    h = [_rounded(rng.standard_normal((n, hidden)), dtype) for n in lengths]
    want = [0.6 * pz.side_by_side(x, pz.part(plain, "m."), m, 1e-3) for x in h]
    nxt = {"rms": P.RMSNorm(name="n", width=hidden, eps=0.1, suffix=""), "layer": P.LayerNorm(name="n", width=hidden, eps=1e-5, suffix=""), "none": None}[kind]
    nw = _bind(nxt, rng, dtype)["n"] if nxt is not None else None
    state = torch.zeros((4,) + mix.right.state_spec().shape, dtype=torch.float32, device=DEV)
    k_pool, v_pool = _pools(mix.left, 9, dtype)
    pages = _Pages(50)
    tol = (2 if dtype == "bfloat16" else 1) * PART_TOL[dtype]
    for seqs, lo, hi in _steps(lengths, PIECES):
        ctx = _ctx(mix.rt, hi, [b - a for a, b in zip(lo, hi)], [slots[i] for i in seqs])
        cat = lambda arrays: np.concatenate([arrays[i][a:b] for i, a, b in zip(seqs, lo, hi)])
        rows = torch.tensor(cat(h), dtype=DT[dtype], device=DEV)
        caches = [P.LayerCache(k_pool=k_pool, v_pool=v_pool, table=pages.table(seqs, hi)), P.LayerCache(state=state)]
        if nxt is None:
            _close(_np(mix.forward(ctx, rows, caches)), cat(want), tol)
            continue
        x = rng.standard_normal(rows.shape)
        xt = _f32(x)
        left_over = mix.forward(ctx, rows, caches, residual=base.Residual(xt, nxt))
        full = x + cat(want)
        _close(_np(xt), full, tol)
        if kind == "rms":
            assert isinstance(left_over, base.NormedAhead) and left_over.norm is nxt and nxt.forward(xt, left_over) is left_over.rows
            _close(_np(left_over.rows), pz.norm(full, nw, 0.1), 2 * tol)
        else:
            assert isinstance(left_over, K.RowSquares) and left_over.unscaled is None


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("name", ["zis_a", "zis_c"])
def test_the_second_stream_changes_no_bit(name, dtype, monkeypatch):
    """Replayed and launched, whether the left mixer runs beside the right one or in front of it."""
    outs = []
    monkeypatch.setattr(P.SideBySide, "side_bytes", 0)
    for rows in (64, 0):
        monkeypatch.setattr(P.SideBySide, "side_rows", rows)
        for graphs in (True, False):
            eng = H.engine(name, dtype, use_graphs=graphs)
            a, b = eng.alloc_slot(), eng.alloc_slot()
            toks = H.tokens(name, 140, 13)
            got = [_np(eng.step([(a, list(toks[:60])), (b, list(toks[70:75]))], want="all"))]
            for t in range(60):
                got.append(_np(eng.step([(a, [toks[60 + t]]), (b, [toks[75 + t]])], want="all")))
            outs.append(np.concatenate(got))
    assert all(np.array_equal(o, outs[0]) for o in outs[1:])


@pytest.mark.parametrize("block", ["pre_norm", "sandwich", "parallel", "post_norm", "output_norm"])
def test_every_block_hands_a_pair_of_mixers_their_own_caches(block):
    """A mixer made of two asks the cache for two units, in whatever block it stands."""
    W = 32
    n = lambda name: ("norm", "rmsnorm", dict(name=name, width=W, eps=1e-5, suffix=""))
    rec = lambda p: ("delta", dict(prefix=p, hidden=W, n_heads=2, n_kv_heads=1, head_dim=8, v_dim=12, conv_taps=2, eps=1e-5))
    pair = ("side_by_side", dict(hidden=W, left=rec("l."), right=rec("r."), left_norm="lo", right_norm="ro", eps=1e-5))
    more = {"pre_norm": ["mixer_norm"], "sandwich": ["mixer_norm", "post_mixer_norm"], "parallel": ["mixer_norm"], "post_norm": ["mixer_norm"],
            "output_norm": ["mixer_norm"]}[block]
    mod = importlib.import_module("daisi-llogos_amd.models.model")
    layer = mod.LayerSpec(mixer=pair, block=block, more={k: n(k) for k in more})
    model = mod.Model(mod.ModelSpec(vocab_size=20, hidden_size=W, embed_name="e", layers=[layer], final_norm=n("f")[1:], head_name="head"))
    assert len(model.cache_needs()) == 2 and all(needs[1] is not None for needs in model.cache_needs())
    rng = np.random.default_rng(3)
    tensors = {s.name: torch.tensor(rng.standard_normal(s.shape) * 0.3, dtype=torch.float32) for s in model.tensor_specs()}
    model.bind(tensors.get, P.Runtime(DEV, torch.float32))
    blk = model.layers[0]
    outs = []
    for cuts in ([9], [4, 1, 1, 3]):
        caches = [P.LayerCache(state=torch.zeros((2,) + m.state_spec().shape, device=DEV)) for m in blk.cache_parts()]
        x_all = np.random.default_rng(4).standard_normal((9, W))
        at, got = 0, []
        for c in cuts:
            x, p = blk.forward(_ctx(model.rt, [at + c], [c], [1]), _f32(x_all[at:at + c]), None, caches)
            got.append(_np(x) + (_np(K.sum_parts(p, None, torch.float32)) if isinstance(p, torch.Tensor) else 0.0))
            at += c
        outs.append(np.concatenate(got))
    _close(outs[1], outs[0], 3e-5)


@pytest.mark.parametrize("experts,top,count,keep,K_,T", [(8, 2, 4, 2, 96, 9), (6, 3, 2, 1, 72, 70), (9, 4, 3, 2, 40, 5), (64, 8, 8, 3, 256, 65), (4, 2, 4, 3, 16, 30), (300, 20, 30, 7, 64, 3),
                                                         (5, 2, 1, 1, 48, 20), (8, 3, 4, 4, 48, 20)])
@pytest.mark.parametrize("rows", H.DTYPES)
def test_the_routers_choice_within_groups_by_their_two_largest(experts, top, count, keep, K_, T, rows):
    rng = np.random.default_rng(experts + top)
    h, w = _rounded(rng.standard_normal((T, K_)), rows), _rounded(rng.uniform(-0.4, 0.4, size=(experts, K_)), "float32")
    s = pz.sigmoid(h @ w.T)
    want_c = np.stack([pz.choose(s[i], top, count, keep) for i in range(T)])
    got_c, got_w = K.moe_router(torch.tensor(h, dtype=DT[rows], device=DEV), _f32(w), None, count, keep, top, 0.7, scores="sigmoid", renorm=False,
                                group_score="best_two")
    got_c, got_w = got_c.cpu().numpy(), _np(got_w)
    same = (got_c == want_c).all(axis=1)                       # (a row whose choice hangs on the last bits of two scores is left out)
    assert same.sum() >= T - max(1, T // 50)
    assert np.abs(got_w - 0.7 * np.take_along_axis(s, want_c, axis=1))[same].max() <= 1e-5
    if 1 < count and keep < count and experts // count > 1 and T > 20:      # the groups' largest alone would choose otherwise
        one_c, _ = K.moe_router(torch.tensor(h, dtype=DT[rows], device=DEV), _f32(w), None, count, keep, top, 0.7, scores="sigmoid", renorm=False)
        assert (one_c.cpu().numpy() != got_c).any()
    with pytest.raises(K.KernelError):
        K.moe_router(torch.tensor(h, dtype=DT[rows], device=DEV), _f32(w), None, count, keep, top, 1.0, group_score="best_three")


@pytest.mark.parametrize("dtype,form", [("float32", "auto"), ("bfloat16", "auto"), ("bfloat16", "plain"), ("bfloat16", "few"), ("bfloat16", "tiles64"), ("bfloat16", "tiles128")])
@pytest.mark.parametrize("experts,top,groups,ff,limit,shared,hidden,T", [
    (6, 1, (3, 2), 40, 1.0, (56, 0.5), 96, 9), (1, 1, None, 16, 0.6, None, 32, 3), (4, 4, None, 24, 1.2, (24, 1.2), 48, 70), (8, 3, (4, 2), 72, 2.0, (40, 1.0), 64, 300),
    (16, 1, (4, 1), 96, 1.5, None, 128, 1), (3, 2, None, 132, 1.0, (16, 3.0), 200, 150), (2, 1, (2, 1), 30, 0.5, (33, 0.8), 36, 40)])
def test_the_mixture_of_bounded_experts_alone(dtype, form, experts, top, groups, ff, limit, shared, hidden, T, monkeypatch):
    """Every form of the experts' product; the shared expert's own width and bound; the factor on the output; as a tensor
    and added to a stream.  Another bound would be another result."""
    monkeypatch.setattr(K, "MOE_PRODUCT", form)
    rng = np.random.default_rng(experts * 10 + top)
    more = dict(shared_intermediate=shared[0], shared_limit=shared[1]) if shared else {}
    if groups:
        more.update(groups=groups[0], keep=groups[1])
    part = P.RoutedMoE(prefix="f.", hidden=hidden, n_experts=experts, top=top, intermediate=ff, correction=False, scores="sigmoid", renorm=False,
                       group_score="best_two", limit=limit, out_scale=0.3, **more)
    plain = _bind(part, rng, dtype)
    h = _rounded(rng.standard_normal((T, hidden)), dtype)
    t = pz.part(plain, "f.")
    entry = zc.moe(experts, top, ff, limit, groups, shared)
    want = 0.3 * pz.mixture(h, t, entry)
    s = pz.sigmoid(h @ t["router"].T)
    chosen = np.stack([pz.choose(s[i], top, *(groups or (1, 1))) for i in range(T)])
    ht = torch.tensor(h, dtype=DT[dtype], device=DEV)
    got_c, _ = K.moe_router(ht, part.router_w, None, part.groups, part.keep, top, 1.0, scores="sigmoid", renorm=False, group_score="best_two")
    same = (got_c.cpu().numpy() == chosen).all(axis=1)
    assert same.sum() >= T - max(1, T // 50)
    got = _np(part.forward(None, ht))
    assert np.isfinite(got).all() and np.abs(got - want)[same].max() <= PART_TOL[dtype] * max(1.0, np.abs(want).max())
    for other in (dict(entry, expert={"ff": ff, "limit": limit * 1.2}),) + ((dict(entry, shared={"ff": shared[0], "limit": shared[1] * 1.2}),) if shared else ()):
        assert np.abs(0.3 * pz.mixture(h, t, other) - want).max() > 30 * PART_TOL["float32"] * np.abs(want).max()
    x = torch.randn((T, hidden), dtype=torch.float32, device=DEV)
    xt = x.clone()
    left = part.forward(None, ht, residual=base.Residual(xt, None))
    assert isinstance(left, K.RowSquares) and np.abs(_np(xt) - (_np(x) + got)).max() <= 1e-5 * max(1.0, np.abs(got).max())


@pytest.mark.parametrize("dtype", H.DTYPES)
def test_the_loops_entry_without_vectors(dtype):
    rng = np.random.default_rng(1)
    part = P.LoopEntry(matrix="in", steps=None, width=24, times=2)
    w = _bind(part, rng, dtype)
    assert set(w) == {"in"}
    x, x0, d = (_rounded(rng.standard_normal((5, 24)), dtype) for _ in range(3))
    for number in range(2):
        for delta in (None, d):
            full = x + (0 if delta is None else d)
            out, left = part.forward(None, _f32(x), None if delta is None else _f32(delta), _f32(x0), number)
            assert left is None and out.dtype == torch.float32
            _close(_np(out), np.concatenate([full, x0], axis=1) @ w["in"].T, 2 * PART_TOL[dtype])
        half = _f32(d).bfloat16()                              # what the stream still lacks may come in the matrices' type
        out, _ = part.forward(None, _f32(x), half, _f32(x0), number)
        _close(_np(out), np.concatenate([x + _np(half), x0], axis=1) @ w["in"].T, 2 * PART_TOL[dtype])


# ---------------------------------------------------------------------------
# whole models
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("name", list(zc.ALL))
def test_a_whole_prompt_then_the_rest_token_by_token(name, dtype):
    toks = H.tokens(name, 250, 1)
    want = H.plain_logits(name, toks, dtype=dtype)
    eng = H.engine(name, dtype)
    s = eng.alloc_slot()
    got = [_np(_run(eng, s, toks, 0, 180))]
    for t in range(180, 250):                                   # over a page's border
        got.append(_np(_run(eng, s, toks, t, t + 1)))
    H.close(np.concatenate(got), want, dtype, f"{name} prompt and decoding")


@pytest.mark.parametrize("name", list(zc.ALL))
def test_the_residual_stream_after_every_layer_run(name):
    toks = H.tokens(name, 40, 6)
    cfg, w = H.plain(name)
    want = []
    pz.forward(cfg, w, list(toks), want)
    eng = H.engine(name, "float32", use_graphs=False)
    got = []
    for blk in eng.model.layers:
        def wrapped(ctx, x, pending, caches, _o=blk.forward, **kw):
            x, p = _o(ctx, x, pending, caches, **kw)
            got.append(_np(x) + (_np(K.sum_parts(p, None, torch.float32)) if isinstance(p, torch.Tensor) else 0.0))
            return x, p
        blk.forward = wrapped
    _run(eng, eng.alloc_slot(), toks, 0, 40)
    assert len(got) == len(want) == len(pz.runs(cfg))
    for i, (g, w_) in enumerate(zip(got, want)):
        assert np.abs(g - w_).max() <= 5e-5 * np.abs(w_).max(), f"run {i}"


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("name", list(zc.ALL))
def test_the_first_tokens_one_by_one_and_portions_down_to_two_tokens(name, dtype):
    toks = H.tokens(name, 140, 2)
    want = H.plain_logits(name, toks, dtype=dtype)
    eng = H.engine(name, dtype, n_slots=2)
    a, b = eng.alloc_slot(), eng.alloc_slot()
    one = np.concatenate([_np(_run(eng, a, toks, t, t + 1)) for t in range(70)])          # from the very first token on
    H.close(one, want[:70], dtype, "token by token from the start")
    cuts, at, got = [2, 3, 59, 1, 2, 64, 7, 2], 0, []
    for c in cuts:
        got.append(_np(_run(eng, b, toks, at, at + c)))
        at += c
    H.close(np.concatenate(got), want, dtype, "portions")
    if dtype == "float32":                                      # in 32-bit a row's arithmetic hardly depends on the cut
        assert np.abs(np.concatenate(got)[:70] - one).max() <= 5e-5 * np.abs(want).max()


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("name", ["zis_a", "zis_b", "zis_c"])
def test_unequal_batches_against_each_alone_with_slots_and_pages_used_again(name, dtype):
    eng = H.engine(name, dtype, max_tokens=448, n_slots=3)              # 7 pages: the second batch needs the first one's
    for turn, lens in enumerate([(130, 9, 70), (200, 3, 66)]):
        seqs = [H.tokens(name, n + 6, 10 * turn + i) for i, n in enumerate(lens)]
        slots = [eng.alloc_slot() for _ in seqs]
        assert slots == [0, 1, 2]
        got = [[] for _ in seqs]
        out = _np(eng.step([(s, list(t[:n])) for s, t, n in zip(slots, seqs, lens)], want="all"))
        at = 0
        for i, n in enumerate(lens):
            got[i].append(out[at:at + n])
            at += n
        live = [0, 1, 2]
        for step in range(6):
            if step == 3:                                       # the shortest request ends earlier
                eng.free_slot(slots[1])
                live = [0, 2]
            out = _np(eng.step([(slots[i], [seqs[i][lens[i] + step]]) for i in live], want="all"))
            for j, i in enumerate(live):
                got[i].append(out[j:j + 1])
        for i in live:
            eng.free_slot(slots[i])
        for i, t in enumerate(seqs):
            g = np.concatenate(got[i])
            H.close(g, H.plain_logits(name, t, dtype=dtype)[:len(g)], dtype, f"{name} batch {turn} sequence {i}")
    assert eng.cache.free_pages() == [7] * len(eng.cache.groups)


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("name", ["zis_a", "zis_b", "zis_c"])
def test_long_decoding_replayed_and_launched(name, dtype):
    toks = H.tokens(name, 210, 3)
    want = H.plain_logits(name, toks, dtype=dtype)
    outs = {}
    for graphs in (True, False):
        eng = H.engine(name, dtype, use_graphs=graphs)
        assert (eng.graphs is not None) == graphs
        s = eng.alloc_slot()
        got = [_np(_run(eng, s, toks, 0, 5))] + [_np(_run(eng, s, toks, t, t + 1)) for t in range(5, 210)]
        outs[graphs] = np.concatenate(got)
        H.close(outs[graphs], want, dtype, f"long decoding, graphs {graphs}")
        free = eng.cache.free_pages()
        windows = [g.spec.window for g in eng.cache.groups]
        for n, w_ in zip(free, windows):                        # pages behind the window have been given back
            assert n >= eng.cache.n_pages - ((w_ + 62) // 64 + 2)
    assert np.array_equal(outs[True], outs[False])              # a replayed step is the launched step


def test_what_the_design_is_made_of_decides_and_is_there():
    """Left out of the plain implementation one by one, every mechanism moves the logits of late positions by many times
    the bound; the engine agrees with the plain implementation that has them all."""
    name = "zis_c"
    cfg, w = H.plain(name)
    toks = H.tokens(name, 420, 4)
    want = H.plain_logits(name, toks)

    def config(change):
        c = json.loads(json.dumps(cfg))
        for L_ in c["layers"]:
            change(L_)
        return pz.forward(c, w, list(toks))

    def left(fn):
        return config(lambda L_: fn(L_["mixer"]["left"]) if L_["type"] == "parallel" else None)

    def weights(fn):
        return pz.forward(cfg, {k: fn(k, v) for k, v in w.items()}, list(toks))

    others = {
        "window + 1": left(lambda m: m["mask"].update(size=m["mask"]["size"] + 1)), "window - 1": left(lambda m: m["mask"].update(size=m["mask"]["size"] - 1)),
        "base": left(lambda m: m["rot"].update(base=m["rot"]["base"] * 1.5)), "stretching": left(lambda m: m["rot"].pop("scaling", None)),
        "scale": left(lambda m: m.update(scale=m["scale"] * 1.02)), "all rotated": left(lambda m: m["rot"].update(dims=m["dim"])),
        "groups": config(lambda L_: L_["mlp"] and L_["mlp"]["router"].pop("groups")), "limit": config(lambda L_: L_["mlp"] and L_["mlp"]["expert"].update(limit=1e9)),
        "shared limit": config(lambda L_: L_["mlp"] and "shared" in L_["mlp"] and L_["mlp"]["shared"].update(limit=1e9)),
        "shared": config(lambda L_: L_["mlp"] and L_["mlp"].pop("shared", None)), "factor": pz.forward(dict(cfg, residual_mult=1.0), w, list(toks)),
        "biases": weights(lambda k, v: v * 0 if k.endswith((".q.b", ".k.b", ".v.b")) else v), "decays": weights(lambda k, v: v + 0.2 if k.endswith("dt_bias") else v),
        "first tap": weights(lambda k, v: np.concatenate([v[:, :1] * 0, v[:, 1:]], axis=1) if k.endswith(".conv") else v),
        "x0": weights(lambda k, v: np.concatenate([v[:, :len(v)], v[:, len(v):] * 0], axis=1) if k == "loop.in" else v),
        "norms side by side": weights(lambda k, v: v * 0 + 1 if k.endswith(".out") else v),
    }
    keep = {n: getattr(pz, n) for n in ("delta", "delta_recurrence", "length_one", "short_conv", "choose")}
    try:
        pz.delta = lambda h, *a: np.concatenate([keep["delta"](h[:300], *a), keep["delta"](h[300:], *a)])            # a state lost at position 300
        others["state"] = pz.forward(cfg, w, list(toks))
        pz.delta = keep["delta"]

        def before_the_write(q, k, v, beta, g, S=None):        # a read-out that does not see the token's own write
            S, out = np.zeros((q.shape[1], q.shape[2], v.shape[2])), np.zeros(v.shape)
            for t in range(len(q)):
                S = g[t][:, :, None] * S
                out[t] = np.einsum("hij,hi->hj", S, q[t])
                S = S + k[t][:, :, None] * (beta[t][:, None] * (v[t] - np.einsum("hij,hi->hj", S, k[t])))[:, None, :]
            return out, S
        pz.delta_recurrence = before_the_write
        others["own write"] = pz.forward(cfg, w, list(toks))

        def only_added(q, k, v, beta, g, S=None):              # nothing is taken back
            S, out = np.zeros((q.shape[1], q.shape[2], v.shape[2])), np.zeros(v.shape)
            for t in range(len(q)):
                S = g[t][:, :, None] * S + k[t][:, :, None] * (beta[t][:, None] * v[t])[:, None, :]
                out[t] = np.einsum("hij,hi->hj", S, q[t])
            return out, S
        pz.delta_recurrence = only_added
        others["taking back"] = pz.forward(cfg, w, list(toks))
        pz.delta_recurrence = keep["delta_recurrence"]
        pz.length_one = lambda x: x
        others["unit vectors"] = pz.forward(cfg, w, list(toks))
        pz.length_one = keep["length_one"]
        pz.short_conv = lambda x, taps: keep["short_conv"](x, taps[:, ::-1])
        others["order of the taps"] = pz.forward(cfg, w, list(toks))
        pz.short_conv = keep["short_conv"]
    finally:
        for n, fn in keep.items():
            setattr(pz, n, fn)
    for what, other in others.items():
        assert H.distance(other[300:], want[300:]) > 10 * H.TOL["float32"], what
    for dt in H.DTYPES:
        eng = H.engine(name, dt)
        s = eng.alloc_slot()
        got = [_np(_run(eng, s, toks, 0, 300))] + [_np(_run(eng, s, toks, t, t + 1)) for t in range(300, 420)]
        H.close(np.concatenate(got), H.plain_logits(name, toks, dtype=dt), dt, "everything there")


def test_greedy_generation_through_the_entry_point():
    name = "zis_a"
    cfg, w = H.plain(name)
    prompts = [list(H.tokens(name, 9, 7)), list(H.tokens(name, 60, 8)), list(H.tokens(name, 2, 9))]
    llm = L.Llogos(H.folder(name), dtype="float32", max_context=128, max_batch=2)        # three requests, two at a time
    out = llm.generate(prompts, L.GenerationParams.greedy(max_tokens=10, stop_tokens=()))
    for p, got in zip(prompts, out.tokens):
        assert got == pz.generate_greedy(cfg, w, p, 10)
    assert out.finish_reasons == ["length"] * 3


@pytest.mark.parametrize("dtype", H.DTYPES)
def test_the_trace_runner_on_a_model_of_the_design(tmp_path, dtype):
    name = "zis_a"
    vocab = zc.ALL[name]["vocab"]
    a, b = H.tokens(name, 75, 11), H.tokens(name, 12, 12)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:70], "want": [0, 63, 64, 69]}, {"id": "b", "tokens": b[:9], "want": [8]}], "end": []}]
    for i in range(3):
        steps.append({"step": 1 + i, "entries": [{"id": "a", "tokens": [a[70 + i]], "want": [0]}, {"id": "b", "tokens": [b[9 + i]], "want": [0]}],
                      "end": ["b"] if i == 2 else []})
    steps.append({"step": 4, "entries": [{"id": "a", "tokens": list(a[73:75]), "want": [1]}], "end": ["a"]})
    out = str(tmp_path / "out")
    cmd = [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", H.folder(name, dtype=dtype), "--dtype", dtype, "--out", out,
           "--max-tokens", "192"]
    p = subprocess.run(cmd, input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.split("\n") if l] == [f"done {i}" for i in range(5)]
    read = lambda i: np.fromfile(os.path.join(out, f"{i}.f32"), dtype="<f4").reshape(-1, vocab)
    pa, pb = H.plain_logits(name, a, dtype=dtype), H.plain_logits(name, b, dtype=dtype)
    H.close(read(0), np.concatenate([pa[[0, 63, 64, 69]], pb[8:9]]), dtype, "step 0")
    for i in range(3):
        H.close(read(1 + i), np.concatenate([pa[70 + i:71 + i], pb[9 + i:10 + i]]), dtype, f"step {1 + i}")
    H.close(read(4), pa[74:75], dtype, "step 4")


def test_the_command_line_on_a_model_of_the_design(tmp_path):
    """`random` writes a model folder from a configuration file; generation from token ids prints what the
    plain loop generates; --bench prints its block."""
    name = "zis_d"
    cfg_file = tmp_path / "config.json"
    cfg_file.write_text(json.dumps(zc.ALL[name]))
    out = tmp_path / "model"
    run = lambda *args: subprocess.run([sys.executable, "-m", "daisi-llogos_amd", *args], capture_output=True, text=True, timeout=600, cwd=ROOT)
    p = run("random", "--config", str(cfg_file), "--output-dir", str(out), "--seed", "4")
    assert p.returncode == 0, p.stderr[-2000:]
    cfg, w = pz.load(str(out))
    prompt = list(H.tokens(name, 11, 21))
    p = run("--model", str(out), "--prompt", " ".join(map(str, prompt)), "-n", "6", "-t", "0", "--repeat-penalty", "1.0",
            "--dtype", "float32", "--max-context", "64")
    assert p.returncode == 0, p.stderr[-2000:]
    assert [int(t) for t in p.stdout.split()] == pz.generate_greedy(cfg, w, prompt, 6)
    p = run("--model", str(out), "--bench", "--batch", "2", "-n", "8", "--prompt-len", "20", "--max-context", "64")
    assert p.returncode == 0, p.stderr[-2000:]
    assert "decode" in (p.stdout + p.stderr)


def _drawn(seed: int) -> dict:
    """A configuration drawn from a seed over everything the file can vary."""
    rng = np.random.default_rng(seed)
    pick = lambda *xs: xs[int(rng.integers(len(xs)))]
    W = int(pick(40, 48, 64, 72, 96)) if seed < 16 else int(pick(50, 100))          # (widths that no vector load divides, too)

    def recurrence(**ranks):
        kv = int(pick(1, 2, 3))
        return zc.rec(kv * int(pick(1, 1, 2)), kv, int(pick(4, 7, 16, 20, 40, 64)), int(pick(4, 16, 30, 72)), int(pick(1, 2, 3, 4, 5)), **ranks)

    layers = []
    for i in range(int(rng.integers(2, 6))):
        mlp = None
        if pick(True, True, True, False):
            count = int(pick(1, 2, 3))
            experts = count * int(rng.integers(1, 4))
            keep = int(rng.integers(1, count + 1))
            top = int(rng.integers(1, experts // count * keep + 1))
            mlp = zc.moe(experts, top, int(pick(8, 20, 32, 33)), float(pick(0.3, 1.0, 7.0)), pick(None, (count, keep)) if top <= experts else (count, keep),
                         pick(None, (int(pick(16, 21)), float(pick(0.5, 7.0)))))
        if pick(True, False):
            layers.append(zc.delta(recurrence(), mlp))
        else:
            kv, d = int(pick(1, 2)), int(pick(8, 16, 20, 64))
            scaling = pick(None, (float(pick(2.0, 8.0)), 1.0, float(pick(2.0, 4.0)), int(pick(40, 200))))
            left = zc.att(kv * int(pick(1, 2, 3)), kv, d, int(pick(8, 16, 20, 64)), float(pick(0.2, 0.3)), pick(None, 1, 5, 33, 64, 65, 90, 500),
                          int(pick(0, 2, 6, d)), float(pick(100.0, 10000.0)), scaling)
            layers.append(zc.parallel(left, recurrence(decay_rank=int(pick(3, 8, 16)), gate_rank=int(pick(1, 8, 20))), mlp))
    cfg = {"architecture": "Zisedra", "vocab": int(pick(50, 131)), "width": W, "norm": {"eps": float(pick(1e-5, 1e-6))}, "layers": layers,
           "torch_dtype": "bfloat16"}
    if pick(True, True, False):
        start = int(rng.integers(0, len(layers)))
        cfg["loop"] = zc.loop(start, int(rng.integers(start + 1, len(layers) + 1)), int(pick(1, 2, 3)))
    if pick(True, True, False):
        cfg["residual_mult"] = float(pick(0.25, 0.8, 1.2))
    return cfg


@pytest.mark.parametrize("seed", range(20))
def test_configurations_drawn_from_seeds(seed, tmp_path):
    """Ragged prompts, single tokens, a sequence that ends early and a new prompt in the freed slot beside one that goes on."""
    from safetensors.torch import load_file, save_file
    cfg = _drawn(seed)
    rng = np.random.default_rng(seed)
    seqs = [[int(t) for t in rng.integers(0, cfg["vocab"], size=n)] for n in (90, 17, 70, 40)]
    for dtype in H.DTYPES:
        path = L.write_random_model(str(tmp_path / dtype), cfg, seed=seed, std=0.08)
        file = os.path.join(path, "model.safetensors")
        save_file(H.sharpen(load_file(file), H.fixed_choice(dtype)), file)
        pcfg, w = pz.load(path)
        want = [pz.forward(pcfg, w, s) for s in seqs]
        eng = L.Engine.from_folder(path, dtype=dtype, max_tokens=512, n_slots=3)
        s0, s1, s2 = eng.alloc_slot(), eng.alloc_slot(), eng.alloc_slot()
        got = [[], [], [], []]
        out = _np(eng.step([(s0, seqs[0][:66]), (s1, seqs[1][:3]), (s2, seqs[2][:64])], want="all"))
        got[0].append(out[:66]); got[1].append(out[66:69]); got[2].append(out[69:])
        for step in range(6):
            out = _np(eng.step([(s0, [seqs[0][66 + step]]), (s1, [seqs[1][3 + step]]), (s2, [seqs[2][64 + step]])], want="all"))
            for i in range(3):
                got[i].append(out[i:i + 1])
        eng.free_slot(s1)
        s3 = eng.alloc_slot()
        assert s3 == s1
        out = _np(eng.step([(s0, seqs[0][72:90]), (s3, seqs[3][:40])], want="all"))      # a continued prompt beside a new one in the freed slot
        got[0].append(out[:18]); got[3].append(out[18:])
        for i, n in ((0, 90), (1, 9), (2, 70), (3, 40)):
            H.close(np.concatenate(got[i]), want[i][:n], dtype, f"seed {seed} sequence {i}")
