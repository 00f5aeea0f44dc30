"""The Peponex design on the GPU against the plain implementation: every mechanism alone, whole prompts,
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

import peponex_configs as pc
import peponex_helpers as H
import plain_peponex as pp

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
    lim = {"norm": (0.7, 1.3), "router": (-0.4, 0.4), "unit": (0.0, 0.8), "decay": (-4.0, -0.5), "bonus": (-0.5, 1.5)}
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


# ---------------------------------------------------------------------------
# mechanisms alone
# ---------------------------------------------------------------------------
# (heads, key channels, value channels)
DECAYS = [(2, 24, 40), (3, 10, 18), (1, 16, 16), (2, 64, 128), (3, 128, 64), (1, 256, 200), (5, 3, 7), (2, 33, 5), (1, 96, 300), (2, 128, 128)]


@pytest.mark.parametrize("segments", [0, 1, 3])
@pytest.mark.parametrize("cuts", [PIECES, WHOLE])
@pytest.mark.parametrize("shape", DECAYS)
def test_the_recurrence_alone_in_pieces(shape, cuts, segments, monkeypatch):
    """Whole prompts, portions and single tokens against the plain recurrence, rows of products in one part and in three;
    a decay of one, of near zero and of exactly zero between them; the state at the end too."""
    monkeypatch.setattr(K, "DECAY_SEGMENTS", segments)
    heads, D, V = shape
    rng = np.random.default_rng(heads * 1000 + D + V)
    decay = [(0.9, 1.0, 0.02, 0.999, 0.0)[(h + D) % 5] for h in range(heads)]
    powers = K.decay_powers(decay, DEV)
    lengths, slots = (150, 70, 3), [2, 0, 3]
    extra = 12                                                 # columns behind q, k and v that are another's
    width = heads * (2 * D + V)
    rows = [rng.standard_normal((n, width + extra)) for n in lengths]
    act = [pp.silu(np.asarray(torch.tensor(r, dtype=torch.float32).double())) for r in rows]
    want, ends = [], []
    for a in act:
        n = len(a)
        o, S = pp.decay_recurrence(a[:, :heads * D].reshape(n, heads, D), a[:, heads * D:2 * heads * D].reshape(n, heads, D),
                                   a[:, 2 * heads * D:width].reshape(n, heads, V), decay)
        want.append(o.reshape(n, heads * V))
        ends.append(S)
    state = torch.zeros((5, heads * D * V), dtype=torch.float32, device=DEV)
    state[[1, 4]] = float("nan")                               # nobody's
    rt = P.Runtime(DEV, torch.float32)
    got = [np.zeros((n, heads * V)) for n in lengths]
    for step, (seqs, lo, hi) in enumerate(_steps(lengths, cuts)):
        ctx = _ctx(rt, hi, [b - a for a, b in zip(lo, hi)], [slots[i] for i in seqs])
        r = np.concatenate([rows[i][a:b] for i, a, b in zip(seqs, lo, hi)])
        if step % 2:
            noise = rng.standard_normal((2,) + r.shape)
            t = torch.stack([_f32(noise[0]), _f32(noise[1]), _f32(r) - _f32(noise[0]) - _f32(noise[1])])
        else:
            t = _f32(r)
        o = _np(K.decay_scan(ctx, t, powers, state, heads, D, V))
        at = 0
        for i, a, b in zip(seqs, lo, hi):
            got[i][a:b] = o[at:at + b - a]
            at += b - a
    for i in range(3):
        size = np.abs(want[i]).max()
        assert np.isfinite(got[i]).all() and np.abs(got[i] - want[i]).max() <= 2e-5 * max(1.0, size), f"sequence {i}"
        S = _np(state[slots[i]]).reshape(heads, D, V)
        assert np.abs(S - ends[i]).max() <= 2e-5 * max(1.0, np.abs(ends[i]).max()), f"state {i}"


def test_the_recurrence_carries_a_loud_token_over_hundreds():
    """One token's product is all that the state holds besides small ones; 600 tokens later it still decides, whatever the
    cut; without it, or with a decay a thousandth off, the result is another by far."""
    rng = np.random.default_rng(8)
    heads, D, V, n = 2, 32, 48, 640
    decay = (0.999, 0.9999)
    rows = rng.standard_normal((n, heads * (2 * D + V))) * 0.05
    rows[20] = np.abs(rng.standard_normal(rows.shape[1])) * 8.0
    split = lambda a: (a[:, :heads * D].reshape(n, heads, D), a[:, heads * D:2 * heads * D].reshape(n, heads, D), a[:, 2 * heads * D:].reshape(n, heads, V))
    act = pp.silu(np.asarray(torch.tensor(rows, dtype=torch.float32).double()))
    want = pp.decay_recurrence(*split(act), decay)[0].reshape(n, -1)
    size = np.abs(want[600:]).max()
    quiet = act.copy(); quiet[20] = 0.0
    assert np.abs(pp.decay_recurrence(*split(quiet), decay)[0].reshape(n, -1)[600:] - want[600:]).max() > 0.1 * size
    assert np.abs(pp.decay_recurrence(*split(act), (0.998, 0.9999))[0].reshape(n, -1)[600:] - want[600:]).max() > 0.05 * size
    rt = P.Runtime(DEV, torch.float32)
    for cuts in ([640], [31, 1, 33, 2, 500] + [1] * 73, [600] + [1] * 40):
        state = torch.zeros((1, heads * D * V), dtype=torch.float32, device=DEV)
        at, got = 0, []
        for c in cuts:
            got.append(_np(K.decay_scan(_ctx(rt, [at + c], [c], [0]), _f32(rows[at:at + c]), K.decay_powers(decay, DEV), state, heads, D, V)))
            at += c
        got = np.concatenate(got)
        assert np.abs(got[20:] - want[20:]).max() <= 2e-5 * np.abs(want).max()
        assert np.abs(got[600:] - want[600:]).max() <= 5e-5 * size


def test_the_recurrence_refuses_what_does_not_fit():
    rt = P.Runtime(DEV, torch.float32)
    ctx, pw, st = _ctx(rt, [4], [4], [0]), K.decay_powers((0.5, 0.5), DEV), torch.zeros((1, 2 * 8 * 8), device=DEV)
    ok = torch.zeros((4, 2 * 24), device=DEV)
    K.decay_scan(ctx, ok, pw, st, 2, 8, 8)
    for bad in (lambda: K.decay_scan(ctx, ok[:, :40].contiguous(), pw, st, 2, 8, 8), lambda: K.decay_scan(ctx, ok[:3], pw, st, 2, 8, 8),
                lambda: K.decay_scan(ctx, ok, pw[:1], st, 2, 8, 8), lambda: K.decay_scan(ctx, ok, pw, st[:, :64].contiguous(), 2, 8, 8),
                lambda: K.decay_scan(ctx, ok.bfloat16(), pw, st, 2, 8, 8), lambda: K.decay_scan(ctx, ok, pw, st.bfloat16(), 2, 8, 8)):
        with pytest.raises(K.KernelError):
            bad()


@pytest.mark.parametrize("rows", H.DTYPES)
@pytest.mark.parametrize("T,N,parts", [(1, 6, 1), (5, 80, 3), (300, 100, 1), (7, 1024, 2), (2, 5001, 1), (260, 4096, 1)])
def test_the_norm_over_a_row_with_a_sigmoid_gate(T, N, parts, rows):
    rng = np.random.default_rng(N)
    o, w, z = rng.standard_normal((T, N)) * 3, rng.uniform(0.5, 1.5, N), rng.standard_normal((parts, T, N + 3)) * 2
    want = pp.norm(o, w, 1e-4) * pp.sigmoid(z.sum(0)[:, 3:])
    gate = _f32(z)[..., 3:] if parts > 1 else _f32(z[0])[:, 3:]
    got = K.gated_row_norm(_f32(o), _f32(w), gate, 1e-4, DT[rows])
    assert got.dtype == DT[rows] and np.abs(_np(got) - want).max() <= (1e-5 if rows == "float32" else 1e-2) * np.abs(want).max()


@pytest.mark.parametrize("rows", H.DTYPES)
@pytest.mark.parametrize("T,W", [(1, 6), (5, 96), (70, 72), (3, 1001)])
def test_sums_into_the_stream(T, W, rows):
    rng = np.random.default_rng(W)
    x, d, again, vec = rng.standard_normal((T, W)), rng.standard_normal((3, T, W)), rng.standard_normal((T, W)), rng.standard_normal(W)
    for use in range(8):
        xt = _f32(x)
        want = x + (d.sum(0) if use & 1 else 0) + (again if use & 2 else 0) + (vec if use & 4 else 0)
        got = K.stream_add(xt, _f32(d) if use & 1 else None, again=_f32(again) if use & 2 else None, vector=_f32(vec) if use & 4 else None,
                           rows_dtype=DT[rows])
        assert np.abs(_np(xt) - want).max() <= 1e-5
        assert (got is xt) == (rows == "float32") and np.abs(_np(got) - want).max() <= (1e-5 if rows == "float32" else 4e-3 * np.abs(want).max())
        if rows == "float32" and use == 1:
            half = _f32(d[0]).bfloat16()
            xt = _f32(x)
            assert K.stream_add(xt, half) is None and np.abs(_np(xt) - (x + _np(half))).max() <= 1e-5


@pytest.mark.parametrize("dtype", H.DTYPES)
def test_a_tables_row_behind_a_gate(dtype):
    rng = np.random.default_rng(4)
    z, table, ids = rng.standard_normal((2, 9, 22)) * 2, _rounded(rng.standard_normal((31, 22)), dtype), [3, 30, 0, 3, 7, 7, 1, 2, 29]
    want = pp.gelu_tanh(z.sum(0)) * table[ids]
    got = K.gated_lookup(_f32(z), torch.tensor(table, dtype=DT[dtype], device=DEV), _i32(ids), DT[dtype])
    assert np.abs(_np(got) - want).max() <= PART_TOL[dtype] * np.abs(want).max()


# (heads, key channels, value channels, hidden)
LIGHTNINGS = [(2, 24, 40, 56), (3, 10, 18, 72), (1, 16, 16, 40), (2, 64, 128, 64), (4, 128, 128, 96), (5, 8, 8, 33)]


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("cuts", [PIECES, WHOLE])
@pytest.mark.parametrize("shape", LIGHTNINGS)
def test_the_lightning_mixer_alone_in_pieces(shape, cuts, dtype):
    heads, D, V, hidden = shape
    rng = np.random.default_rng(heads * 10 + D)
    decay = [0.3 + 0.69 * (h + 1) / heads for h in range(heads)]
    mix = P.Lightning(prefix="m.", hidden=hidden, n_heads=heads, head_dim=D, v_dim=V, decay=decay, eps=1e-5)
    plain = _bind(mix, rng, dtype)
    assert set(plain) == {"m.q", "m.k", "m.v", "m.g", "m.o", "m.norm"} and mix.kv_spec() is None
    lengths, slots = (150, 70, 3), [1, 3, 0]
    h = [_rounded(rng.standard_normal((n, hidden)), dtype) for n in lengths]
    m = {"heads": heads, "dim": D, "vdim": V, "decay": decay}
    want = [pp.lightning(x, pp.part(plain, "m."), m, 1e-5) for x in h]
    state = torch.zeros((4,) + mix.state_spec().shape, dtype=torch.float32, device=DEV)
    got = _in_pieces(mix, h, lengths, slots, cuts, dtype, lambda seqs: P.LayerCache(state=state))
    for g, w_ in zip(got, want):
        assert np.isfinite(g).all() and np.abs(g - w_).max() <= PART_TOL[dtype] * max(1.0, np.abs(w_).max())
    no_gate = pp.lightning(h[0], dict(pp.part(plain, "m."), g=np.zeros((heads * V, hidden))), m, 1e-5)
    assert np.abs(no_gate - want[0]).max() > 100 * PART_TOL["float32"] * np.abs(want[0]).max()


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
            o = _np(x - before) if isinstance(left, K.RowSquares) else _np(K.sum_parts(left, None, torch.float32))
            assert isinstance(left, K.RowSquares) or torch.equal(x, before)
        else:
            o = _np(K.sum_parts(mix.forward(ctx, rows, cache), None, torch.float32))
        at = 0
        for i, a, b in zip(seqs, lo, hi):
            got[i][a:b] = o[at:at + b - a]
            at += b - a
    return got


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("shape", [(3, 16, 12, 56), (5, 8, 3, 40), (1, 64, 16, 72), (2, 32, 40, 64)])
def test_the_wkv_mixer_alone_in_pieces(shape, dtype):
    heads, D, rank, hidden = shape
    rng = np.random.default_rng(heads * 10 + D)
    mix = P.WKV(prefix="m.", hidden=hidden, n_heads=heads, head_dim=D, decay_rank=rank, eps=1e-5)
    plain = _bind(mix, rng, dtype)
    lengths, slots = (150, 70, 3), [1, 3, 0]
    h = [np.asarray(torch.tensor(rng.standard_normal((n, hidden)), dtype=torch.float32).double()) for n in lengths]
    want = [pp.wkv(x, pp.part(plain, "m."), {"heads": heads, "dim": D}, 1e-5) for x in h]
    state = torch.zeros((4,) + mix.state_spec().shape, dtype=torch.float32, device=DEV)
    got = _in_pieces(mix, h, lengths, slots, PIECES, dtype, lambda seqs: P.LayerCache(state=state), f32_rows=True)
    for g, w_ in zip(got, want):
        assert np.isfinite(g).all() and np.abs(g - w_).max() <= (2 if dtype == "bfloat16" else 1) * PART_TOL[dtype] * max(1.0, np.abs(w_).max())


# (heads, dim, rotated width, value width, rank, hidden)
LATENTS = [(3, 24, 8, 40, 48, 56), (2, 12, 6, 20, 18, 72), (4, 64, 64, 64, 64, 64), (6, 32, 32, 80, 96, 96), (2, 128, 64, 128, 128, 64), (3, 48, 48, 96, 40, 64),
           (1, 8, 8, 8, 16, 16)]
WINDOWS = [1, 2, 37, 63, 64, 65, 66, 100, 400]


def _latent(shape, window, dtype, rng, pairing="split_half", scale=None, scaled=None):
    heads, d, r, dv, rank, hidden = shape
    # scores that spread over some units whatever the sizes: sharp, and still within what bfloat16 queries resolve
    scale = scale or 5.0 / (0.36 * np.sqrt(float(d) * hidden * rank))
    mix = P.LatentAttention(prefix="m.", hidden=hidden, n_heads=heads, dim=d, rot_dim=r, v_dim=dv, q_rank=0, kv_rank=rank, scale=scale, eps=1e-5,
                            position=P.Rotary(r, r, 300.0, pairing=pairing), sink=False, window=window)
    mix.rt = P.Runtime(DEV, DT[dtype])                         # (the cache's shape depends on the type)
    plain = _bind(mix, rng, dtype, scaled=dict({"m.q": 2.0, "m.uk": 2.0}, **(scaled or {})))
    m = {"heads": heads, "dim": d, "rot_dim": r, "vdim": dv, "kv_rank": rank, "scale": scale, "mask": {"size": window}, "rot": {"dims": r, "base": 300.0}}
    return mix, plain, m


def _pools(mix, pages, dtype):
    spec = mix.kv_spec()
    k = torch.full((pages, 1, 64 * spec.head_dim), float("nan"), dtype=DT[dtype], device=DEV)
    v = torch.full((pages, 1, 64 * spec.head_dim), float("nan"), dtype=DT[dtype], device=DEV) if spec.values else None
    return k, v


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("cuts", [PIECES, WHOLE])
@pytest.mark.parametrize("shape", LATENTS)
@pytest.mark.parametrize("window", WINDOWS)
def test_the_window_attention_through_a_latent_alone_in_pieces(window, shape, cuts, dtype, monkeypatch):
    """Pages in any order that start as NaN; as soon as no later query can see a page its place in the table is
    taken away, as the cache does.  Whole prompts of head shapes that the matrix cores take must go over keys
    and values a head, in pages of the step's own that start as NaN too."""
    heads, d, r, dv, rank, hidden = shape
    rng = np.random.default_rng(heads * 10 + rank + window)
    mix, plain, m = _latent(shape, window, dtype, rng)
    assert mix.kv_spec().window == window
    lengths = (150, 70, 3)
    h = [_rounded(rng.standard_normal((n, hidden)), dtype) for n in lengths]
    want = [pp.latent_attention(x, pp.part(plain, "m."), m, 1e-5) for x in h]
    k_pool, v_pool = _pools(mix, 9, dtype)
    pages = {0: [7, 2, 5], 1: [0, 8], 2: [3]}
    by_head = cuts is WHOLE and dtype == "bfloat16" and d + r in (64, 96, 128, 192) and dv in (64, 80, 96, 128)
    ran = []
    if by_head:
        keep = mix._forward_prompt
        monkeypatch.setattr(mix, "_forward_prompt", lambda *a, **k: (ran.append(1), keep(*a, **k))[1])
        monkeypatch.setattr(K, "attention_generic", lambda *a, **k: pytest.fail("the kernel for any shape ran"))
        fresh = torch.empty

        def poisoned(*a, **k):
            t = fresh(*a, **k)
            if t.dtype == torch.bfloat16 and t.dim() == 3:
                t.fill_(float("nan"))
            return t
        monkeypatch.setattr(torch, "empty", poisoned)
    seen = [0, 0, 0]                                           # tokens of each sequence so far

    def cache_of(seqs):
        table = np.full((len(seqs), 3), -1, dtype=np.int32)
        for row, i in enumerate(seqs):
            for j, p in enumerate(pages[i]):
                if 64 * j + 63 > seen[i] - window:             # (GroupPages.release_behind_window)
                    table[row, j] = p
        return P.LayerCache(k_pool=k_pool, v_pool=v_pool, table=_i32(table))

    got = [np.zeros((n, hidden)) for n in lengths]
    for seqs, lo, hi in _steps(lengths, cuts):
        ctx = _ctx(mix.rt, hi, [b - a for a, b in zip(lo, hi)], [0, 1, 2][:len(seqs)])
        rows = torch.tensor(np.concatenate([h[i][a:b] for i, a, b in zip(seqs, lo, hi)]), dtype=DT[dtype], device=DEV)
        o = _np(K.sum_parts(mix.forward(ctx, rows, cache_of(seqs)), None, torch.float32))
        at = 0
        for i, a, b in zip(seqs, lo, hi):
            got[i][a:b] = o[at:at + b - a]
            at += b - a
            seen[i] = b
    for i, (g, w_) in enumerate(zip(got, want)):
        assert np.isfinite(g).all()
        assert np.abs(g - w_).max() <= (2 if dtype == "bfloat16" else 1) * PART_TOL[dtype] * max(1.0, np.abs(w_).max()), f"sequence {i}"
    assert len(ran) == (1 if by_head else 0)


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("pairing", ["split_half", "interleaved"])
@pytest.mark.parametrize("shape", [(2, 24, 8, 40, 48, 56), (2, 64, 64, 64, 64, 64)])
def test_both_pairings_and_no_window(pairing, shape, dtype):
    """Without a window, and with a partial rotation (rot_dims below the part's width), whole and in pieces."""
    heads, d, r, dv, rank, hidden = shape
    rng = np.random.default_rng(3)
    mix, plain, m = _latent(shape, 0, dtype, rng, pairing)
    mix.position = P.Rotary(r, r // 2, 300.0, pairing=pairing)
    mix.position.bind(None, mix.rt)
    m["mask"]["size"], m["rot"]["dims"] = 10 ** 9, r // 2
    t = pp.part(plain, "m.")
    if pairing == "interleaved":                               # the same attention with the rotated dimensions in another order
        order = np.concatenate([np.arange(0, r // 2, 2), np.arange(1, r // 2, 2), np.arange(r // 2, r)])
        q = t["q"].reshape(heads, d + r, hidden).copy()
        q[:, d:] = q[:, d:][:, order]
        dkv = t["dkv"].copy()
        dkv[rank:] = dkv[rank:][order]
        t = dict(t, q=q.reshape(-1, hidden), dkv=dkv)
    n = 150
    h = _rounded(rng.standard_normal((n, hidden)), dtype)
    want = pp.latent_attention(h, t, m, 1e-5)
    for cuts in ([150], [70, 1, 2, 76, 1]):
        k_pool, v_pool = _pools(mix, 3, dtype)
        at, got = 0, []
        for c in cuts:
            ctx = _ctx(mix.rt, [at + c], [c], [0])
            cache = P.LayerCache(k_pool=k_pool, v_pool=v_pool, table=_i32([[2, 0, 1]]))
            got.append(_np(K.sum_parts(mix.forward(ctx, torch.tensor(h[at:at + c], dtype=DT[dtype], device=DEV), cache), None, torch.float32)))
            at += c
        assert np.abs(np.concatenate(got) - want).max() <= (2 if dtype == "bfloat16" else 1) * PART_TOL[dtype] * max(1.0, np.abs(want).max())


@pytest.mark.parametrize("window", [40, 64, 65, 129, 150])
@pytest.mark.parametrize("shape", [(2, 32, 32, 80, 96, 64), (2, 24, 8, 40, 48, 64)])
def test_a_key_at_the_windows_edge_decides(window, shape):
    """A loud token's key stands out for every query that sees it: the last one that does and the first that does not are
    told apart in a prompt, behind a portion's start and in decoding (a window one longer or shorter is another result by a
    hundred times the bound there)."""
    rng = np.random.default_rng(window)
    heads, d, r, dv, rank, hidden = shape
    mix, plain, m = _latent(shape, window, "float32", rng, scale=0.05)
    t = pp.part(plain, "m.")
    loud, n = 50, 50 + window + 20
    h = rng.standard_normal((n, hidden))
    # every query leans towards the loud token's key in the unrotated part
    kv = h @ t["dkv"].T
    c = pp.norm(kv[:, :rank], t["dkv.norm"], 1e-5)
    q = t["q"].reshape(heads, d + r, hidden).copy()
    key = (c[loud] @ t["uk"].T).reshape(heads, d)
    bias = rng.standard_normal(hidden)
    bias /= np.linalg.norm(bias)
    h += bias * 6.0
    kv = h @ t["dkv"].T
    c = pp.norm(kv[:, :rank], t["dkv.norm"], 1e-5)
    key = (c[loud] @ t["uk"].T).reshape(heads, d)
    for hd in range(heads):
        q[hd, :d] += np.outer(key[hd] / np.linalg.norm(key[hd]) * 12.0, bias)
    t = dict(t, q=q.reshape(-1, hidden))
    t = {k_: _rounded(v_, "bfloat16") for k_, v_ in t.items()}
    h = np.asarray(torch.tensor(h, dtype=torch.float32).double())
    want = pp.latent_attention(h, t, m, 1e-5)
    last = loud + window - 1                                   # the last query that sees the loud key
    shorter = pp.latent_attention(h, t, dict(m, mask={"size": window - 1}), 1e-5)
    longer = pp.latent_attention(h, t, dict(m, mask={"size": window + 1}), 1e-5)
    size = np.abs(want).max()
    assert np.abs(shorter[last] - want[last]).max() > 100 * PART_TOL["float32"] * size
    assert np.abs(longer[last + 1] - want[last + 1]).max() > 100 * PART_TOL["float32"] * size
    for dtype in H.DTYPES:
        mix, _, _ = _latent(shape, window, dtype, np.random.default_rng(window), scale=0.05)
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
                got = np.concatenate(got)
                err = np.abs(got - want).max(axis=1)
                assert err.max() <= (PART_TOL[dtype] if dtype == "float32" else 0.1) * size, f"{dtype} from {first} on, {tail}: worst at {err.argmax()}"


@pytest.mark.parametrize("experts,top,K_,T", [(8, 1, 96, 9), (5, 2, 72, 70), (6, 6, 40, 5), (64, 8, 256, 65), (1, 1, 16, 1), (300, 70, 64, 3)])
@pytest.mark.parametrize("rows", H.DTYPES)
@pytest.mark.parametrize("renorm", [False, True])
def test_the_sigmoid_routers_choice_and_weights(experts, top, K_, T, rows, renorm):
    rng = np.random.default_rng(experts + top)
    h, w = _rounded(rng.standard_normal((T, K_)), rows), _rounded(rng.uniform(-0.4, 0.4, size=(experts, K_)), "float32")
    want_c, want_w = pp.route(h, w, top)
    if renorm:
        want_w = want_w / want_w.sum(1, keepdims=True)
    got_c, got_w = K.moe_router(torch.tensor(h, dtype=DT[rows], device=DEV), _f32(w), None, 1, 1, top, 2.0, scores="sigmoid", renorm=renorm)
    got_c, got_w = got_c.cpu().numpy(), _np(got_w)
    same = (got_c == want_c).all(axis=1)                       # (a row whose choice hangs on the last bits of two scores is left out)
    assert same.sum() >= T - max(1, T // 50) and np.abs(got_w - 2.0 * want_w)[same].max() <= 1e-5
    with pytest.raises(K.KernelError):
        K.moe_router(torch.tensor(h, dtype=DT[rows], device=DEV), _f32(w), None, 1, 1, top, 1.0, scores="tanh")


@pytest.mark.parametrize("dtype,form", [("float32", "auto"), ("bfloat16", "auto"), ("bfloat16", "plain"), ("bfloat16", "few"),
                                        ("bfloat16", "tiles64"), ("bfloat16", "tiles128")])
@pytest.mark.parametrize("experts,top,ff,hidden,T", [(6, 1, 40, 96, 9), (1, 1, 16, 32, 3), (4, 4, 24, 48, 70), (8, 3, 72, 64, 300), (16, 1, 96, 128, 1),
                                                     (3, 2, 132, 200, 150), (2, 1, 30, 36, 40)])
def test_experts_weighed_on_their_inputs(dtype, form, experts, top, ff, hidden, T, monkeypatch):
    """Every form of the experts' product; the result as a tensor and added to a stream, with and without the stream's new
    rows.  Weights on the outputs would be another result."""
    monkeypatch.setattr(K, "MOE_PRODUCT", form)
    rng = np.random.default_rng(experts * 10 + top)
    moe = P.RoutedMoE(prefix="f.", hidden=hidden, n_experts=experts, top=top, intermediate=ff, correction=False, scores="sigmoid", renorm=False, weigh="input")
    plain = _bind(moe, rng, dtype)
    h = _rounded(rng.standard_normal((T, hidden)), dtype)
    t, mlp = pp.part(plain, "f."), {"router": {"experts": experts, "top": top}}
    want = pp.mixture(h, t, mlp)
    ht = torch.tensor(h, dtype=DT[dtype], device=DEV)
    got = _np(moe.forward(None, ht))
    chosen, weights = pp.route(h, t["router"], top)
    got_c, _ = K.moe_router(ht, moe.router_w, None, 1, 1, top, 1.0, scores="sigmoid", renorm=False)
    same = (got_c.cpu().numpy() == chosen).all(axis=1)
    assert same.sum() >= T - max(1, T // 50)
    assert np.abs(got - want)[same].max() <= PART_TOL[dtype] * max(1.0, np.abs(want).max())
    outside = np.zeros_like(want)
    for row in range(T):
        for e, w_ in zip(chosen[row], weights[row]):
            outside[row] += w_ * pp.gated_ff(h[row:row + 1], t[f"e{e}.gate"], t[f"e{e}.up"], t[f"e{e}.down"])[0]
    assert np.abs(outside - want).max() > 100 * PART_TOL["float32"] * np.abs(want).max()
    x = torch.randn((T, hidden), dtype=torch.float32, device=DEV)
    for reader in (None, P.TokenSide("s.", "e", hidden, 5, 4, 0, 1, 1e-5)):
        if reader is not None:
            reader.ones = torch.ones(hidden, device=DEV)
        xt = x.clone()
        left = moe.forward(None, ht, residual=base.Residual(xt, reader))
        assert isinstance(left, K.RowSquares) and np.abs(_np(xt) - (_np(x) + got)).max() <= 1e-5 * max(1.0, np.abs(got).max())
        if reader is None or dtype == "float32":
            assert left.unscaled is None
        else:
            assert left.norm_w is reader.ones and torch.equal(left.unscaled, xt.to(torch.bfloat16))
    with pytest.raises(ValueError):
        P.RoutedMoE(prefix="f.", hidden=hidden, n_experts=experts, top=top, intermediate=ff, identity=1, weigh="input")


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("hidden,dim,T,kind", [(96, 20, 5, "rms"), (72, 6, 70, "rms"), (256, 64, 3, "rms"), (64, 24, 200, "rms"), (96, 20, 5, "layer"), (48, 8, 9, "none")])
def test_the_second_embedding_alone(hidden, dim, T, kind, dtype):
    """Whatever completed the stream before it (a delta, its parts, a product that has added itself, another part), and
    whatever norm reads it next (one kernel closes and norms; a norm of another kind runs by itself; none)."""
    rng = np.random.default_rng(hidden)
    side = P.TokenSide("s.", "table", hidden, 31, dim, 2, 3, 1e-5)
    plain = _bind(side, rng, dtype)
    assert plain["table"].shape == (31, 3 * dim)
    nxt = {"rms": P.RMSNorm(name="n", width=hidden, eps=1e-5, suffix=""), "layer": P.LayerNorm(name="n", width=hidden, eps=1e-5, suffix=""), "none": None}[kind]
    if nxt is not None:
        nw = _bind(nxt, rng, dtype)["n"]
    ids = rng.integers(0, 31, size=T)
    ctx = _ctx(side.rt, [T], [T], [0], ids)
    x, d = rng.standard_normal((T, hidden)), rng.standard_normal((3, T, hidden))
    for pending in ("none", "delta", "parts", "squares", "ahead"):
        full = x + (d[0] if pending == "delta" else d.sum(0) if pending == "parts" else 0)
        e = _rounded(plain["table"], dtype)[ids][:, 2 * dim:]
        want = full + pp.token_side(_rounded(full, dtype), e, pp.part(plain, "s."), 1e-5)
        xt = _f32(x)
        given = {"none": None, "delta": _f32(d[0]), "parts": _f32(d), "squares": K.RowSquares(None, hidden), "ahead": base.NormedAhead(None, None)}[pending]
        out, left = side.forward(ctx, xt, given, nxt)
        got = _np(out) + (_np(left) if isinstance(left, torch.Tensor) else 0.0)
        assert np.abs(got - want).max() <= PART_TOL[dtype] * np.abs(want).max(), pending
        if kind == "rms":
            assert left.norm is nxt and np.abs(_np(nxt.forward(out, left)) - pp.norm(want, nw, 1e-5)).max() <= 2 * PART_TOL[dtype] * 3
        elif kind == "none":
            assert left.norm is None


def test_the_loops_entry_by_sums():
    rng = np.random.default_rng(1)
    part = P.LoopAdd(steps="st", width=24, times=3)
    st = _bind(part, rng, "float32")["st"]
    x, x0, d = rng.standard_normal((5, 24)), rng.standard_normal((5, 24)), rng.standard_normal((2, 5, 24))
    for number in range(3):
        for delta in (None, d):
            xt = _f32(x)
            out, left = part.forward(None, xt, None if delta is None else _f32(delta), _f32(x0), number)
            want = x + st[number] + (x0 if number else 0) + (0 if delta is None else d.sum(0))
            assert left is None and np.abs(_np(out) - want).max() <= 1e-5
    with pytest.raises(ValueError):
        part.forward(None, _f32(x), None, _f32(x0), 3)


# ---------------------------------------------------------------------------
# whole models
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("name", list(pc.ALL))
def test_a_whole_prompt_then_the_rest_token_by_token(name, dtype):
    toks = H.tokens(name, 250, 1)
    want = H.plain_logits(name, toks, dtype=dtype)
    eng = H.engine(name, dtype)
    s = eng.alloc_slot()
    got = [_np(_run(eng, s, toks, 0, 180))]
    for t in range(180, 250):                                   # over a page's border
        got.append(_np(_run(eng, s, toks, t, t + 1)))
    H.close(np.concatenate(got), want, dtype, f"{name} prompt and decoding")


@pytest.mark.parametrize("name", list(pc.ALL))
def test_the_residual_stream_after_every_layer_run(name):
    toks = H.tokens(name, 40, 6)
    cfg, w = H.plain(name)
    want = []
    pp.forward(cfg, w, list(toks), want)
    eng = H.engine(name, "float32", use_graphs=False)
    got = []
    for blk in eng.model.layers:
        def wrapped(ctx, x, pending, caches, _o=blk.forward, **kw):
            x, p = _o(ctx, x, pending, caches, **kw)
            got.append(_np(x) + (_np(K.sum_parts(p, None, torch.float32)) if isinstance(p, torch.Tensor) else 0.0))
            return x, p
        blk.forward = wrapped
    _run(eng, eng.alloc_slot(), toks, 0, 40)
    assert len(got) == len(want) == len(pp.runs(cfg))
    for i, (g, w_) in enumerate(zip(got, want)):
        assert np.abs(g - w_).max() <= 5e-5 * np.abs(w_).max(), f"run {i}"


@pytest.mark.parametrize("dtype", H.DTYPES)
@pytest.mark.parametrize("name", list(pc.ALL))
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
@pytest.mark.parametrize("name", ["pep_a", "pep_b", "pep_c"])
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
@pytest.mark.parametrize("name", ["pep_a", "pep_b", "pep_c"])
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
    name = "pep_c"
    cfg, w = H.plain(name)
    toks = H.tokens(name, 420, 4)
    want = H.plain_logits(name, toks)
    mixers, mix, side = dict(pp.MIXERS), pp.mixture, pp.token_side

    def changed(**kw):
        c = json.loads(json.dumps(cfg))
        for L_ in c["layers"]:
            if L_["type"] == "latent_attention":
                L_["mixer"]["mask"]["size"] += kw.get("window", 0)
                L_["mixer"]["rot"]["base"] *= kw.get("base", 1.0)
            if L_["type"] == "lightning":
                L_["mixer"]["decay"] = [d * kw.get("decay", 1.0) for d in L_["mixer"]["decay"]]
        if "cap" in kw:
            c["logit_softcap"] = kw["cap"]
        return c

    def scan_without_a_past(fn):
        def run(h, *a):                                        # a state that is lost at position 300
            return np.concatenate([fn(h[:300], *a), fn(h[300:], *a)])
        return run

    def loop_without_state(c, t, tokens):                      # what the passes add: no vectors, or no embedding output
        t = dict(t)
        t["loop.step"] = np.zeros_like(t["loop.step"])
        return pp.forward(c, t, tokens)

    others = {"window + 1": pp.forward(changed(window=1), w, list(toks)), "window - 1": pp.forward(changed(window=-1), w, list(toks)),
              "rotation": pp.forward(changed(base=1.5), w, list(toks)), "decay": pp.forward(changed(decay=0.99), w, list(toks)),
              "cap": pp.forward(changed(cap=None), w, list(toks)), "steps": loop_without_state(cfg, w, list(toks))}
    try:
        for kind in ("wkv", "lightning"):
            pp.MIXERS[kind] = scan_without_a_past(mixers[kind])
            others[kind + " state"] = pp.forward(cfg, w, list(toks))
            pp.MIXERS.update(mixers)
        pp.token_side = lambda x, e, t, eps: side(x, np.roll(e, 1, axis=1), t, eps)
        others["side columns"] = pp.forward(cfg, w, list(toks))
        pp.token_side = side

        def weight_on_the_output(h, t, mlp):
            chosen, weights = pp.route(h, t["router"], mlp["router"]["top"])
            out = np.zeros_like(h)
            for row in range(len(h)):
                for e, wt in zip(chosen[row], weights[row]):
                    out[row] += wt * pp.gated_ff(h[row:row + 1], t[f"e{e}.gate"], t[f"e{e}.up"], t[f"e{e}.down"])[0]
            return out
        pp.mixture = weight_on_the_output
        others["weight on the output"] = pp.forward(cfg, w, list(toks))
    finally:
        pp.MIXERS.update(mixers)
        pp.mixture, pp.token_side = mix, side
    for what, other in others.items():
        assert H.distance(other[300:], want[300:]) > 10 * H.TOL["float32"], what
    for dt in H.DTYPES:
        eng = H.engine(name, dt)
        s = eng.alloc_slot()
        got = [_np(_run(eng, s, toks, 0, 300))] + [_np(_run(eng, s, toks, t, t + 1)) for t in range(300, 420)]
        H.close(np.concatenate(got), H.plain_logits(name, toks, dtype=dt), dt, "everything there")


def test_greedy_generation_through_the_entry_point():
    name = "pep_a"
    cfg, w = H.plain(name)
    prompts = [list(H.tokens(name, 9, 7)), list(H.tokens(name, 60, 8)), list(H.tokens(name, 2, 9))]
    llm = L.Llogos(H.folder(name), dtype="float32", max_context=128, max_batch=2)        # three requests, two at a time
    out = llm.generate(prompts, L.GenerationParams.greedy(max_tokens=10, stop_tokens=()))
    for p, got in zip(prompts, out.tokens):
        assert got == pp.generate_greedy(cfg, w, p, 10)
    assert out.finish_reasons == ["length"] * 3


@pytest.mark.parametrize("dtype", H.DTYPES)
def test_the_trace_runner_on_a_model_of_the_design(tmp_path, dtype):
    name = "pep_a"
    vocab = pc.ALL[name]["vocab"]
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
    name = "pep_d"
    cfg_file = tmp_path / "config.json"
    cfg_file.write_text(json.dumps(pc.ALL[name]))
    out = tmp_path / "model"
    run = lambda *args: subprocess.run([sys.executable, "-m", "daisi-llogos_amd", *args], capture_output=True, text=True, timeout=600, cwd=ROOT)
    p = run("random", "--config", str(cfg_file), "--output-dir", str(out), "--seed", "4")
    assert p.returncode == 0, p.stderr[-2000:]
    cfg, w = pp.load(str(out))
    prompt = list(H.tokens(name, 11, 21))
    p = run("--model", str(out), "--prompt", " ".join(map(str, prompt)), "-n", "6", "-t", "0", "--repeat-penalty", "1.0",
            "--dtype", "float32", "--max-context", "64")
    assert p.returncode == 0, p.stderr[-2000:]
    assert [int(t) for t in p.stdout.split()] == pp.generate_greedy(cfg, w, prompt, 6)
    p = run("--model", str(out), "--bench", "--batch", "2", "-n", "8", "--prompt-len", "20", "--max-context", "64")
    assert p.returncode == 0, p.stderr[-2000:]
    assert "decode" in (p.stdout + p.stderr)


def _drawn(seed: int) -> dict:
    """A configuration drawn from a seed over everything the file can vary."""
    rng = np.random.default_rng(seed)
    pick = lambda *xs: xs[int(rng.integers(len(xs)))]
    W = int(pick(40, 48, 64, 72, 96)) if seed < 16 else int(pick(50, 100))          # (widths that no vector load divides, too)
    layers = []
    for i in range(int(rng.integers(2, 6))):
        mlp = None
        kind = pick(None, "dense", "moe", "moe")
        if kind == "dense":
            mlp = pc.dense(int(pick(24, 50, 64)))
        elif kind == "moe":
            experts = int(rng.integers(1, 7))
            mlp = pc.moe(experts, int(rng.integers(1, experts + 1)), int(pick(8, 20, 32)))
        kind = pick("wkv", "lightning", "latent")
        heads = int(pick(1, 2, 3, 5))
        if kind == "wkv":
            layers.append(pc.wkv(heads, int(pick(4, 8, 16, 20, 48)), int(pick(1, 8, 16)), mlp))
        elif kind == "lightning":
            layers.append(pc.lightning(heads, int(pick(4, 16, 20, 40, 64)), int(pick(4, 16, 30, 72)), rng.uniform(0.1, 1.0, size=heads).tolist(), mlp))
        else:
            layers.append(pc.latent(heads, int(pick(8, 16, 20, 32)), int(pick(2, 8, 16, 32)), int(pick(8, 16, 20, 64)), int(pick(8, 24, 30, 64)),
                                    float(pick(0.2, 0.3)), int(pick(1, 5, 33, 64, 65, 90, 500)), float(pick(100.0, 10000.0)), mlp))
    cfg = {"architecture": "Peponex", "vocab": int(pick(50, 131)), "width": W, "norm": {"eps": float(pick(1e-5, 1e-6))}, "layers": layers,
           "torch_dtype": "bfloat16"}
    if pick(True, True, False):
        start = int(rng.integers(0, len(layers)))
        cfg["loop"] = pc.loop(start, int(rng.integers(start + 1, len(layers) + 1)), int(pick(1, 2, 3)))
    if pick(True, True, False):
        cfg["token_side"] = {"dim": int(pick(6, 16, 24))}
    if pick(True, False):
        cfg["logit_softcap"] = float(pick(3.0, 20.0))
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
        pcfg, w = pp.load(path)
        want = [pp.forward(pcfg, w, s) for s in seqs]
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
