"""Small configurations of the Zisedra design for tests.  Between them every size differs from layer to layer and from the
others of its layer (heads, key heads, key and value widths that differ either way, sizes that are no multiple of 16
or of 4), both layer types come in several orders, windows are shorter than a page, as long as one, longer, of a
single key and longer than any test's sequence; heads are rotated in part, whole or not at all, with and without
stretched frequencies; convolutions have one tap to six; the loop covers all layers, some or one, two or three times or
once, or is absent; the feed-forward is absent, with and without groups (one expert a group too) and a shared expert,
with bounds that many sums reach and bounds that none does; the factor on a sublayer is one, below and above it."""


def rec(heads, kv_heads, dim, vdim, conv, **ranks):
    return dict({"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, **ranks)


def att(heads, kv_heads, dim, vdim, scale, window, dims=None, base=10000.0, scaling=None):
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window is not None:
        out["mask"] = {"size": window}
    if dims:
        out["rot"] = {"base": base, "dims": dims}
        if scaling:
            out["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return out


def delta(mixer, mlp=None):
    return {"type": "delta", "mixer": mixer, "mlp": mlp}


def parallel(left, right, mlp=None):
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": mlp}


def moe(experts, top, ff, limit, groups=None, shared=None):
    router = {"experts": experts, "top": top}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    out = {"kind": "moe", "router": router, "expert": {"ff": ff, "limit": limit}}
    if shared:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def loop(start, stop, times):
    return {"start": start, "stop": stop, "times": times}


ZIS_A = {   # a looped pair in the middle; a window shorter than a page; a layer without a feed-forward
    "architecture": "Zisedra", "vocab": 131, "width": 96, "norm": {"eps": 1e-5}, "residual_mult": 0.45, "loop": loop(1, 3, 2),
    "layers": [delta(rec(4, 2, 24, 40, 4), moe(6, 2, 40, 1.0, (3, 2), (56, 0.6))),
               parallel(att(3, 1, 24, 40, 0.4, 37, 12, 500.0, (4.0, 1.0, 4.0, 64)), rec(3, 3, 16, 24, 3, decay_rank=12, gate_rank=20), moe(4, 1, 24, 3.0)),
               delta(rec(2, 1, 32, 16, 2), None),
               parallel(att(4, 2, 16, 16, 0.3, 90, 16), rec(2, 1, 24, 56, 5, decay_rank=7, gate_rank=9), moe(5, 5, 32, 0.8, None, (24, 5.0)))],
    "torch_dtype": "bfloat16",
}

ZIS_B = {   # all layers three times; odd widths; a window of one page; no rotation; groups of one expert; no factor named
    "architecture": "Zisedra", "vocab": 90, "width": 72, "norm": {"eps": 1e-6}, "loop": loop(0, 2, 3),
    "layers": [parallel(att(2, 2, 12, 20, 0.5, 64), rec(5, 1, 6, 9, 1, decay_rank=5, gate_rank=3), moe(4, 2, 20, 1.5, (4, 3), (30, 0.9))),
               delta(rec(3, 3, 10, 18, 6), moe(9, 3, 12, 0.5, (3, 1)))],
    "torch_dtype": "bfloat16",
}

ZIS_C = {   # head shapes that the matrix-core kernels take, windows over page borders
    "architecture": "Zisedra", "vocab": 190, "width": 128, "norm": {"eps": 1e-5}, "residual_mult": 0.7, "loop": loop(2, 4, 2),
    "layers": [parallel(att(4, 2, 64, 64, 0.15, 100, 32, 2000.0, (8.0, 1.0, 4.0, 512)), rec(2, 2, 64, 64, 4, decay_rank=16, gate_rank=16),
                        moe(8, 3, 64, 2.0, (4, 2), (96, 2.0))),
               delta(rec(4, 2, 32, 128, 4), moe(16, 4, 48, 2.0, (4, 2))),
               parallel(att(4, 1, 96, 128, 0.12, 65, 96, 2000.0), rec(1, 1, 128, 64, 4, decay_rank=32, gate_rank=16), moe(8, 2, 64, 1.2, (2, 1), (64, 1.0))),
               delta(rec(2, 1, 128, 128, 4), moe(4, 2, 48, 2.0, (2, 2), (40, 3.0))),
               parallel(att(2, 1, 128, 128, 0.1, 193, 64, 500000.0, (4.0, 1.0, 2.0, 100)), rec(3, 1, 48, 80, 3, decay_rank=8, gate_rank=24), None)],
    "torch_dtype": "bfloat16",
}

ZIS_D = {   # one head each, a loop of one pass, a window longer than the sequences, a factor above one
    "architecture": "Zisedra", "vocab": 67, "width": 48, "norm": {"eps": 1e-5}, "residual_mult": 1.3, "loop": loop(1, 2, 1),
    "layers": [delta(rec(1, 1, 16, 16, 4), None),
               parallel(att(1, 1, 16, 16, 0.4, 1000, 8, 100.0), rec(1, 1, 16, 16, 4, decay_rank=4, gate_rank=4), moe(1, 1, 24, 0.7, None, (16, 0.7)))],
    "torch_dtype": "bfloat16",
}

ZIS_E = {   # no loop; a window of a single key (itself), then no window at all; the last layer is alone
    "architecture": "Zisedra", "vocab": 75, "width": 64, "norm": {"eps": 1e-5}, "residual_mult": 0.6,
    "layers": [parallel(att(2, 1, 16, 24, 0.3, 1, 4, 50.0), rec(4, 2, 20, 12, 2, decay_rank=11, gate_rank=6), moe(6, 3, 16, 1.0, (2, 1))),
               parallel(att(3, 3, 8, 8, 0.5, None, 8), rec(2, 2, 7, 33, 4, decay_rank=3, gate_rank=8), moe(3, 2, 33, 1.0, None, (17, 1.1))),
               delta(rec(6, 3, 9, 15, 4), moe(2, 1, 40, 0.4))],
    "torch_dtype": "bfloat16",
}

ALL = {"zis_a": ZIS_A, "zis_b": ZIS_B, "zis_c": ZIS_C, "zis_d": ZIS_D, "zis_e": ZIS_E}
