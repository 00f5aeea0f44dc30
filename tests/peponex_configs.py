"""Small configurations of the Peponex design for tests.  Between them every size differs from layer to layer
and from the others of its layer (heads, key and value widths that differ either way, widths and ranks that are
no multiple of 16 or of 8), the three layer types come in several orders, windows are shorter than a page, as
long as one, longer, of a single key and longer than any test's sequence; the loop covers all layers, some or
one, two or three times or once, or is absent; the feed-forward is absent, dense or a mixture with one choice,
several or all of the experts; decays reach from near zero to one; the second embedding and the bend of the
logits are there or not."""


def wkv(heads, dim, decay_rank, mlp=None):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim, "decay_rank": decay_rank}, "mlp": mlp}


def lightning(heads, dim, vdim, decay, mlp=None):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}, "mlp": mlp}


def latent(heads, dim, rot_dim, vdim, kv_rank, scale, window, base=10000.0, mlp=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                      "mask": {"size": window}, "rot": {"base": base, "dims": rot_dim}}, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def loop(start, stop, times):
    return {"start": start, "stop": stop, "times": times}


PEP_A = {   # a looped pair in the middle; a window shorter than a page; a layer without a feed-forward
    "architecture": "Peponex", "vocab": 131, "width": 96, "norm": {"eps": 1e-5}, "logit_softcap": 6.0, "token_side": {"dim": 20},
    "loop": loop(1, 3, 2),
    "layers": [wkv(3, 16, 12, dense(136)),
               lightning(2, 24, 40, (0.5, 0.97), moe(5, 2, 40)),
               latent(3, 24, 8, 40, 40, 0.3, 37, mlp=moe(3, 1, 24)),
               wkv(2, 32, 20, None)],
    "torch_dtype": "bfloat16",
}

PEP_B = {   # all layers three times; odd widths; no second embedding, no bend; a window of one page; every expert chosen
    "architecture": "Peponex", "vocab": 90, "width": 72, "norm": {"eps": 1e-6}, "loop": loop(0, 3, 3),
    "layers": [latent(2, 12, 6, 20, 18, 0.35, 64, base=500.0, mlp=moe(3, 3, 20)),
               lightning(3, 10, 18, (0.2, 0.9, 0.999), dense(50)),
               wkv(5, 8, 3, moe(4, 1, 30))],
    "torch_dtype": "bfloat16",
}

PEP_C = {   # head shapes that the matrix-core kernels take (keys of 128, 64 and 192 dimensions), windows over page borders
    "architecture": "Peponex", "vocab": 190, "width": 128, "norm": {"eps": 1e-5}, "logit_softcap": 12.0, "token_side": {"dim": 32},
    "loop": loop(2, 5, 2),
    "layers": [latent(4, 64, 64, 64, 64, 0.1, 100, mlp=dense(96)),
               wkv(2, 64, 16, moe(8, 3, 64)),
               lightning(2, 64, 128, (0.93, 0.998), moe(4, 2, 48)),
               latent(6, 32, 32, 80, 96, 0.12, 65, base=2000.0, mlp=dense(64)),
               latent(2, 128, 64, 128, 128, 0.08, 193, mlp=None),
               lightning(1, 128, 64, (0.99,), dense(72))],
    "torch_dtype": "bfloat16",
}

PEP_D = {   # one head each, a decay of one, a loop of one pass, a window longer than the sequences
    "architecture": "Peponex", "vocab": 67, "width": 48, "norm": {"eps": 1e-5}, "logit_softcap": 9.0, "token_side": {"dim": 8},
    "loop": loop(1, 2, 1),
    "layers": [lightning(1, 16, 16, (1.0,), None),
               latent(1, 8, 8, 16, 24, 0.4, 1000, base=100.0, mlp=moe(1, 1, 24))],
    "torch_dtype": "bfloat16",
}

PEP_E = {   # no loop; a window of a single key (itself); the last layer is attention
    "architecture": "Peponex", "vocab": 75, "width": 64, "norm": {"eps": 1e-5}, "token_side": {"dim": 24},
    "layers": [wkv(1, 48, 7, dense(40)),
               latent(2, 16, 16, 24, 32, 0.3, 1, mlp=moe(6, 4, 16)),
               latent(3, 8, 24, 8, 16, 0.3, 130, mlp=dense(33))],
    "torch_dtype": "bfloat16",
}

ALL = {"pep_a": PEP_A, "pep_b": PEP_B, "pep_c": PEP_C, "pep_d": PEP_D, "pep_e": PEP_E}
