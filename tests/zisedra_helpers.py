"""Shared by the Zisedra tests: model folders of the small configurations (random weights, with the
attention's query and key matrices scaled up so that it is sharp and a lost or extra key or a wrong position shows), the
plain implementation's logits, and the bounds.

Every model comes in two forms.  In the first the router's choice follows the input: a token whose two best
candidates lie closer than rounding moves them changes its experts, which in 32-bit happens about never and in
bfloat16 (a stream that is a hundredth off) to a token in a hundred, whose logits and all later ones then have
nothing to do with the plain result.  The float32 tests use that form.  The bfloat16 tests of whole models use the
second, in which every token's stream has one large channel and the routers read little else, with weights far
apart: the same experts for every token, whose scores still follow the input.  That bfloat16 follows the same rules
for the choice is tested on the feed-forward alone, row by row."""
import functools
import importlib
import os
import tempfile

import numpy as np
import torch

import zisedra_configs as zc
import plain_zisedra as pz

llogos = importlib.import_module("daisi-llogos_amd")
_tmp = tempfile.TemporaryDirectory(prefix="llogos_test_zisedra_")
DTYPES = ["float32", "bfloat16"]
# float32: the engine against float64 arithmetic, relative to the largest logit.  bfloat16: rounding of the
# matrix products' inputs; the bound is loose, and what must not happen (a key too few, a lost state) is
# asserted in float32.
TOL = {"float32": 2e-4, "bfloat16": 0.12}


def sharpen(tensors: dict, fixed_choice: bool = False) -> dict:
    for k in sorted(tensors):
        t = tensors[k]
        if k.endswith((".mix.left.q", ".mix.left.k")):
            tensors[k] = (t.float() * 2.5).to(t.dtype)
        if k.endswith((".left.q.b", ".left.k.b", ".left.v.b")):      # (biases that show)
            tensors[k] = (t.float() * 4.0).to(t.dtype)
        if k == "embed":
            tensors[k] = t = (t.float() * 6.0).to(t.dtype)
        if fixed_choice and k == "embed":
            t[:, 0] = 8.0
        if fixed_choice and k == "loop.in":                     # the large channel passes the head of a pass as it is
            t[0, :] = 0.0
            t[:, 0] = 0.0
            t[:, t.shape[0]] = 0.0
            t[0, 0] = 1.0
        if fixed_choice and k.endswith(".mlp.router"):
            order = np.random.default_rng(len(k) * 1000 + t.shape[0] + int(k[1:k.index(".")])).permutation(t.shape[0])
            new = t.float() * 0.05
            new[:, 0] = 0.3 * (torch.tensor(order).float() - (t.shape[0] - 1) / 2.0)
            tensors[k] = new.to(t.dtype)
    return tensors


def fixed_choice(dtype: str) -> bool:
    return dtype == "bfloat16"


@functools.lru_cache(maxsize=None)
def folder(name: str, seed: int = 5, dtype: str = "float32") -> str:
    from safetensors.torch import load_file, save_file
    path = os.path.join(_tmp.name, f"{name}_{seed}_{'fixed' if fixed_choice(dtype) else 'free'}")
    llogos.write_random_model(path, zc.ALL[name], seed=seed, std=0.08)
    file = os.path.join(path, "model.safetensors")
    save_file(sharpen(load_file(file), fixed_choice(dtype)), file)
    return path


@functools.lru_cache(maxsize=None)
def plain(name: str, seed: int = 5, dtype: str = "float32"):
    return pz.load(folder(name, seed, dtype))


@functools.lru_cache(maxsize=None)
def plain_logits(name: str, tokens: tuple, seed: int = 5, dtype: str = "float32") -> np.ndarray:
    cfg, w = plain(name, seed, dtype)
    return pz.forward(cfg, w, list(tokens))


def tokens(name: str, n: int, seed: int) -> tuple:
    rng = np.random.default_rng(seed)
    return tuple(int(t) for t in rng.integers(0, zc.ALL[name]["vocab"], size=n))


def engine(name: str, dtype: str, max_tokens: int = 1024, n_slots: int = 4, seed: int = 5, **options):
    return llogos.Engine.from_folder(folder(name, seed, dtype), dtype=dtype, max_tokens=max_tokens, n_slots=n_slots, **options)


def distance(got, want) -> float:
    """Largest difference of the logits, relative to the largest logit's size, without what all logits of a position share
    (the table's large channel is the head's too)."""
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    assert got.shape == want.shape, f"shape {got.shape} vs {want.shape}"
    assert np.isfinite(got).all(), "not finite"
    got, want = got - got.mean(axis=-1, keepdims=True), want - want.mean(axis=-1, keepdims=True)
    return float(np.abs(got - want).max() / max(1e-9, np.abs(want).max()))


def close(got, want, dtype: str, what: str = "") -> float:
    d = distance(got, want)
    assert d <= TOL[dtype], f"{what}: relative error {d:.3e} > {TOL[dtype]:.1e} ({dtype})"
    return d
