"""A plain, slow implementation of the Zisedra decoder: whole sequences, no cache, NumPy float64,
one function for each mechanism.  It shares no code with the package under test: config.json is
read with ``json``, the weights with the ``safetensors`` library.

The design in short (x is the residual stream [T, width], positions p count from 0, m a constant):

    x = x0 = E[token]
    per layer:  x = x + m mixer(N1(x));   x = x + m ff(N2(x))
    logits = E N_final(x)

N(y) = y / sqrt(mean(y^2) + eps) * w.  Mixers: a recurrence by the gated delta rule (`delta`), or window
attention beside such a recurrence whose decay is one number a key channel (`parallel`: half the sum of
both outputs, each normed).  The feed-forward is a mixture of experts with clamped gates, chosen by the
sigmoids of a router's logits within the best groups, beside a shared expert.  A run of layers is gone
through several times: ahead of every pass x = W [x ; x0].
"""
from __future__ import annotations

import json
import math
import os

import numpy as np


# --------------------------------------------------------------------------
# mechanisms
# --------------------------------------------------------------------------

def unit_rows(x: np.ndarray, eps: float) -> np.ndarray:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    x = np.asarray(x, dtype=np.float64)
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def norm(x: np.ndarray, w: np.ndarray, eps: float) -> np.ndarray:
    return unit_rows(x, eps) * np.asarray(w, dtype=np.float64)


def sigmoid(z: np.ndarray) -> np.ndarray:
    return 1.0 / (1.0 + np.exp(-np.asarray(z, dtype=np.float64)))


def silu(z: np.ndarray) -> np.ndarray:
    z = np.asarray(z, dtype=np.float64)
    return z * sigmoid(z)


def softplus(z: np.ndarray) -> np.ndarray:
    z = np.asarray(z, dtype=np.float64)
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def length_one(x: np.ndarray) -> np.ndarray:
    """x / sqrt(sum(x^2) + 1e-6) over the last axis."""
    x = np.asarray(x, dtype=np.float64)
    return x / np.sqrt((x * x).sum(axis=-1, keepdims=True) + 1e-6)


def short_conv(x: np.ndarray, taps: np.ndarray) -> np.ndarray:
    """x [T, C], taps [C, n]: the last tap multiplies the row itself, the ones before it the rows before."""
    T, n = x.shape[0], taps.shape[1]
    out = np.zeros_like(x)
    for j in range(n):
        back = n - 1 - j
        if back < T:
            out[back:] += x[:T - back] * taps[:, j]
    return out


def delta_recurrence(q, k, v, beta, g, S=None):
    """q, k [T, H, D], v [T, H, V], beta [T, H], g [T, H, D]; S [H, D, V].  The state decays, the token writes what its
    key does not recall yet, then the token reads."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2])) if S is None else np.array(S, dtype=np.float64)
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum("hij,hi->hj", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = np.einsum("hij,hi->hj", S, q[t])
    return out, S


def delta_inputs(h, t, m: dict):
    """(q, k, v, beta, g) of the recurrence; one decay a head where the tensor `a` is, one a key channel where `a1`, `a2` are."""
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q, k, v = (silu(short_conv(h @ t[s].T, t[s + ".conv"])) for s in "qkv")
    of = np.arange(H) // (H // G)
    q = (length_one(q.reshape(T, G, D)) / math.sqrt(D))[:, of]
    k = length_one(k.reshape(T, G, D))[:, of]
    beta = sigmoid(h @ t["b"].T)
    if "a" in t:
        z = (h @ t["a"].T + t["dt_bias"])[:, :, None]
    else:
        z = ((h @ t["a1"].T) @ t["a2"].T + t["dt_bias"]).reshape(T, H, D)
    g = np.exp(-np.exp(t["A_log"])[None, :, None] * softplus(z)) * np.ones((T, H, D))
    return q, k, v.reshape(T, H, V), beta, g


def delta(h, t, m: dict, eps: float) -> np.ndarray:
    H, V = m["heads"], m["vdim"]
    o, _ = delta_recurrence(*delta_inputs(h, t, m))
    gate = silu(h @ t["g"].T) if "g" in t else sigmoid((h @ t["g1"].T) @ t["g2"].T)
    return (norm(o, t["norm"], eps).reshape(-1, H * V) * gate) @ t["o"].T


def frequencies(dims: int, base: float, scaling=None) -> np.ndarray:
    """base^(-2i / dims); with a scaling, long wavelengths are slowed by `factor`, short ones kept, those between mixed."""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling:
            wave = 2.0 * math.pi / f
            if wave > scaling["original"] / scaling["low"]:
                f = f / scaling["factor"]
            elif wave >= scaling["original"] / scaling["high"]:
                s = (scaling["original"] / wave - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return np.array(out)


def rotate(x: np.ndarray, positions, f: np.ndarray) -> np.ndarray:
    """x [T, heads, n]: dimensions 2i and 2i + 1 are a pair turned by p * f_i; those behind 2 len(f) pass."""
    x = np.array(x, dtype=np.float64)
    a = (np.asarray(positions, dtype=np.float64)[:, None] * f[None, :])[:, None, :]
    u, v = x[..., 0:2 * len(f):2].copy(), x[..., 1:2 * len(f):2].copy()
    x[..., 0:2 * len(f):2] = u * np.cos(a) - v * np.sin(a)
    x[..., 1:2 * len(f):2] = v * np.cos(a) + u * np.sin(a)
    return x


def window_softmax(scores: np.ndarray, size: int) -> np.ndarray:
    """Row i sees columns i - size + 1 .. i."""
    i, j = np.arange(scores.shape[0])[:, None], np.arange(scores.shape[1])[None, :]
    s = np.where((i - j >= 0) & (i - j < size), scores, -np.inf)
    e = np.exp(s - s.max(axis=1, keepdims=True))
    return e / e.sum(axis=1, keepdims=True)


def window_attention(h, t, m: dict) -> np.ndarray:
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q, k, v = (h @ t[s].T + t[s + ".b"] for s in "qkv")
    f = frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling")) if m.get("rot") else np.zeros(0)
    q = rotate(q.reshape(T, H, D), np.arange(T), f)
    k = rotate(k.reshape(T, G, D), np.arange(T), f)
    v = v.reshape(T, G, V)
    out = np.zeros((T, H, V))
    for head in range(H):
        kv = head // (H // G)
        out[:, head] = window_softmax((q[:, head] @ k[:, kv].T) * m["scale"], m["mask"]["size"] if m.get("mask") else T) @ v[:, kv]
    return out.reshape(T, H * V) @ t["o"].T


def side_by_side(h, t, m: dict, eps: float) -> np.ndarray:
    left = window_attention(h, part(t, "left."), m["left"])
    right = delta(h, part(t, "right."), m["right"], eps)
    return 0.5 * (norm(left, t["left.out"], eps) + norm(right, t["right.out"], eps))


def clamped_ff(h, t, limit: float) -> np.ndarray:
    """The gate is bounded above, the up half on both sides; a logistic of 1.702 times the gate; one is added to up."""
    g = np.minimum(h @ t["gate"].T, limit)
    u = np.clip(h @ t["up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ t["down"].T


def choose(s: np.ndarray, top: int, count: int, keep: int) -> np.ndarray:
    """The `top` largest scores of one token within the `keep` best of `count` groups (a group's score: its two largest)."""
    groups = s.reshape(count, -1)
    score = np.sort(groups, axis=1)[:, ::-1][:, :2].sum(axis=1)
    kept = np.argsort(-score, kind="stable")[:keep]
    masked = np.full_like(groups, -np.inf)
    masked[kept] = groups[kept]
    return np.argsort(-masked.reshape(-1), kind="stable")[:top]


def mixture(h, t, m: dict) -> np.ndarray:
    r = m["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    s = sigmoid(h @ t["router"].T)
    out = np.zeros_like(h)
    for i in range(h.shape[0]):
        for e in choose(s[i], r["top"], groups["count"], groups["keep"]):
            out[i] += s[i, e] * clamped_ff(h[i:i + 1], part(t, f"e{e}."), m["expert"]["limit"])[0]
    if m.get("shared"):
        out += clamped_ff(h, part(t, "shared."), m["shared"]["limit"])
    return out


# --------------------------------------------------------------------------
# the whole model
# --------------------------------------------------------------------------

def part(tensors: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def layer(x, t, entry: dict, eps: float, mult: float) -> np.ndarray:
    mixer = delta if entry["type"] == "delta" else side_by_side
    x = x + mult * mixer(norm(x, t["norm1"], eps), part(t, "mix."), entry["mixer"], eps)
    if entry["mlp"] is not None:
        x = x + mult * mixture(norm(x, t["norm2"], eps), part(t, "mlp."), entry["mlp"])
    return x


def runs(cfg: dict) -> list:
    """The layers in the order in which they run: (layer, whether a pass starts with it)."""
    n, lo = len(cfg["layers"]), cfg.get("loop")
    if not lo:
        return [(i, False) for i in range(n)]
    order = [(i, False) for i in range(lo["start"])]
    for _ in range(lo["times"]):
        order += [(i, i == lo["start"]) for i in range(lo["start"], lo["stop"])]
    return order + [(i, False) for i in range(lo["stop"], n)]


def forward(cfg: dict, w: dict, tokens, layers=None) -> np.ndarray:
    """Logits [T, vocab]; with a list `layers` the stream after every layer run is appended to it."""
    eps, mult = cfg["norm"]["eps"], cfg.get("residual_mult", 1.0)
    x = x0 = w["embed"][np.asarray(tokens)]
    for i, enters in runs(cfg):
        if enters:
            x = np.concatenate([x, x0], axis=1) @ w["loop.in"].T
        x = layer(x, part(w, f"l{i}."), cfg["layers"][i], eps, mult)
        if layers is not None:
            layers.append(x.copy())
    return norm(x, w["final.norm"], eps) @ w["embed"].T


def generate_greedy(cfg: dict, w: dict, prompt, n: int) -> list:
    """n tokens, each the first largest logit after everything before it (the whole sequence is run again each time)."""
    seq, out = list(prompt), []
    for _ in range(n):
        out.append(int(np.argmax(forward(cfg, w, seq)[-1])))
        seq.append(out[-1])
    return out


def load(folder: str):
    """(config, weights as float64) of a model folder."""
    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json")) as fh:
        cfg = json.load(fh)
    return cfg, {k: v.double().numpy() for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
