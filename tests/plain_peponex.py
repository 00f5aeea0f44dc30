"""A plain, slow implementation of the Peponex decoder: whole sequences, no cache, NumPy float64,
one function for each mechanism.  It shares no code with the package under test: config.json is
read with ``json``, the weights with the ``safetensors`` library.

The design in short (x is the residual stream [T, width], positions p count from 0):

    x = x0 = E[token]
    per layer:  x = x + mixer(N1(x));   x = x + ff(N2(x));   x = x + unit(P (gelu(G x) * e_token)) * n
    logits = cap * tanh(W_head N_final(x) / cap)

N(y) = y / sqrt(mean(y^2) + eps) * w.  Mixers: a recurrence with a matrix state per head whose decay is
made from the token (`wkv`), a recurrence with a fixed decay per head (`lightning`), and attention through
a low-rank latent over a sliding window (`latent_attention`).  Feed-forwards: SwiGLU, or a mixture of
SwiGLU experts whose router weighs the chosen experts' inputs by the sigmoid of their logits.  The last
term of a layer takes the layer's own part e of a second embedding of the token.  A run of layers is gone
through several times: ahead of pass t the stream gets step[t], from the second pass on also x0.
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


def gelu_tanh(z: np.ndarray) -> np.ndarray:
    z = np.asarray(z, dtype=np.float64)
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def before(h: np.ndarray) -> np.ndarray:
    """The row before every row; zeros before the first."""
    out = np.zeros_like(h)
    out[1:] = h[:-1]
    return out


def wkv_recurrence(r, k, v, w, u, S=None):
    """r, k, w [T, H, D], v [T, H, D], u [H, D]; S [H, D (key), D (value)].  A token's output sees the state
    before it and its own product with the bonus u; then every key channel decays and the product joins."""
    T, H, D = r.shape
    S = np.zeros((H, D, v.shape[2])) if S is None else np.array(S, dtype=np.float64)
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hi,hij->hj", r[t], S + u[:, :, None] * kv)
        S = w[t][:, :, None] * S + kv
    return out, S


def wkv(h, t, m: dict, eps: float) -> np.ndarray:
    H, D = m["heads"], m["dim"]
    T = h.shape[0]
    prev = before(h)
    mix = {s: h + (prev - h) * t["mu." + s] for s in "rkvgw"}
    heads = lambda y: y.reshape(T, H, D)
    r, k, v = (heads(mix[s] @ t[s].T) for s in "rkv")
    w = heads(np.exp(-np.exp(np.tanh(mix["w"] @ t["w1"].T) @ t["w2"].T + t["w0"])))
    o, _ = wkv_recurrence(r, k, v, w, t["u"])
    o = unit_rows(o, eps).reshape(T, H * D) * t["norm"] * silu(mix["g"] @ t["g"].T)
    return o @ t["o"].T


def decay_recurrence(q, k, v, decay, S=None):
    """q, k [T, H, D], v [T, H, V], decay [H]; S [H, D, V].  The state decays, the token's product joins, then the
    token reads it."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2])) if S is None else np.array(S, dtype=np.float64)
    decay = np.asarray(decay, dtype=np.float64)[:, None, None]
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        S = decay * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hi,hij->hj", q[t], S)
    return out, S


def lightning(h, t, m: dict, eps: float) -> np.ndarray:
    H, D, V = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q, k = (silu(h @ t[s].T).reshape(T, H, D) for s in "qk")
    v = silu(h @ t["v"].T).reshape(T, H, V)
    o, _ = decay_recurrence(q, k, v, m["decay"])
    return (norm(o.reshape(T, H * V), t["norm"], eps) * sigmoid(h @ t["g"].T)) @ t["o"].T


def rotate(x: np.ndarray, positions, dims: int, base: float) -> np.ndarray:
    """x [T, ..., n]: of the first `dims` dimensions, i and i + dims / 2 are a pair turned by p * base^(-2i / dims)."""
    x = np.array(x, dtype=np.float64)
    half = dims // 2
    f = np.array([float(base) ** (-2.0 * i / dims) for i in range(half)])
    a = np.asarray(positions, dtype=np.float64)[:, None] * f[None, :]
    a = a.reshape((x.shape[0],) + (1,) * (x.ndim - 2) + (half,))
    u, v = x[..., :half].copy(), x[..., half:dims].copy()
    x[..., :half] = u * np.cos(a) - v * np.sin(a)
    x[..., half:dims] = v * np.cos(a) + u * np.sin(a)
    return x


def window_softmax(scores: np.ndarray, size: int) -> np.ndarray:
    """Row i sees columns i - size + 1 .. i."""
    i, j = np.arange(scores.shape[0])[:, None], np.arange(scores.shape[1])[None, :]
    s = np.where((i - j >= 0) & (i - j < size), scores, -np.inf)
    e = np.exp(s - s.max(axis=1, keepdims=True))
    return e / e.sum(axis=1, keepdims=True)


def latent_attention(h, t, m: dict, eps: float) -> np.ndarray:
    H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    T = h.shape[0]
    p = np.arange(T)
    q = (h @ t["q"].T).reshape(T, H, d + r)
    kv = h @ t["dkv"].T
    c = norm(kv[:, :rank], t["dkv.norm"], eps)
    q_rot = rotate(q[..., d:], p, m["rot"]["dims"], m["rot"]["base"])
    k_rot = rotate(kv[:, rank:], p, m["rot"]["dims"], m["rot"]["base"])          # one for all heads
    k = (c @ t["uk"].T).reshape(T, H, d)
    v = (c @ t["uv"].T).reshape(T, H, dv)
    out = np.zeros((T, H, dv))
    for head in range(H):
        s = (q[:, head, :d] @ k[:, head].T + q_rot[:, head] @ k_rot.T) * m["scale"]
        out[:, head] = window_softmax(s, m["mask"]["size"]) @ v[:, head]
    return out.reshape(T, H * dv) @ t["o"].T


def gated_ff(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(h, router_w, top: int):
    """(chosen [T, top] experts, weights [T, top]): the largest sigmoid scores, as they are."""
    s = sigmoid(np.asarray(h, dtype=np.float64) @ np.asarray(router_w, dtype=np.float64).T)
    chosen = np.argsort(-s, axis=1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=1)


def mixture(h, t, mlp: dict):
    """The weight is on the expert's input."""
    h = np.asarray(h, dtype=np.float64)
    chosen, weights = route(h, t["router"], mlp["router"]["top"])
    out = np.zeros_like(h)
    for row in range(h.shape[0]):
        for e, w in zip(chosen[row], weights[row]):
            out[row] += gated_ff(w * h[row:row + 1], t[f"e{e}.gate"], t[f"e{e}.up"], t[f"e{e}.down"])[0]
    return out


def token_side(x, e, t, eps: float) -> np.ndarray:
    """What the layer's own part e [T, dim] of the second embedding adds to the stream x."""
    return norm((gelu_tanh(x @ t["gate"].T) * e) @ t["proj"].T, t["norm"], eps)


def softcap(z: np.ndarray, cap) -> np.ndarray:
    return z if not cap else cap * np.tanh(z / cap)


# --------------------------------------------------------------------------
# the model
# --------------------------------------------------------------------------

MIXERS = {"wkv": wkv, "lightning": lightning, "latent_attention": latent_attention}


def load(folder: str):
    """(config dict, {name: float64 array}) of a model folder."""
    import torch
    from safetensors import safe_open
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    tensors = {}
    with safe_open(os.path.join(folder, "model.safetensors"), framework="pt") as f:
        for name in f.keys():
            tensors[name] = f.get_tensor(name).to(torch.float64).numpy()
    return cfg, tensors


def part(tensors: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def layer(cfg: dict, tensors: dict, i: int, x: np.ndarray, tokens) -> np.ndarray:
    L, eps, p = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    x = x + MIXERS[L["type"]](norm(x, tensors[p + "norm1"], eps), part(tensors, p + "mix."), L["mixer"], eps)
    mlp = L.get("mlp")
    if mlp:
        t = part(tensors, p + "mlp.")
        h = norm(x, tensors[p + "norm2"], eps)
        x = x + (gated_ff(h, t["gate"], t["up"], t["down"]) if mlp["kind"] == "dense" else mixture(h, t, mlp))
    side = cfg.get("token_side")
    if side:
        e = tensors["side.embed"][np.asarray(tokens)][:, i * side["dim"]:(i + 1) * side["dim"]]
        x = x + token_side(x, e, part(tensors, p + "side."), eps)
    return x


def runs(cfg: dict):
    """(layer, pass number or None) in the order in which the layers run; the number stands at a pass's first layer."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return out + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg: dict, tensors: dict, tokens, streams: list = None) -> np.ndarray:
    """Logits [T, vocab] of one whole sequence.  streams: a list that receives the stream after every layer run."""
    x0 = tensors["embed"][np.asarray(tokens)]
    x = x0
    for i, number in runs(cfg):
        if number is not None:
            x = x + tensors["loop.step"][number] + (x0 if number > 0 else 0.0)
        x = layer(cfg, tensors, i, x, tokens)
        if streams is not None:
            streams.append(x.copy())
    z = norm(x, tensors["final.norm"], cfg["norm"]["eps"]) @ tensors["head"].T
    return softcap(z, cfg.get("logit_softcap"))


def generate_greedy(cfg: dict, tensors: dict, prompt, n: int) -> list:
    """n tokens, each the first largest logit after everything before it (the whole sequence is run again each time)."""
    seq, out = list(prompt), []
    for _ in range(n):
        tok = int(np.argmax(forward(cfg, tensors, seq)[-1]))
        out.append(tok)
        seq.append(tok)
    return out
