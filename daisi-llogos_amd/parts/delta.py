"""A recurrent mixer with a matrix state per head whose writes replace what the state recalls already
(the gated delta rule):

    q, k, v = silu(conv(W_q h)), silu(conv(W_k h)), silu(conv(W_v h))     conv: a short causal convolution over time on
                                                                          every channel; G key heads, H value heads
    q, k    <- q / |q| / sqrt(dim), k / |k|                               per head, |x| = sqrt(sum(x^2) + 1e-6)
    beta    = sigmoid(W_b h)                                              one a head
    g       = exp(-exp(A_log) * softplus(z + dt_bias))                    z = W_a h, one a head, or
                                                                          z = W_a2 W_a1 h, one a head and key channel
    S <- diag(g) S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q per head (head h: key head h // (H / G))
    out     = W_o ( norm(o) per head * act(gate) )                        gate = W_g h or W_g2 W_g1 h; act silu or sigmoid

All projections that read h are one stacked product; with a decay or a gate of low rank their second
matrices are one more, on both low-rank rows side by side.  A sequence's state is S of every head and the last
rows of [q | k | v] in front of the convolution, float32, in one state row per cache slot."""
from __future__ import annotations

from typing import Callable, List, Optional

import torch

from ..ops import kernels as K
from .base import LayerCache, Mixer, Residual, Runtime, StateSpec, StepContext, TensorSpec, mark, register_mixer
from .linear import Linear


@register_mixer("delta")
class Delta(Mixer):
    graph_safe = True
    takes_normed_rows = True       # h goes into the stacked product alone
    adds_to_residual = True

    def __init__(self, prefix: str, hidden: int, n_heads: int, n_kv_heads: int, head_dim: int, v_dim: int, conv_taps: int, eps: float,
                 decay_rank: int = 0, gate_rank: int = 0, gate: str = "silu", out_scale: float = 1.0, suffix: str = ""):
        """decay_rank: 0 for one decay a head, else the inner width of a decay a key channel.  gate_rank: 0 for a gate with
        one matrix, else its inner width.  gate: its activation, silu or sigmoid.  out_scale: a factor on the output."""
        if n_heads % n_kv_heads:
            raise ValueError(f"{n_heads} heads are not a multiple of {n_kv_heads} key heads")
        if not (0 < head_dim <= K.DELTA_MAX_DIM and 0 < v_dim <= K.DELTA_MAX_V):
            raise ValueError(f"heads of {head_dim} key and {v_dim} value channels: at most {K.DELTA_MAX_DIM} and {K.DELTA_MAX_V}")
        if not 1 <= conv_taps <= K.MAX_CONV_TAPS:
            raise ValueError(f"a convolution of {conv_taps} taps is outside 1..{K.MAX_CONV_TAPS}")
        if gate not in ("silu", "sigmoid"):
            raise ValueError(f"unknown gate '{gate}' (silu, sigmoid)")
        self.prefix, self.hidden, self.suffix = prefix, int(hidden), suffix
        self.n_heads, self.n_kv_heads = int(n_heads), int(n_kv_heads)
        self.k_dim, self.v_dim, self.conv_taps, self.eps = int(head_dim), int(v_dim), int(conv_taps), float(eps)
        self.decay_rank, self.gate_rank, self.gate, self.out_scale = int(decay_rank), int(gate_rank), gate, float(out_scale)
        H, G, D, V = self.n_heads, self.n_kv_heads, self.k_dim, self.v_dim
        self.Wq, self.Wv = G * D, H * V
        n_decay = H * D if self.decay_rank else H
        names, outs = ["q", "k", "v"], [self.Wq, self.Wq, self.Wv]
        self.low: List[tuple] = []                           # (first matrix, second, rank, outputs) of the low-rank projections
        if self.decay_rank:
            self.low.append(("a1", "a2", self.decay_rank, n_decay))
        if self.gate_rank:
            self.low.append(("g1", "g2", self.gate_rank, self.Wv))
        for one, _, rank, _ in self.low:
            names.append(one)
            outs.append(rank)
        if not self.gate_rank:
            names.append("g")
            outs.append(self.Wv)
        if not self.decay_rank:
            names.append("a")
            outs.append(n_decay)
        names.append("b")
        outs.append(H)
        self._first = {n: sum(outs[:i]) for i, n in enumerate(names)}        # each projection's first column
        self.inp = Linear([prefix + n for n in names], hidden, outs, suffix=suffix)
        # the second matrices, block by block on the diagonal: one product over both low-rank rows
        self.low2 = Linear([prefix + "low"], sum(l[2] for l in self.low), [sum(l[3] for l in self.low)], suffix="") if self.low else None
        self.o = Linear([prefix + "o"], self.Wv, [hidden], suffix=suffix)
        self.shape = K.DeltaShape(H=H, G=G, D=D, V=V, taps=self.conv_taps, channelwise=bool(self.decay_rank), b_col=self._first["b"])
        self.conv_w = self.a_log = self.dt_bias = self.norm_w = None

    def state_spec(self) -> StateSpec:
        return StateSpec((self.shape.state_floats,), torch.float32)

    def tensor_specs(self) -> List[TensorSpec]:
        p, sh = self.prefix, self.shape
        specs = self.inp.tensor_specs() + self.o.tensor_specs()
        specs += [TensorSpec(p + n + ".conv", (w, self.conv_taps), "taps") for n, w in (("q", self.Wq), ("k", self.Wq), ("v", self.Wv))]
        specs += [TensorSpec(p + two + self.suffix, (n, rank), "matrix") for _, two, rank, n in self.low]
        specs += [TensorSpec(p + "A_log", (sh.H,), "a_log"), TensorSpec(p + "dt_bias", (sh.n_decay,), "dt_bias"),
                  TensorSpec(p + "norm", (self.v_dim,), "norm")]
        return specs

    def bind(self, get: Callable[[str], Optional[torch.Tensor]], rt: Runtime) -> None:
        super().bind(get, rt)
        self.inp.bind(get, rt)
        self.o.bind(get, rt)
        if self.low2 is not None:
            blocks = [get(self.prefix + two + self.suffix) for _, two, _, _ in self.low]
            self.low2.bind(lambda name: torch.block_diag(*blocks), rt)
        f32 = lambda name: get(self.prefix + name).to(device=rt.device, dtype=torch.float32).contiguous()
        self.conv_w = torch.cat([f32(n + ".conv") for n in ("q", "k", "v")], dim=0).t().contiguous()     # [taps, width]
        self.a_log, self.dt_bias = f32("A_log"), f32("dt_bias")
        self.norm_w = f32("norm") * self.out_scale           # (the output product is linear: a factor on it may stand here)

    def matrix_elements(self) -> int:
        # (a token's products with the state count like matrices of its size: to recall, to write, to read)
        blocks = sum(rank * n for _, _, rank, n in self.low)
        return self.inp.matrix_elements() + self.o.matrix_elements() + blocks + 3 * self.n_heads * self.k_dim * self.v_dim

    def forward(self, ctx: StepContext, h, cache: LayerCache, residual: Optional[Residual] = None):
        if cache.state is None:
            raise RuntimeError("the recurrent mixer needs its per-sequence state")
        sh, f32 = self.shape, torch.float32
        rows = self.inp.product(h, f32_ok=True)              # [(parts,) T, q | k | v | ...]
        if rows.dtype != f32:
            rows = K.sum_parts(rows, None, f32)
        low = None
        if self.low2 is not None:
            ranks = self.low2.in_features
            a = K.activation(rows, "none", self.rt.dtype, cols=ranks, first=self._first[self.low[0][0]])
            low = self.low2.product(a, f32_ok=True)          # [(parts,) T, z of every decay | gate]
            if low.dtype != f32:
                low = K.sum_parts(low, None, f32)
        z = low if self.decay_rank else rows[..., self._first["a"]:]
        gate = low[..., low.shape[-1] - self.Wv:] if self.gate_rank else rows[..., self._first["g"]:]
        mark(ctx, "projections")
        args = (ctx, sh, rows, self.conv_w, z, self.dt_bias, self.a_log)
        silu = self.gate == "silu"
        if ctx.is_decode and K.delta_step_threads(sh.D, sh.V):
            y = K.delta_step(*args, gate, silu, self.norm_w, self.eps, cache.state, self.rt.dtype)
            mark(ctx, "recurrence")
        else:
            act, logd, beta = K.delta_prepare(*args, cache.state)
            mark(ctx, "conv")
            o = K.delta_scan(ctx, sh, act, logd, beta, cache.state)
            mark(ctx, "recurrence")
            y = K.delta_out(o, gate, silu, self.norm_w, self.eps, sh.H, self.rt.dtype)
            mark(ctx, "head_norm")
        out = self.o.add_to(y, residual) if residual is not None else None
        if out is None:
            out = self.o.product(y, f32_ok=True)             # maybe in parts: whoever reads it adds them
        mark(ctx, "o")
        return out
