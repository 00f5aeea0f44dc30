"""A recurrent mixer with a matrix state per head whose decay is one fixed number a head (lightning
attention):

    q, k, v = silu(W_q h), silu(W_k h), silu(W_v h)         (heads x dim, heads x dim, heads x v_dim)
    S <- decay S + k_t v_t^T;   o_t = S^T q_t               per head
    out     = W_o ( norm([o of all heads]) * sigmoid(W_g h) )

The four projections that read h are one stacked product.  A sequence's state is S of every head,
float32, in one state row per cache slot: [heads * dim * v_dim]."""
from __future__ import annotations

from typing import Callable, List, Optional, Sequence

import torch

from ..ops import kernels as K
from .base import LayerCache, Mixer, Residual, Runtime, StateSpec, StepContext, TensorSpec, mark, register_mixer
from .linear import Linear


@register_mixer("lightning")
class Lightning(Mixer):
    graph_safe = True
    adds_to_residual = True

    def __init__(self, prefix: str, hidden: int, n_heads: int, head_dim: int, v_dim: int, decay: Sequence[float], eps: float,
                 suffix: str = ""):
        self.prefix, self.hidden, self.suffix = prefix, int(hidden), suffix
        self.n_heads, self.head_dim, self.v_dim = int(n_heads), int(head_dim), int(v_dim)
        self.decay, self.eps = tuple(float(d) for d in decay), float(eps)
        if len(self.decay) != self.n_heads:
            raise ValueError(f"{len(self.decay)} decays for {self.n_heads} heads")
        if self.head_dim > K.DECAY_SCAN_MAX_DIM:
            raise ValueError(f"a head of {self.head_dim} key channels is more than the recurrence takes ({K.DECAY_SCAN_MAX_DIM})")
        inner_k, inner_v = self.n_heads * self.head_dim, self.n_heads * self.v_dim
        self.inner = inner_v
        # q, k and v in front (what the recurrence reads), the gate's logits behind them
        self.inp = Linear([prefix + s for s in ("q", "k", "v", "g")], hidden, [inner_k, inner_k, inner_v, inner_v], suffix=suffix)
        self.o = Linear([prefix + "o"], inner_v, [hidden], suffix=suffix)
        self.norm_w = self.powers = None

    def state_spec(self) -> StateSpec:
        return StateSpec((self.n_heads * self.head_dim * self.v_dim,), torch.float32)

    def tensor_specs(self) -> List[TensorSpec]:
        return self.inp.tensor_specs() + self.o.tensor_specs() + [TensorSpec(self.prefix + "norm", (self.inner,), "norm")]

    def bind(self, get: Callable[[str], Optional[torch.Tensor]], rt: Runtime) -> None:
        super().bind(get, rt)
        self.inp.bind(get, rt)
        self.o.bind(get, rt)
        self.norm_w = get(self.prefix + "norm").to(device=rt.device, dtype=torch.float32).contiguous()
        self.powers = K.decay_powers(self.decay, rt.device)

    def matrix_elements(self) -> int:
        # (a token's products with the state count like a matrix of that size: one to join it, one to read it)
        return super().matrix_elements() + 2 * self.n_heads * self.head_dim * self.v_dim

    def forward(self, ctx: StepContext, h: torch.Tensor, cache: LayerCache, residual: Optional[Residual] = None):
        if cache.state is None:
            raise RuntimeError("the recurrent mixer needs its per-sequence state")
        rows = self.inp.product(h, f32_ok=True)               # [(parts,) T, q | k | v | g]
        if rows.dtype != torch.float32:
            rows = K.sum_parts(rows, None, torch.float32)
        mark(ctx, "projections")
        o = K.decay_scan(ctx, rows, self.powers, cache.state, self.n_heads, self.head_dim, self.v_dim)
        mark(ctx, "recurrence")
        gate = rows[..., rows.shape[-1] - self.inner:]
        y = K.gated_row_norm(o, self.norm_w, gate, self.eps, self.rt.dtype)
        mark(ctx, "head_norm")
        out = self.o.add_to(y, residual) if residual is not None else None
        if out is None:
            out = self.o.product(y, f32_ok=True)
        mark(ctx, "o")
        return out
