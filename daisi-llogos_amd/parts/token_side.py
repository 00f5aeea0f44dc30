"""A second embedding of the token that enters the stream behind every layer, each layer taking its own
part of the token's row:

    e = E_side[token][index * dim : (index + 1) * dim]
    g = gelu_tanh(W_gate x) * e;   y = W_proj g;   x <- x + y / sqrt(mean(y^2) + eps) * w

x is the stream itself, not normed.  A layer's columns of the table are kept as a table of their own, so
the layers share nothing and hold the whole once between them."""
from __future__ import annotations

from typing import Callable, List, Optional

import torch

from ..ops import kernels as K
from .base import Norm, NormedAhead, Part, Runtime, StepContext, TensorSpec, mark, register_part
from .linear import Linear
from .norm import RMSNorm, add_normed


@register_part("token_side")
class TokenSide(Part):
    # the product that completes the stream may leave its rows (as a norm's rows of weight one) for the gate's product
    takes_row_squares = True
    plain_rows = True

    def __init__(self, prefix: str, embedding: str, hidden: int, vocab: int, dim: int, index: int, count: int, eps: float, suffix: str = ""):
        if not 0 <= index < count:
            raise ValueError(f"part {index} of {count}")
        self.prefix, self.table_name, self.hidden, self.vocab = prefix, embedding, int(hidden), int(vocab)
        self.dim, self.index, self.count = int(dim), int(index), int(count)
        self.gate = Linear([prefix + "gate"], hidden, [self.dim], suffix=suffix)
        self.proj = Linear([prefix + "proj"], self.dim, [hidden], suffix=suffix)
        self.norm = RMSNorm(name=prefix + "norm", width=hidden, eps=eps, suffix=suffix)
        self.table: Optional[torch.Tensor] = None
        self.ones: Optional[torch.Tensor] = None

    def tensor_specs(self) -> List[TensorSpec]:
        return [TensorSpec(self.table_name, (self.vocab, self.count * self.dim), "table")] + self.gate.tensor_specs() \
            + self.proj.tensor_specs() + self.norm.tensor_specs()

    def bind(self, get: Callable[[str], Optional[torch.Tensor]], rt: Runtime) -> None:
        super().bind(get, rt)
        for part in (self.gate, self.proj, self.norm):
            part.bind(get, rt)
        columns = get(self.table_name)[:, self.index * self.dim:(self.index + 1) * self.dim]
        self.table = columns.to(device=rt.device, dtype=rt.dtype).contiguous()
        self.ones = torch.ones(self.hidden, dtype=torch.float32, device=rt.device)

    def weight_bytes(self) -> int:
        return sum(p.weight_bytes() for p in (self.gate, self.proj, self.norm))      # (of the table a step reads a row a token)

    def row_weight(self) -> Optional[torch.Tensor]:
        return self.ones

    def forward(self, ctx: StepContext, x: torch.Tensor, pending, next_norm: Optional[Norm] = None):
        """x: the float32 stream; pending: what it still lacks, or what the product that completed it left.
        Returns (x, NormedAhead) with x complete and `next_norm`'s rows made on the way where they can be."""
        if isinstance(pending, K.RowSquares):
            rows = pending.unscaled if pending.norm_w is self.ones else None
            pending = None
        else:
            rows = None
            if isinstance(pending, NormedAhead):
                pending = None
        if rows is None:
            rows = K.stream_add(x, pending, rows_dtype=self.rt.dtype)
        g = K.gated_lookup(self.gate.product(rows, f32_ok=True), self.table, ctx.ids, self.rt.dtype)
        mark(ctx, "side_gate")
        y = self.proj.product(g, f32_ok=True)
        mark(ctx, "side_proj")
        out = add_normed(x, y, self.norm, next_norm)
        mark(ctx, "norm")
        return x, out
