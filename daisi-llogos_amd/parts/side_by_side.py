"""Two mixers that read the same rows, each behind a norm of its own on its output:

    out = scale * ( norm(left(h)) * w_left + norm(right(h)) * w_right ) / 2

norm(x) = x / sqrt(mean(x^2) + eps) over the model's width.  Each mixer keeps what it keeps (pages, a state)
as it would alone.  Both outputs, which may come as partial sums of a split product, their norms, the sum with the
stream and the norm that reads the stream next are one kernel (ops.kernels.pair_norm).

The two mixers depend on the rows alone, so in steps of few rows, whose kernels are short and wait for one another, the
left one is queued on a second stream beside the right one (inside a captured step the two become branches of the
graph); both streams meet before the outputs do.  Every use of the second stream begins by waiting for the first, so
memory that either stream's allocator hands out again is no longer read by the other.  It pays where both mixers stream
large matrices (8 layer runs at 4,096 wide, 84 MB in the left mixer, with a mixture's shared expert beside its others
likewise: batch 1 1,646 -> 1,480 us a step, batch 8 2,866 -> 2,671; at 2,048 wide 1,016 -> 1,031 and 1,355 -> 1,359), so it
is taken from `side_bytes` of matrices in the left mixer on.  `LLOGOS_PARALLEL_STREAMS=0` keeps everything on one stream."""
from __future__ import annotations

import os
from typing import Callable, List, Optional, Tuple

import torch

from ..ops import kernels as K
from .base import MIXERS, LayerCache, Mixer, NormedAhead, Part, Residual, Runtime, StepContext, TensorSpec, make, mark, register_mixer
from .norm import RMSNorm


@register_mixer("side_by_side")
class SideBySide(Mixer):
    adds_to_residual = True
    takes_caches = True
    side_rows = 0 if os.environ.get("LLOGOS_PARALLEL_STREAMS", "1") == "0" else 64     # steps of up to so many rows use the second stream
    side_bytes = 40 << 20        # ... when the left mixer's matrices take at least so many bytes
    _side_streams = {}

    def __init__(self, hidden: int, left: Tuple[str, dict], right: Tuple[str, dict], left_norm: str, right_norm: str, eps: float,
                 out_scale: float = 1.0):
        """left, right: (kind, parameters) of the two mixers; left_norm, right_norm: names of the norms' weights."""
        self.hidden, self.eps, self.out_scale = int(hidden), float(eps), float(out_scale)
        self.left, self.right = (make(MIXERS, "mixer", kind, **params) for kind, params in (left, right))
        for m in (self.left, self.right):
            if m.takes_float32_rows:
                raise ValueError("a mixer that wants its rows as float32 is not built beside another")
        self.norm_names = (left_norm, right_norm)
        self.norm_w: List[torch.Tensor] = []
        self.takes_normed_rows = self.left.takes_normed_rows and self.right.takes_normed_rows

    @property
    def graph_safe(self) -> bool:
        return self.left.graph_safe and self.right.graph_safe

    def cache_parts(self) -> List[Part]:
        return self.left.cache_parts() + self.right.cache_parts()

    def tensor_specs(self) -> List[TensorSpec]:
        return self.left.tensor_specs() + self.right.tensor_specs() + [TensorSpec(n, (self.hidden,), "norm") for n in self.norm_names]

    def bind(self, get: Callable[[str], Optional[torch.Tensor]], rt: Runtime) -> None:
        super().bind(get, rt)
        self.left.bind(get, rt)
        self.right.bind(get, rt)
        # half of the sum, and the factor on the output, stand in the weights
        self._left_bytes = self.left.weight_bytes()
        self.norm_w = [get(n).to(device=rt.device, dtype=torch.float32).contiguous() * (0.5 * self.out_scale) for n in self.norm_names]

    def weight_bytes(self) -> int:
        return super().weight_bytes() + sum(w.numel() * w.element_size() for w in self.norm_w)

    def forward(self, ctx: StepContext, h, caches: List[LayerCache], residual: Optional[Residual] = None):
        n = len(self.left.cache_parts())
        side, rows = None, h if isinstance(h, torch.Tensor) else h.x
        if ctx.n_tokens <= self.side_rows and ctx.probe is None and self._left_bytes >= self.side_bytes:
            main = torch.cuda.current_stream(rows.device)
            side = self._side_streams.get(rows.device)
            if side is None:
                side = self._side_streams[rows.device] = torch.cuda.Stream(device=rows.device)
            side.wait_stream(main)                           # the rows are there
            with torch.cuda.stream(side):
                a = self.left.forward(ctx, h, self.left.caches_of(caches[:n]))
        else:
            a = self.left.forward(ctx, h, self.left.caches_of(caches[:n]))
        b = self.right.forward(ctx, h, self.right.caches_of(caches[n:]))
        if side is not None:
            torch.cuda.current_stream(rows.device).wait_stream(side)
        if residual is None:
            out = K.pair_norm(a, b, *self.norm_w, self.eps)
            mark(ctx, "pair_norm")
            return out
        nxt = residual.norm
        if isinstance(nxt, RMSNorm):
            dtype = torch.float32 if nxt.float32_rows else self.rt.dtype
            rows = K.pair_norm(a, b, *self.norm_w, self.eps, x=residual.x, next_w=nxt.weight, next_eps=nxt.eps, out_dtype=dtype)
            mark(ctx, "pair_norm")
            return NormedAhead(rows, nxt)
        K.pair_norm(a, b, *self.norm_w, self.eps, x=residual.x)
        mark(ctx, "pair_norm")
        return K.RowSquares(None, self.hidden)               # the stream is complete, nothing is left beside it
