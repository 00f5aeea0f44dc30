"""The head of a pass through a run of layers that is gone through several times with the same
weights: the stream and the embedding output go through one matrix together, and the pass's own
vector is added,

    x <- W_in [x ; x0] [+ step[t]]         W_in [width, 2 width] (x first), step [times, width] (optional), t the pass

in front of the first layer of every pass, the first pass too.  `LoopAdd` is the form without a matrix."""
from __future__ import annotations

from typing import Callable, List, Optional

import torch

from ..ops import kernels as K
from .base import NormedAhead, Part, Runtime, StepContext, TensorSpec, register_part
from .linear import Linear


@register_part("loop_entry")
class LoopEntry(Part):
    def __init__(self, matrix: str, steps: Optional[str], width: int, times: int):
        """steps: the name of the passes' vectors, None for passes without."""
        self.width, self.times, self.steps_name = int(width), int(times), steps
        self.mix = Linear([matrix], 2 * self.width, [self.width], suffix="")
        self.steps: Optional[torch.Tensor] = None

    def tensor_specs(self) -> List[TensorSpec]:
        steps = [TensorSpec(self.steps_name, (self.times, self.width), "bias")] if self.steps_name else []
        return self.mix.tensor_specs() + steps

    def bind(self, get: Callable[[str], Optional[torch.Tensor]], rt: Runtime) -> None:
        super().bind(get, rt)
        self.mix.bind(get, rt)
        if self.steps_name is None:
            return
        self.steps = get(self.steps_name).to(device=rt.device, dtype=torch.float32).contiguous()

    def forward(self, ctx: StepContext, x: torch.Tensor, pending, x0: torch.Tensor, number: int):
        """(new stream, None): `pending` (a delta that the stream still lacks) is added on the way."""
        if not 0 <= number < self.times:
            raise ValueError(f"pass {number} of {self.times}")
        if isinstance(pending, (NormedAhead, K.RowSquares)):
            pending = None                         # the stream is complete already
        elif pending is not None and pending.dtype != torch.float32:
            pending = K.sum_parts(pending, None, torch.float32)
        both = K.concat_rows(x, x0, self.rt.dtype, delta=pending, write_back=False)
        out = K.sum_parts(self.mix.product(both, f32_ok=True), None if self.steps is None else self.steps[number], torch.float32)
        return out, None


@register_part("loop_add")
class LoopAdd(Part):
    """The same place filled by sums alone: x <- x + step[t], from the second pass on also + x0."""

    def __init__(self, steps: str, width: int, times: int):
        self.width, self.times, self.steps_name = int(width), int(times), steps
        self.steps: Optional[torch.Tensor] = None

    def tensor_specs(self) -> List[TensorSpec]:
        return [TensorSpec(self.steps_name, (self.times, self.width), "bias")]

    def bind(self, get: Callable[[str], Optional[torch.Tensor]], rt: Runtime) -> None:
        super().bind(get, rt)
        self.steps = get(self.steps_name).to(device=rt.device, dtype=torch.float32).contiguous()

    def forward(self, ctx: StepContext, x: torch.Tensor, pending, x0: torch.Tensor, number: int):
        if not 0 <= number < self.times:
            raise ValueError(f"pass {number} of {self.times}")
        if isinstance(pending, (NormedAhead, K.RowSquares)):
            pending = None                         # the stream is complete already
        K.stream_add(x, pending, again=x0 if number > 0 else None, vector=self.steps[number])
        return x, None
