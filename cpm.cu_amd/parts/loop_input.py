"""The start of a pass over a span of layers that run several times in a row.

Before pass t of the span the residual x is replaced by a product of itself and of the embedding's output x0, plus a
vector of the pass:   x <- W [x | x0] + step[t].

The product reads x and x0 in the activations' element type; its float result and the vector take the residual's place
in the norm that follows (ReplacingBranch).
"""
from __future__ import annotations

from typing import List, Mapping

import torch

from .. import ops
from .base import Part, ReplacingBranch, ResidualStream, Runtime, StepContext, WeightSpec
from .linear import Linear
from .norm import row_branch


class LoopInput(Part):
    def __init__(self, weight_name: str, step_name: str, hidden_size: int, times: int):
        if times < 1:
            raise ValueError(f"loop input: {times} passes")
        self.hidden_size, self.times, self.step_name = hidden_size, int(times), step_name
        self.proj = Linear([(weight_name, hidden_size)], 2 * hidden_size)

    def parts(self) -> List[Part]:
        return [self.proj]

    def weight_specs(self) -> List[WeightSpec]:
        return [WeightSpec(self.step_name, (self.times, self.hidden_size), "slight")]

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime):
        self.rt = rt
        self.step = tensors[self.step_name].to(torch.float32).contiguous()

    def _pair(self, n: int, ctx: StepContext) -> torch.Tensor:
        return ctx.ws.get("loop.pair", (n, 2 * self.hidden_size), self.rt.dtype)

    def start(self, x0: torch.Tensor, ctx: StepContext):
        """Keep the embedding's output of the step's tokens (x0 float32 [n, H])."""
        ops.add_rows(x0, out=self._pair(x0.shape[0], ctx)[:, self.hidden_size:])

    def forward(self, stream: ResidualStream, ctx: StepContext, t: int):
        """Pass t begins: the residual (with its pending branch) becomes the pass's input, left pending."""
        x = stream.x
        pair = self._pair(x.shape[0], ctx)
        with ctx.timed("loop_input"):
            pending, here = stream.take_pending(), pair[:, :self.hidden_size]
            ops.norm_rows(x, here, None, **row_branch(pending, stream.pending_scale))
            y = self.proj.forward_float(pair, ctx, "loop.in")
        stream.pending = ReplacingBranch(x, y, self.step[t])
        stream.pending_scale = 1.0
