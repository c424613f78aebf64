"""Short convolutions on what a layer's sub-layers read.

The normed rows h of a layer pass, for each sub-layer, a causal convolution over time of its own, one filter a channel,
added to the rows themselves:

    h_k[t] = h[t] + sum_j w_k[:, j] h[t - taps + 1 + j]            zeros before the sequence's start, no bias

All sub-layers of a parallel layer convolve the same rows, so one copy of the last taps - 1 rows is kept a sequence and
layer run, as float fixed-size state of the cache entry.  The normed rows stay float until the convolutions have run.
"""
from __future__ import annotations

from typing import List, Mapping, Sequence, Tuple

import torch

from .. import ops
from ..cache.paged import CacheView, StateSpec
from .base import Norm, Part, ResidualStream, Runtime, StepContext, WeightSpec, branch_for


class InputConvolution(Part):
    STATE = "input_conv"

    def __init__(self, names: Sequence[str], hidden_size: int, taps: int):
        """``names``: a checkpoint tensor [hidden_size, taps] for each sub-layer (one or two)."""
        if taps < 1:
            raise ValueError(f"input convolution: {taps} taps")
        if not 1 <= len(names) <= 2:
            raise ValueError(f"input convolution: {len(names)} sub-layers (one or two)")
        self.names, self.hidden_size, self.taps = list(names), hidden_size, int(taps)

    def weight_specs(self) -> List[WeightSpec]:
        return [WeightSpec(n, (self.hidden_size, self.taps), "conv_taps") for n in self.names]

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime):
        self.rt = rt
        self.weights = [tensors[n].to(torch.float32).t().contiguous() for n in self.names]      # [taps, hidden]

    def state(self) -> Tuple[Tuple[str, StateSpec], ...]:
        if self.taps == 1:
            return ()
        return ((self.STATE, StateSpec((self.taps - 1, self.hidden_size), torch.float32)),)

    def forward(self, norm: Norm, stream: ResidualStream, ctx: StepContext, cache: CacheView) -> List[torch.Tensor]:
        """The pending branch added, the rows normed and convolved: one tensor [n, H] a sub-layer."""
        x, pending = stream.x, branch_for(norm, stream.take_pending())
        state = cache.state.get(self.STATE) if cache is not None else None
        tags = [f"block.h{k + 1}" for k in range(len(self.weights))]
        if ctx.single_token:
            outs = norm.forward_convolved(x, pending, stream.pending_scale, ctx, self.weights, state, tags)
            if outs is not None:
                return outs
        kw = {"out_dtype": torch.float32} if norm.takes_out_dtype else {}
        h = norm.forward(x, pending, stream.pending_scale, ctx, tag="block.h", **kw)
        outs = [ctx.ws.get(tag, tuple(h.shape), self.rt.dtype) for tag in tags]
        ops.conv_rows(h, self.weights, state, outs, ctx.cu_q, ctx.seq_slot, max(ctx.q_lens))
        return outs
