"""Inputs of a layer that come from the tokens themselves, beside the residual.

A table holds ``dim`` numbers a token and layer (all layers' columns side by side).  After a layer's sub-layers,

    y = P ( gelu_tanh(G x) * e ),   e = the layer's columns of table[token],     x <- x + y / rms(y) * w

x the residual as the layer left it.  The gate product reads x in the activations' element type; the root mean square,
its weight and the sum are float.  The last step is left pending for the norm that follows (NormedBranch).
"""
from __future__ import annotations

from typing import List, Mapping, Optional

import torch

from .. import ops
from .base import NORMS, NormedBranch, Part, Runtime, StepContext, WeightSpec
from .linear import Linear


class TokenTable(Part):
    """The table [vocab, columns], shared by the layers that read it."""

    def __init__(self, name: str, vocab_size: int, columns: int):
        self.name, self.vocab_size, self.columns = name, vocab_size, columns
        self.table: Optional[torch.Tensor] = None

    def weight_specs(self) -> List[WeightSpec]:
        return [WeightSpec(self.name, (self.vocab_size, self.columns), "table")]

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime):
        self.table = tensors[self.name].to(rt.dtype).contiguous()


class TokenInput(Part):
    def __init__(self, table: TokenTable, offset: int, dim: int, hidden_size: int, gate_name: str, proj_name: str,
                 norm_name: str, eps: float, activation: str = "gelu_tanh"):
        if dim < 1 or offset < 0 or offset + dim > table.columns:
            raise ValueError(f"token input: columns {offset}..{offset + dim} of a table of {table.columns}")
        self.source, self.offset, self.dim, self.activation = table, int(offset), int(dim), activation
        self.gate = Linear([(gate_name, dim)], hidden_size)
        self.proj = Linear([(proj_name, hidden_size)], dim)
        self.norm = NORMS.build("rms_norm", name=norm_name, hidden_size=hidden_size, eps=eps)

    def parts(self) -> List[Part]:
        return [self.gate, self.proj, self.norm]            # the table belongs to the model

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime):
        self.rt = rt

    def forward(self, x: torch.Tensor, ctx: StepContext) -> NormedBranch:
        """x [n, H]: the residual in the engine's element type."""
        n = x.shape[0]
        with ctx.timed("token_input"):
            g = ctx.ws.get("side.act", (n, self.dim), self.rt.dtype)
            if n <= ops.LOOKUP_STRIP_ROWS and self.gate.tiled is not None and x.shape[1] % 8 == 0:
                ops.lookup_strip(x, self.gate.tiled, self.source.table, self.offset, ctx.token_ids, g, self.activation)
            else:
                z = self.gate.forward(x, ctx, "side.gate", out_dtype=torch.float32 if n <= ops.SKINNY_MAX_ROWS else None,
                                      partials=True)
                ops.gated_lookup(z, self.source.table, self.offset, ctx.token_ids, g, self.activation)
            y = self.proj.forward(g, ctx, "side.proj", out_dtype=torch.float32, partials=True)
        return NormedBranch(y, self.norm, ctx, "side.norm")
