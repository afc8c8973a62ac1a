"""What stands before a pass of looped layers: a product of the residual stream and the embedding's output."""

from __future__ import annotations

import torch

from pyre_amd.hip import ops
from pyre_amd.hip.ops import Partials
from pyre_amd.parts.base import Part, PassInputSpec, TensorSpec, take
from pyre_amd.parts.block import Hidden, without_bias
from pyre_amd.parts.linear import Linear


class PassInput(Part):
    """x <- W [x; x0]. W is kept as its two halves: the embedding's half of the product is the same for every pass, so it
    is made once a step, and a pass multiplies the stream alone. The two halves' results are the residual stream and its
    pending term afterwards, which the next norm's kernel adds as it adds any other."""

    def __init__(self, spec: PassInputSpec):
        self.spec = spec
        self.from_stream = Linear(spec.hidden_size, spec.hidden_size, "pass.stream")
        self.from_start = Linear(spec.hidden_size, spec.hidden_size, "pass.start")

    def tensor_specs(self) -> list[TensorSpec]:
        return [TensorSpec(self.spec.name, (self.spec.hidden_size, 2 * self.spec.hidden_size))]

    def bind(self, tensors, runtime) -> None:
        w = take(tensors, self.spec.name)
        self.from_stream.set(w[:, :self.spec.hidden_size])
        self.from_start.set(w[:, self.spec.hidden_size:])

    def linears(self) -> list:
        return [self.from_start, self.from_stream]

    def _rows(self, ctx, state: Hidden) -> torch.Tensor:
        """The stream, its pending term included, in the engine's element type."""
        h = ctx.workspace.get("block.h", (ctx.n_tokens, self.spec.hidden_size), ctx.dtype)
        ops.add_rms_terms(state.resid, without_bias(ctx, state.pending), None, 0.0, h)
        state.pending = None
        return h

    def start(self, ctx, state: Hidden) -> Partials:
        """The embedding's half of the product (the stream is the embedding's output here)."""
        return self.from_start.forward(ctx, self._rows(ctx, state), ctx.n_tokens)

    def enter(self, ctx, state: Hidden, start: Partials) -> None:
        pending = self.from_stream.forward(ctx, self._rows(ctx, state), ctx.n_tokens)
        ops.reduce_partials(start, state.resid, ctx.n_tokens)
        state.pending = pending
