"""A residual of several streams, and layers whose sublayers stand between them (hyper-connections)."""

from __future__ import annotations

from dataclasses import dataclass

import torch

from pyre_amd.hip import ops
from pyre_amd.parts.base import (Block, HyperConnectionBlockSpec, HyperConnectionSpec, LayerNormSpec, RMSNormSpec, TensorSpec,
                                 make_part, take)
from pyre_amd.parts.block import Hidden


@dataclass
class StreamWeights:
    """What a sublayer's connection holds, float32: ``into [S]``, ``out [S]``, ``mix [S, S]`` (from, to)."""

    into: torch.Tensor
    out: torch.Tensor
    mix: torch.Tensor


def connection_tensors(c: HyperConnectionSpec) -> list[TensorSpec]:
    return [TensorSpec(f"{c.prefix}.in", (c.streams,), init="gain"), TensorSpec(f"{c.prefix}.out", (c.streams,), init="gain"),
            TensorSpec(f"{c.prefix}.mix", (c.streams, c.streams), init="normal:0.5")]


class StreamReader:
    """What stands before a sublayer (or behind the last layer): the pending result goes back into the streams, one
    mixture of them is formed and normed, all in one kernel. ``norm``: a bound layer norm or RMS norm; its weights are
    taken in float32."""

    def __init__(self, norm, weights: StreamWeights | None = None):
        if not isinstance(norm.spec, (LayerNormSpec, RMSNormSpec)):
            raise ValueError(f"streams are read through a layer norm or an RMS norm, not {norm.spec.kind!r}")
        self.center = isinstance(norm.spec, LayerNormSpec)
        self.eps = norm.spec.eps
        self.gain = norm.gain.float().contiguous()
        shift = getattr(norm, "shift", None)
        self.shift = None if shift is None else shift.float().contiguous()
        self.into = None if weights is None else weights.into

    def read(self, ctx, state: Hidden, out: torch.Tensor, rows: torch.Tensor | None = None) -> None:
        """``out`` = the normed mixture; the streams take the pending result on the way (with ``rows`` only those rows
        are formed and nothing is stored)."""
        dst = mix = back = None
        if state.pending is not None:
            mix, back = state.weights.mix, state.weights.out
            if rows is None:
                dst = ctx.workspace.get("resid.streams", (ctx.n_tokens, state.streams * self.gain.numel()), torch.float32)
        ops.stream_norm(state.resid, dst, state.streams, state.pending, mix, back, self.into, self.gain, self.shift, self.eps,
                        out, self.center, rows)
        if dst is not None:
            state.resid, state.pending = dst, None


def summed_streams(state: Hidden, n: int) -> torch.Tensor:
    """The sum of the streams after the pending result, a copy (a debugging aid, plain torch)."""
    hidden = state.resid.shape[1] if state.pending is None else state.pending.width
    x = state.resid[:n].view(n, -1, hidden).expand(n, state.streams, hidden)
    if state.pending is None:
        return x.sum(1)
    y = state.pending.data[:, :n].float().sum(0)
    mixed = torch.zeros(n, hidden, device=x.device, dtype=torch.float32)
    for s in range(state.streams):
        mixed += float(state.weights.mix[s].sum()) * x[:, s]
    return mixed + float(state.weights.out.sum()) * y


class HyperConnectionBlock(Block):
    """A mixer and a feed-forward (or the mixer alone), each reading a mixture of the residual's streams through a norm
    and handing its result back to all of them. Nothing is added here: a result is the pending term, which the next
    reader's kernel mixes in as it reads the streams."""

    def __init__(self, spec: HyperConnectionBlockSpec):
        self.spec = spec
        self.mixer = make_part("mixer", spec.mixer)
        self.mixer_norm = make_part("norm", spec.mixer_norm)
        self.feed_forward = self.feed_forward_norm = None
        self.connections = [spec.mixer_connection]
        if spec.feed_forward is not None:
            self.feed_forward = make_part("feed_forward", spec.feed_forward)
            self.feed_forward_norm = make_part("norm", spec.feed_forward_norm)
            self.connections.append(spec.feed_forward_connection)
        for c in self.connections:
            if not 1 <= c.streams <= ops.MAX_STREAMS:
                raise ValueError(f"hyper-connections: {c.streams} streams are outside 1..{ops.MAX_STREAMS}")
        self.weights: list[StreamWeights] = []
        self.readers: list[StreamReader] = []

    def parts(self):
        return tuple(p for p in (self.mixer_norm, self.mixer, self.feed_forward_norm, self.feed_forward) if p is not None)

    def tensor_specs(self) -> list[TensorSpec]:
        return [s for p in self.parts() for s in p.tensor_specs()] + [s for c in self.connections for s in connection_tensors(c)] + \
               [TensorSpec(name, tuple(shape), optional=True) for name, shape in self.spec.unused]

    def bind(self, tensors, runtime) -> None:
        for p in self.parts():
            p.bind(tensors, runtime)
        for name, _ in self.spec.unused:
            if name in tensors:
                take(tensors, name)
        self.weights = [StreamWeights(*(take(tensors, f"{c.prefix}.{x}").float().contiguous() for x in ("in", "out", "mix")))
                        for c in self.connections]
        norms = [self.mixer_norm] + ([self.feed_forward_norm] if self.feed_forward is not None else [])
        self.readers = [StreamReader(norm, w) for norm, w in zip(norms, self.weights)]

    def linears(self) -> list:
        return [lin for p in self.parts() for lin in p.linears()]

    def cache_specs(self) -> list:
        if hasattr(self.mixer, "cache_specs"):
            return list(self.mixer.cache_specs())
        spec = self.mixer.cache_spec()
        return [] if spec is None else [spec]

    def step_arrays(self) -> list:
        return self.mixer.step_arrays()

    def forward(self, ctx, state: Hidden, caches: list) -> None:
        h = ctx.workspace.get("block.h", (ctx.n_tokens, self.readers[0].gain.numel()), ctx.dtype)
        self.readers[0].read(ctx, state, h)
        cache = caches if hasattr(self.mixer, "cache_specs") else (caches[0] if caches else None)
        state.pending, state.weights = self.mixer.forward(ctx, h, cache), self.weights[0]
        if self.feed_forward is None:
            return
        self.readers[1].read(ctx, state, h)
        state.pending, state.weights = self.feed_forward.forward(ctx, h), self.weights[1]
