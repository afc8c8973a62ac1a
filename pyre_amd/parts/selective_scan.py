"""A selective scan: a float32 state per channel and request whose decay, input and output every token chooses itself."""

from __future__ import annotations

import math

import torch

from pyre_amd.hip import ops
from pyre_amd.parts.base import SelectiveScanSpec, StateCacheSpec, TensorSpec, take
from pyre_amd.parts.branch import COLUMN_ALIGN, BranchMixer
from pyre_amd.parts.linear import Linear


class SelectiveScan(BranchMixer):
    """[x | z] = W_in h; x <- silu(conv over time(x) + b); [low | B | C] = W_x x; dt = softplus(W_dt low + b); per channel
    S <- exp(dt A) S + dt x B, y = S . C + D x with A = -exp(A_log); y silu(z); then the output matrix.

    Keeps two states per request: S float32 [inner, state] and the last ``taps - 1`` projected rows of x, which the
    convolution of the next step's first tokens reads.

    Step sizes are 32-bit numbers, so in the 16-bit mode the product that makes them takes ``low`` as two bfloat16 numbers
    (rounded, and what the rounding left) against W_dt twice; a step of single tokens makes them inside its scan's kernel."""

    role = "ssm"

    def __init__(self, spec: SelectiveScanSpec):
        if spec.inner <= 0 or spec.dt_rank <= 0 or not (0 < spec.state <= ops.SSM_MAX_STATE):
            raise ValueError(f"selective scan: inner and dt_rank must be positive, the state {spec.state} within 1..{ops.SSM_MAX_STATE}")
        if spec.dt_rank + 2 * spec.state > ops.SSM_MAX_SELECTED:
            raise ValueError(f"selective scan: a dt_rank of {spec.dt_rank} beside a state of {spec.state} is more than the kernel takes")
        if not (1 <= spec.conv_taps <= ops.CONV_MAX_TAPS):
            raise ValueError(f"selective scan: {spec.conv_taps} taps are outside 1..{ops.CONV_MAX_TAPS}")
        self.spec = spec
        self.hidden_size = spec.hidden_size
        self.inner = spec.inner
        self.padded_rank = -(-spec.dt_rank // COLUMN_ALIGN) * COLUMN_ALIGN
        self.taps = self.conv_b = self.dt_b = self.A2 = self.skip = None
        self.select = self.steps = None   # the products over x and over low

    def cache_specs(self) -> list:
        s = self.spec
        specs = [StateCacheSpec((s.inner, s.state), "float32")]
        if s.conv_taps > 1:
            specs.append(StateCacheSpec((s.conv_taps - 1, s.inner), "float32"))
        return specs

    def cache_spec(self):
        return self.cache_specs()[0]

    def in_tensors(self):
        return [TensorSpec(f"{self.spec.prefix}.in", (2 * self.spec.inner, self.spec.hidden_size))]

    def out_tensor(self):
        return TensorSpec(f"{self.spec.prefix}.o", (self.spec.hidden_size, self.spec.inner))

    def other_tensors(self):
        s, p = self.spec, self.spec.prefix
        # random weights: taps of the order of one, so that every tap matters; slow and fast channels
        return [TensorSpec(f"{p}.conv", (s.inner, s.conv_taps), init="normal:0.5"), TensorSpec(f"{p}.conv.b", (s.inner,)),
                TensorSpec(f"{p}.x", (s.dt_rank + 2 * s.state, s.inner)), TensorSpec(f"{p}.dt", (s.inner, s.dt_rank)),
                TensorSpec(f"{p}.dt.b", (s.inner,), init="normal:1.0"),
                TensorSpec(f"{p}.A_log", (s.inner, s.state), init="normal:1.0"), TensorSpec(f"{p}.D", (s.inner,), init="gain")]

    def bind_others(self, tensors, runtime) -> None:
        s, p = self.spec, self.spec.prefix
        self.taps = take(tensors, f"{p}.conv").float().t().contiguous()   # [taps, channels]
        self.conv_b = take(tensors, f"{p}.conv.b").float().contiguous()
        self.dt_b = take(tensors, f"{p}.dt.b").float().contiguous()
        self.skip = take(tensors, f"{p}.D").float().contiguous()
        # A log2(e): the kernels take powers of two
        self.A2 = (-torch.exp(take(tensors, f"{p}.A_log").double()) * math.log2(math.e)).float().contiguous()

        def padded(w, rows, cols):
            return torch.nn.functional.pad(w, (0, cols - w.shape[1], 0, rows - w.shape[0])) if tuple(w.shape) != (rows, cols) else w

        width = s.dt_rank + 2 * s.state
        width += -width % COLUMN_ALIGN
        self.select = Linear(s.inner, width, "ssm.x")
        self.select.set(padded(take(tensors, f"{p}.x"), width, s.inner))
        dt = padded(take(tensors, f"{p}.dt"), s.inner, self.padded_rank)
        if runtime.dtype != torch.float32:
            dt = torch.cat([dt, dt], dim=1)
        self.steps = Linear(dt.shape[1], s.inner, "ssm.dt")
        self.steps.set(dt)

    def inner_linears(self) -> list:
        return [self.select, self.steps]

    def attend(self, ctx, proj, col0, cache, o, scale) -> None:
        s, n, ws = self.spec, ctx.n_tokens, ctx.workspace
        state, conv = (cache[0], cache[1]) if isinstance(cache, (list, tuple)) else (cache, None)
        single = ctx.host.max_q_len == 1 and n == ctx.n_seqs
        x = ws.get("ssm.rows", (n, s.inner), ctx.dtype)
        ops.ssm_conv(proj, col0, self.taps, self.conv_b, conv.tensor if conv is not None else None, state.slots,
                     ctx.seq_of_token, ctx.q_start, ctx.n_seqs, x, n, single=single)
        sel = self.select.forward(ctx, x, n)
        shared = (proj, col0 + s.inner, self.A2, self.skip, state.tensor)
        if single:
            ops.ssm_step(self.steps.weight, self.dt_b, x, sel, s.dt_rank, *shared, state.slots, ctx.n_seqs, scale, o)
            return
        low = ws.get("ssm.low", (n, self.steps.in_features), ctx.dtype)
        ops.ssm_low(sel, s.dt_rank, low, n)
        z = self.steps.forward(ctx, low, n)
        ops.ssm_scan(z, self.dt_b, x, sel, s.dt_rank, *shared, ctx.q_start, state.slots, ctx.n_seqs, scale, o, n)
