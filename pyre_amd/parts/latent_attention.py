"""Softmax attention over one compressed row per token, from which every head's keys and values are made."""

from __future__ import annotations

import torch

from pyre_amd.hip import ops
from pyre_amd.parts.attention import STEP_ARRAYS
from pyre_amd.parts.base import LatentAttentionSpec, Mixer, PagedCacheSpec, PagedTensorSpec, TensorSpec, make_part, take
from pyre_amd.parts.linear import Linear


class LatentAttention(Mixer):
    """c = rms_norm(Wdkv h) gain; head i: k = Wuk_i c, v = Wuv_i c, out_i = softmax(q_i k^T scale) v; with a turned part
    r that all heads share, k = [Wuk_i c | r] and q_i = [unturned | turned].

    Only [c | r] is kept, and neither keys nor values are ever made: q_i . (Wuk_i c) = (Wuk_i^T q_i) . c, so a head's
    query is carried into the compressed row's space (a product per head), the attention kernels run with the kept
    rows as the one shared key head and their first part as the value head, and the weighted sum of rows is carried out
    again, Wuv_i (sum_j a_j c_j), the output's gate applied on the way. Queries (or the compressed row that they are
    made of), the kept row and the gate are one input product. A layer without a row of its own (``own_latent`` False)
    reads the pages that another layer of the same sizes wrote."""

    def __init__(self, spec: LatentAttentionSpec):
        row = spec.rank + spec.rot_dim
        if not (0 < spec.rank <= ops.LATENT_MAX_RANK) or row > ops.LATENT_MAX_ROW:
            raise ValueError(f"latent attention: a row of {spec.rank} + {spec.rot_dim} elements is outside 1..{ops.LATENT_MAX_RANK} "
                             f"(1..{ops.LATENT_MAX_ROW} with its turned part), the sizes that the attention kernels take")
        if min(spec.key_dim, spec.value_dim, spec.num_heads) <= 0 or min(spec.rot_dim, spec.q_rank, spec.window) < 0:
            raise ValueError("latent attention: bad head sizes")
        if spec.rot_dim:
            if spec.position is None or spec.position.kind != "rotary" or spec.position.pairing not in ("halves", "neighbours"):
                raise ValueError("latent attention: a turned part needs a rotary position encoding")
            if spec.position.head_dim != spec.rot_dim or spec.position.rotary_dim not in (None, spec.rot_dim):
                raise ValueError(f"latent attention: its turned part of {spec.rot_dim} elements is turned whole")
        self.spec = spec
        self.row = row
        self.position = make_part("position", spec.position) if spec.rot_dim else None
        self.q_dim = spec.num_heads * (spec.key_dim + spec.rot_dim)
        self.o_dim = spec.num_heads * spec.value_dim
        first = spec.q_rank or self.q_dim
        self.row_col = first
        self.gate_col = first + (row if spec.own_latent else 0)
        self.inp = Linear(spec.hidden_size, self.gate_col + (self.o_dim if spec.gated else 0), "lattn.in")
        self.q_up = Linear(spec.q_rank, self.q_dim, "lattn.q_up") if spec.q_rank else None
        self.out = Linear(self.o_dim, spec.hidden_size, "lattn.out")
        self.gain = self.q_gain = self.key_up = self.value_up = self.sink = None

    def cache_spec(self):
        return PagedCacheSpec((PagedTensorSpec("c", (1, self.row), token_axis=1),), self.spec.window)

    def step_arrays(self):
        return list(STEP_ARRAYS)

    def linears(self) -> list:
        return [lin for lin in (self.inp, self.q_up, self.out) if lin is not None]

    def tensor_specs(self) -> list[TensorSpec]:
        s, p = self.spec, self.spec.prefix
        if s.q_rank:
            specs = [TensorSpec(f"{p}.dq", (s.q_rank, s.hidden_size)), TensorSpec(f"{p}.dq.norm", (s.q_rank,), init="gain"),
                     TensorSpec(f"{p}.uq", (self.q_dim, s.q_rank))]
        else:
            specs = [TensorSpec(f"{p}.q", (self.q_dim, s.hidden_size))]
        if s.own_latent:
            specs += [TensorSpec(f"{p}.dkv", (self.row, s.hidden_size)), TensorSpec(f"{p}.dkv.norm", (s.rank,), init="gain")]
        if s.sink:
            specs.append(TensorSpec(f"{p}.sink", (s.num_heads,)))
        if s.gated:
            specs.append(TensorSpec(f"{p}.g", (self.o_dim, s.hidden_size)))
        # random weights: the way up from the compressed row drawn wider, so that keys have the scale of queries
        return specs + [TensorSpec(f"{p}.uk", (s.num_heads * s.key_dim, s.rank), init="normal:0.1"),
                        TensorSpec(f"{p}.uv", (self.o_dim, s.rank), init="normal:0.1"),
                        TensorSpec(f"{p}.o", (s.hidden_size, self.o_dim))]

    def bind(self, tensors, runtime) -> None:
        s, p = self.spec, self.spec.prefix
        parts = [take(tensors, f"{p}.dq" if s.q_rank else f"{p}.q")]
        if s.own_latent:
            parts.append(take(tensors, f"{p}.dkv"))
            self.gain = take(tensors, f"{p}.dkv.norm").float().contiguous()
        if s.gated:
            parts.append(take(tensors, f"{p}.g"))
        w = torch.cat(parts, dim=0) if len(parts) > 1 else parts[0]
        del parts
        self.inp.set(w)
        if s.q_rank:
            self.q_gain = take(tensors, f"{p}.dq.norm").float().contiguous()
            self.q_up.set(take(tensors, f"{p}.uq"))
        if s.sink:
            self.sink = take(tensors, f"{p}.sink").float().contiguous()
        self.out.set(take(tensors, f"{p}.o"))
        # per head [outputs, inputs] both ways: [rank, key_dim] carries a query in, [value_dim, rank] a sum out
        self.key_up = take(tensors, f"{p}.uk").view(s.num_heads, s.key_dim, s.rank).transpose(1, 2).contiguous()
        self.value_up = take(tensors, f"{p}.uv").view(s.num_heads, s.value_dim, s.rank).contiguous()

    def forward(self, ctx, h, cache):
        s, n, ws = self.spec, ctx.n_tokens, ctx.workspace
        heads, rows = s.num_heads, cache["c"]
        q = ws.get("lattn.q", (n, heads, s.key_dim), ctx.dtype)
        wide = ws.get("lattn.q_in", (n, heads, self.row), ctx.dtype)
        turn = {}
        if s.rot_dim:
            cos, sin, _ = self.position.rotary(ctx.runtime)
            turn = dict(cos=cos, sin=sin, neighbours=s.position.pairing == "neighbours", positions=ctx.positions)
        proj = self.inp.forward(ctx, h, n)
        row = (self.row_col, self.gain, rows, cache.slots) if cache.writes and s.own_latent else None
        gate = ws.get("lattn.gate", (n, self.o_dim), torch.float32) if s.gated else None
        latent = dict(row=row, gate=(self.gate_col, self.o_dim, gate) if s.gated else None, eps=s.norm_eps, **turn)
        if s.q_rank:
            cq = ws.get("lattn.cq", (n, s.q_rank), ctx.dtype)
            ops.latent_rows(proj, n, s.rank, s.rot_dim, ctx.dtype, normed_queries=(0, s.q_rank, self.q_gain, cq), **latent)
            ops.latent_rows(self.q_up.forward(ctx, cq, n), n, s.rank, s.rot_dim, ctx.dtype,
                            queries=(0, heads, s.key_dim, q, wide), **turn)
        else:
            ops.latent_rows(proj, n, s.rank, s.rot_dim, ctx.dtype, queries=(0, heads, s.key_dim, q, wide), **latent)
        ops.head_matmul(q, self.key_up, wide, n)
        o_in = ws.get("lattn.o_in", (n, heads, s.rank), ctx.dtype)
        self._attend(ctx, wide, rows, o_in, cache)
        o = ws.get("lattn.o", (n, heads, s.value_dim), ctx.dtype)
        ops.head_matmul(o_in, self.value_up, o, n, gate)
        return self.out.forward(ctx, o.view(n, self.o_dim), n)

    def _attend(self, ctx, q, rows, out, cache) -> None:
        s = self.spec
        step = (ctx.positions, ctx.seq_of_token, cache.table, s.num_heads, s.rank, self.row, cache.page_size, s.scale, s.window,
                self.sink)
        tiles = ctx.host.arrays["attention.prefill_tiles"]
        singles = ctx.host.arrays["attention.decode_tokens"]
        if len(tiles):
            ops.latent_attn_tile(q, rows, out, ctx.arrays["attention.prefill_tiles"], len(tiles), *step)
        if len(singles):
            spans = ops.latent_attn_spans(cache.table.shape[1], cache.page_size, s.window)
            scratch = None
            if spans > 1:
                scratch = ctx.workspace.get("lattn.spans", (len(singles) * s.num_heads * spans * (s.rank + 2),), torch.float32)
            ops.latent_attn_single(q, rows, out, ctx.arrays["attention.decode_tokens"], len(singles), *step, scratch=scratch)
