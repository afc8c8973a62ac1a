"""A model assembled from a :class:`~pyre_amd.parts.base.ModelSpec`."""

from __future__ import annotations

import torch

from pyre_amd.parts.base import ModelSpec, Part, TensorBag, TensorSpec, make_part
from pyre_amd.parts.block import Hidden
from pyre_amd.parts.streams import StreamReader, summed_streams


class LayeredModel(Part):
    """embedding -> layers in the order of ``spec.schedule`` -> final norm -> head.

    The model owns no cache: the engine hands ``forward`` one cache view per entry
    of the order (or None where the entry keeps nothing).
    """

    def __init__(self, spec: ModelSpec):
        self.spec = spec
        self.embedding = make_part("embedding", spec.embedding)
        self.layers = [make_part("block", b) for b in spec.layers]
        self.final_norm = make_part("norm", spec.final_norm)
        self.final_reader = None  #: with a residual of several streams: reads their sum through the final norm
        for b in self.layers:
            if bool(getattr(b, "connections", None)) != bool(spec.streams) or \
                    any(c.streams != spec.streams for c in getattr(b, "connections", ())):
                raise ValueError(f"a layer's connections do not fit the model's {spec.streams} streams")
        self.head = make_part("head", spec.head)
        self.pass_input = make_part("pass_input", spec.pass_input) if spec.pass_input is not None else None
        self.schedule = list(spec.schedule)
        if any(call.enters for call in self.schedule) and (self.pass_input is None or spec.streams):
            raise ValueError("an entry of the order that enters a pass needs the model's pass_input and a residual of one row")
        for pos, call in enumerate(self.schedule):
            if not (0 <= call.layer < len(self.layers)):
                raise ValueError(f"order entry {pos} names layer {call.layer}, there are {len(self.layers)}")
            if call.cache_from is not None and not (0 <= call.cache_from < pos):
                raise ValueError(f"order entry {pos} reads the cache of entry {call.cache_from}, which does not precede it")

    def parts(self):
        passes = () if self.pass_input is None else (self.pass_input,)
        return (self.embedding, *passes, *self.layers, self.final_norm, self.head)

    def tensor_specs(self) -> list[TensorSpec]:
        seen: dict[str, TensorSpec] = {}
        for p in self.parts():
            for s in p.tensor_specs():
                if s.name in seen and seen[s.name].shape != s.shape:
                    raise ValueError(f"tensor {s.name} is asked for with two shapes")
                seen.setdefault(s.name, s)
        return list(seen.values())

    def linears(self) -> list:
        return [lin for p in self.parts() for lin in p.linears()]

    def step_arrays(self) -> list:
        """The arrays that the layers ask of every step, each name once."""
        seen = {}
        for layer in self.layers:
            for spec in layer.step_arrays():
                seen.setdefault(spec.name, spec)
        return list(seen.values())

    def cache_specs(self) -> list[list]:
        """What each entry of the order keeps: a list of cache descriptions, empty for an
        entry that keeps nothing or reads another entry's caches. An embedding that keeps state
        has an entry of its own behind the last layer's."""
        out: list[list] = []
        for pos, call in enumerate(self.schedule):
            own = list(self.layers[call.layer].cache_specs())
            if call.cache_from is None:
                out.append(own)
                continue
            theirs = out[call.cache_from]
            if [type(s) for s in own] != [type(s) for s in theirs]:
                raise ValueError(f"order entry {pos} reads the caches of entry {call.cache_from}, which keeps "
                                 f"{len(theirs)} of other kinds than the {len(own)} that this layer wants")
            out.append([])
        if hasattr(self.embedding, "cache_specs"):  # an embedding with state of its own: one more entry, behind the layers'
            out.append(list(self.embedding.cache_specs()))
        return out

    def tensor_uses(self) -> dict[str, int]:
        """How many parts name each tensor (a part inside a layer counts as its layer)."""
        uses: dict[str, int] = {}
        for p in self.parts():
            for s in p.tensor_specs():
                uses[s.name] = uses.get(s.name, 0) + 1
        return uses

    def bind(self, tensors, runtime) -> None:
        """Every part takes its tensors out of ``tensors``, which is left empty: a tensor that
        its part copies (a fused weight) is free as soon as the last part that named it has it."""
        bag = TensorBag(tensors, self.tensor_uses())
        tensors.clear()
        for p in self.parts():
            p.bind(bag, runtime)
        if self.spec.streams:
            self.final_reader = StreamReader(self.final_norm)

    def forward(self, ctx, caches: list, tap=None) -> torch.Tensor | None:
        """Run the step's tokens; returns float32 logits [n_logits, vocab] (None if none are wanted).
        ``caches[pos]`` is the list of cache views of entry ``pos`` of the order. ``tap(pos, rows)``,
        a debugging aid, is called after every entry with the hidden rows [n, hidden] (float32, the
        residual stream with the pending term added: a copy, made for the tap)."""
        n = ctx.n_tokens
        resid = ctx.workspace.get("resid", (n, self.spec.hidden_size), torch.float32)
        if hasattr(self.embedding, "cache_specs"):
            self.embedding.forward(ctx, resid, caches[len(self.schedule)])
        else:
            self.embedding.forward(ctx, resid)
        state = Hidden(resid, streams=self.spec.streams)
        start = self.pass_input.start(ctx, state) if self.pass_input is not None else None
        for pos, call in enumerate(self.schedule):
            if call.enters:
                self.pass_input.enter(ctx, state, start)
            self.layers[call.layer].forward(ctx, state, caches[pos])
            if tap is not None:
                tap(pos, self._hidden_rows(ctx, state))
        m = ctx.n_logits
        if m == 0:
            return None
        h = ctx.workspace.get("head.h", (m, self.spec.hidden_size), ctx.dtype)
        if self.final_reader is not None:
            self.final_reader.read(ctx, state, h, rows=ctx.logit_rows)
        else:
            self.final_norm.forward(ctx, state.resid, state.pending, h, rows=ctx.logit_rows)
        return self.head.forward(ctx, h, m)

    def _hidden_rows(self, ctx, state: Hidden) -> torch.Tensor:
        """The residual stream as it stands after a layer, the term that the next norm would add
        included (its partial sums in their order, then the bias)."""
        if state.streams:
            return summed_streams(state, ctx.n_tokens)
        rows = state.resid[:ctx.n_tokens].clone()

        def normed(term, post):
            if post is None:
                return term
            if post.kind == "rms":
                term = term / torch.sqrt((term * term).mean(-1, keepdim=True) + post.eps) * post.gain.float()
            else:
                dev = term - term.mean(-1, keepdim=True)
                term = dev / torch.sqrt((dev * dev).mean(-1, keepdim=True) + post.eps) * post.gain.float()
            return term if post.scale is None else term * post.scale.float()

        p = state.pending
        outer = p.outer if p is not None else None
        total = torch.zeros_like(rows)
        while p is not None:
            term = torch.zeros_like(rows)
            for i in range(p.count):
                term += p.data[i, :ctx.n_tokens].float()
            if p.bias is not None:
                term += p.bias.float()
            total += normed(term, p.post) * p.scale  # the term's own norm and scale, as the next norm's kernel applies them
            p = p.more
        return rows + normed(total, outer)
