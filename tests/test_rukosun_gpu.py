"""The Rukosun design through the engine against the plain implementation (``plain_rukosun``): whole prompts layer by
layer, prefill against token-by-token decoding, portions down to two tokens, mixed batches with pages and slots used
again, long decoding past every window, keys made to stand out at the edges of a window and at page borders, a sink that
decides the output, the first tokens of a sequence, each mechanism alone, the kernels alone, greedy generation through the
scheduler, and the programs as processes."""

from __future__ import annotations

import copy
import json

import numpy as np
import pytest
import torch

import plain_rukosun as P
import rukosun_models as M
from helpers import cut, first_bad, random_ids, replay

pytestmark = pytest.mark.gpu
DEV = "cuda:0"

#: bounds on max |difference| / max |logit| of a position: float32 and bfloat16 against the float64 plain run
TOL = {"float32": 2e-5, "bfloat16": 5e-2}
MODELS = {"small": (M.SMALL, 11), "ones": (M.ONES, 12), "wide": (M.WIDE, 13), "odd": (M.ODD, 14), "long": (M.LONG, 15)}


def write_model(folder, raw, seed, change=None):
    """A model folder with random weights; ``change(state)`` may alter them."""
    from safetensors.torch import save_file

    from pyre_amd.registry import config_from_dict
    from pyre_amd.weights import model_tensor_specs, random_state

    cfg = config_from_dict(raw)
    cfg.save(folder)
    state = random_state(model_tensor_specs(cfg), seed, 0.2, 0.2)
    if change is not None:
        change(state)
    save_file({k: v.contiguous() for k, v in state.items()}, str(folder) + "/model.safetensors")
    return (folder, *P.read_folder(folder))


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: write_model(tmp_path_factory.mktemp("rukosun_" + name), raw, seed) for name, (raw, seed) in MODELS.items()}


_rows: dict = {}


def plain_rows(cfg, w, ids):
    """Plain logits, kept: several tests ask for the same."""
    key = (id(w), tuple(ids))
    if key not in _rows:
        _rows[key] = (w, P.forward(w, cfg, ids).float())
    return _rows[key][1]


def engine_of(folder, dtype, **kw):
    from pyre_amd.config.engine import EngineConfig
    from pyre_amd.engine.engine import Engine

    args = dict(dtype=dtype, page_size=8, max_cached_tokens=1024, max_num_seqs=4, max_num_batched_tokens=512,
                use_graphs=False)
    args.update(kw)
    return Engine.from_folder(folder, EngineConfig(**args))


def whole(reqs):
    return [([(r, ids, list(range(len(ids))))], [r]) for r, ids in reqs.items()]


def in_portions(reqs, sizes):
    steps = []
    for r, ids in reqs.items():
        pos, parts = 0, cut(len(ids), sizes)
        for k, n in enumerate(parts):
            steps.append(([(r, ids[pos:pos + n], list(range(n)))], [r] if k == len(parts) - 1 else []))
            pos += n
    return steps


def one_by_one(reqs, first):
    steps = []
    for r, ids in reqs.items():
        steps.append(([(r, ids[:first], list(range(first)))], []))
        steps += [([(r, [ids[t]], [0])], [r] if t == len(ids) - 1 else []) for t in range(first, len(ids))]
    return steps


def assert_close(got, want, tol):
    bad, worst = first_bad(got, want, tol)
    assert bad is None, bad
    return worst


def all_given_back(eng):
    eng.cache.check_invariants()
    return all(g.allocator.num_used == 0 for g in eng.cache.page_groups) and eng.cache.slots.num_used == 0


# ----------------------------------------------------------------------------- whole prompts, layer by layer


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["small", "ones", "wide", "odd", "long"])
def test_every_layer_of_a_whole_prompt(name, dtype, folders):
    from pyre_amd.engine.batch import Entry

    folder, cfg, w = folders[name]
    ids = random_ids(cfg["vocab"], 75, seed=3)
    want, layers = P.forward(w, cfg, ids, return_hidden=True)
    eng = engine_of(folder, dtype)
    seen = {}
    got = eng.step([Entry("a", ids, list(range(len(ids))))], tap=lambda pos, rows: seen.__setitem__(pos, rows.double().cpu()))
    assert len(layers) == len(P.layer_order(cfg)) == len(seen)
    for pos, ref in enumerate(layers):
        d = float((seen[pos] - ref).abs().max() / ref.abs().max())
        assert d <= TOL[dtype], f"layer run {pos}: {d:.2e}"
    d = float((got.double().cpu() - want).abs().max() / want.abs().max())
    assert d <= TOL[dtype], d


@pytest.mark.parametrize("name,dtype,page", [("small", "float32", 8), ("small", "bfloat16", 16), ("ones", "float32", 4),
                                             ("wide", "float32", 16), ("wide", "bfloat16", 8), ("odd", "float32", 8),
                                             ("odd", "bfloat16", 16), ("long", "float32", 32)])
def test_prefill_decode_and_portions_agree_with_plain(name, dtype, page, folders):
    folder, cfg, w = folders[name]
    reqs = {r: random_ids(cfg["vocab"], n, seed=n) for r, n in (("a", 90), ("b", 1), ("c", 37))}
    want = {r: plain_rows(cfg, w, ids) for r, ids in reqs.items()}
    eng = engine_of(folder, dtype, page_size=page)
    assert_close(replay(eng, whole(reqs)), want, TOL[dtype])
    # most of the prompt, then token by token: the windows pass over decoded tokens
    tail = {r: ids for r, ids in reqs.items() if len(ids) > 1}
    assert_close(replay(eng, one_by_one(tail, 6)), want, TOL[dtype])
    # the first tokens of a sequence one by one from the very start: no previous token, then one
    assert_close(replay(eng, one_by_one({"c": reqs["c"][:12]}, 1)), want, TOL[dtype])
    for sizes in ([2], [3, 2, 17, 2, 31, 5], [64, 2, 9], [7, 1, 1, 24]):
        assert_close(replay(eng, in_portions(tail, sizes)), want, TOL[dtype])
    assert all_given_back(eng)


@pytest.mark.parametrize("name,dtype,poison", [("small", "float32", True), ("wide", "float32", True), ("small", "bfloat16", True),
                                               ("wide", "bfloat16", True), ("ones", "float32", True), ("odd", "float32", True),
                                               ("odd", "bfloat16", True)])
def test_mixed_batches_with_pages_and_slots_used_again(name, dtype, poison, folders):
    folder, cfg, w = folders[name]
    reqs = {r: random_ids(cfg["vocab"], n, seed=7 * n) for r, n in (("a", 61), ("b", 9), ("c", 100), ("d", 33), ("e", 2), ("f", 47))}
    want = {r: plain_rows(cfg, w, ids) for r, ids in reqs.items()}
    # three slots, a pool that holds three of the requests at most: everything is used again
    eng = engine_of(folder, dtype, max_num_seqs=3, max_cached_tokens=232, debug_poison=poison)
    fed = {r: 0 for r in reqs}
    live, waiting, steps, k = [], list(reqs), [], 0
    while live or waiting:
        while waiting and len(live) < 3:
            live.append(waiting.pop(0))
        entries, end = [], []
        for r in live:
            n = min([5, 1, 13, 2, 1, 40, 1][k % 7], len(reqs[r]) - fed[r])
            k += 1
            entries.append((r, reqs[r][fed[r]:fed[r] + n], list(range(n))))
            fed[r] += n
            if fed[r] == len(reqs[r]):
                end.append(r)
        steps.append((entries, end))
        live = [r for r in live if r not in end]
    got = replay(eng, steps)
    assert_close(got, want, TOL[dtype])
    assert all_given_back(eng)
    # every request alone gives the same rows, beyond rounding: batch-mates, pages and slots do not matter
    alone = engine_of(folder, dtype)
    for r in ("a", "d"):
        single = replay(alone, whole({r: reqs[r]}))
        for pos in range(len(reqs[r])):
            d = float((single[(r, pos)] - got[(r, pos)]).abs().max() / want[r][pos].abs().max())
            assert d <= (TOL[dtype] if dtype == "float32" else 2 * TOL[dtype]), (r, pos, d)


def test_a_request_left_out_of_steps_goes_on_where_it_was(folders):
    """The previous token and the rows of a request that pauses are still its own when it comes back."""
    folder, cfg, w = folders["small"]
    reqs = {r: random_ids(cfg["vocab"], 30, seed=s) for r, s in (("a", 1), ("b", 2))}
    want = {r: plain_rows(cfg, w, ids) for r, ids in reqs.items()}
    eng = engine_of(folder, "float32")
    steps = [([("a", reqs["a"][:7], [6])], []), ([("b", reqs["b"][:11], [10])], []), ([("b", reqs["b"][11:12], [0])], []),
             ([("a", reqs["a"][7:9], [0, 1]), ("b", reqs["b"][12:13], [0])], []), ([("b", reqs["b"][13:], [0, 16])], ["b"]),
             ([("a", reqs["a"][9:10], [0])], []), ([("a", reqs["a"][10:], [0, 19])], ["a"])]
    assert_close(replay(eng, steps), want, TOL["float32"])


def test_long_decoding_in_a_pool_that_only_windows_make_fit(tmp_path):
    """260 tokens one by one through a model whose layers all have windows: the pages go back as the windows pass."""
    raw = copy.deepcopy(M.SMALL)
    raw["layers"][3]["mixer"]["mask"] = {"size": 14}
    folder, cfg, w = write_model(tmp_path, raw, 21)
    ids = random_ids(cfg["vocab"], 260, seed=1)
    want = {"a": plain_rows(cfg, w, ids)}
    eng = engine_of(folder, "float32", page_size=8, max_cached_tokens=160, debug_poison=True)
    assert_close(replay(eng, one_by_one({"a": ids}, 2)), want, TOL["float32"])
    assert all_given_back(eng)


def test_long_contexts_past_several_spans_of_keys(folders):
    """420 tokens: windows of 270 and 300 keys and none at all, in a whole prompt, in portions, and decoded."""
    folder, cfg, w = folders["long"]
    ids = random_ids(cfg["vocab"], 420, seed=6)
    want = {"a": plain_rows(cfg, w, ids)}
    eng = engine_of(folder, "float32", page_size=16)
    assert_close(replay(eng, whole({"a": ids})), want, TOL["float32"])
    assert_close(replay(eng, in_portions({"a": ids}, [100, 2, 61, 200])), want, TOL["float32"])
    assert_close(replay(eng, one_by_one({"a": ids}, 230)), want, TOL["float32"])
    eng16 = engine_of(folder, "bfloat16", page_size=16)
    assert_close(replay(eng16, whole({"a": ids})), want, TOL["bfloat16"])
    assert_close(replay(eng16, one_by_one({"a": ids}, 300)), want, TOL["bfloat16"])


def test_a_request_longer_than_the_table_of_positions_is_refused(tmp_path):
    from pyre_amd.engine.batch import Entry

    raw = copy.deepcopy(M.ODD)
    raw["max_positions"] = 21
    folder, cfg, w = write_model(tmp_path, raw, 22)
    eng = engine_of(folder, "float32", max_model_len=100)
    assert eng.max_model_len == 21
    ids = random_ids(cfg["vocab"], 22, seed=2)
    got = replay(eng, [([("a", ids[:21], list(range(21)))], [])])
    assert_close(got, {"a": plain_rows(cfg, w, ids[:21])}, TOL["float32"])
    with pytest.raises(Exception):
        eng.step([Entry("a", [ids[21]], [0])])
    eng.finish("a")
    with pytest.raises(Exception):
        eng.step([Entry("b", ids, [0])])
    assert all_given_back(eng)


# ----------------------------------------------------------------------------- keys made to stand out


def _edge_model(first_kind: bool, window: int, scale: float, vocab: int, places: int):
    return M.model(vocab, 32, [M.layer(M.mixer(2, 16, 4, 8, 32, scale, window=window, q_rank=16 if first_kind else 0), 12)],
                   streams=2, places=places)


def _edge_weights(first_kind: bool):
    """Queries and keys read the first half of a normed row, values the second. Tokens 51 and 52 share the first half of
    their rows, and 51's second half has 52's elements in another order (the norm then treats both alike): 51's key
    points where 52's query points, and its value is another. A query of token 52 gives its weight to itself and to an
    earlier 51 if it sees it, so whether it is seen decides the output. Pairs, positions and the turned part are zeros,
    so that a token's row is the same wherever it stands."""

    def change(state):
        width, rank = 32, 32
        state["bigram"].zero_(), state["pos"].zero_()
        state["l0.norm1"].fill_(1.0), state["l0.norm1.b"].zero_()
        g = torch.Generator().manual_seed(4)
        key = torch.linalg.qr(torch.randn(16, 16, generator=g))[0]
        both = torch.zeros(rank + 4, width)
        both[:16, :16] = key                              # the row's first half: the token's key
        both[16:32, 16:] = 0.2 * torch.linalg.qr(torch.randn(16, 16, generator=g))[0]   # its second half: what values are made of
        dt = state["l0.mix.dkv"].dtype
        state["l0.mix.dkv"] = both.to(dt)
        state["l0.mix.dkv.norm"].fill_(1.0)
        up = torch.zeros(2 * 16, rank)
        up[:16, :16] = up[16:, :16] = torch.eye(16)
        state["l0.mix.uk"] = up.to(dt)
        state["l0.mix.uv"][:, :16] = 0
        state["l0.mix.uv"] *= 10
        q = torch.zeros(2 * 20, 16)
        q[:16] = q[20:36] = torch.eye(16)                 # per head 16 unturned elements, then 4 turned ones of zero
        if first_kind:
            down = torch.zeros(16, width)
            down[:, :16] = key
            state["l0.mix.dq"], state["l0.mix.uq"] = down.to(dt), q.to(dt)
            state["l0.mix.dq.norm"].fill_(1.0)
            state["l0.mix.sink"].fill_(-3.0)
        else:
            state["l0.mix.q"] = torch.cat([q @ key, torch.zeros(40, 16)], 1).to(dt)
        state["embed"][51, :16] = state["embed"][52, :16]
        state["embed"][51, 16:] = state["embed"][52, 16:].flip(0)

    return change


def _edge_cases(window):
    # a query position and where its twin stands
    q = window + 28
    border = (q // 16) * 16
    return {"inside": (q, q - (window - 1)), "outside": (q, q - window), "page_border": (border + 7, border), "last_of_a_page": (border + 3, border - 1),
            "next_to_it": (q, q - 1), "chunk_border": (32 * (q // 32) + 5, 32 * (q // 32) - 1), "far": (q + 10, 2)}


@pytest.mark.parametrize("first_kind", [True, False])
@pytest.mark.parametrize("window", [12, 33, 290])
def test_a_key_just_inside_and_just_outside_the_window(first_kind, window, tmp_path):
    length = window + 45
    raw = _edge_model(first_kind, window, 1.2, 53 + length, length)
    folder, cfg, w = write_model(tmp_path, raw, 31, _edge_weights(first_kind))
    base = [t for t in range(1, 54 + length) if t not in (51, 52)][:length]     # no token twice, 51 and 52 nowhere
    reqs = {}
    for name, (i, j) in _edge_cases(window).items():
        ids = list(base)
        ids[i], ids[j] = 52, 51
        reqs[name] = ids
    want = {r: plain_rows(cfg, w, ids) for r, ids in reqs.items()}
    # the construction works: whether the twin is seen decides the logits at the query
    q = _edge_cases(window)["inside"][0]
    seen = float((want["inside"][q] - want["outside"][q]).abs().max() / want["inside"][q].abs().max())
    assert seen > 500 * TOL["float32"] and seen > 2 * TOL["bfloat16"], seen
    eng = engine_of(folder, "float32", page_size=16)
    for steps in (whole(reqs), one_by_one(reqs, q - 8), in_portions(reqs, [window + 27, 2, 5]), in_portions(reqs, [q, 2, 3])):
        assert_close(replay(eng, steps), want, TOL["float32"])
    eng16 = engine_of(folder, "bfloat16", page_size=16)
    for steps in (whole(reqs), one_by_one(reqs, q - 3)):
        assert_close(replay(eng16, steps), want, TOL["bfloat16"])


def test_a_sink_that_decides_the_output(tmp_path):
    """With small scores the sink is a large share of every denominator: leaving it out, counting it twice or scaling it
    would move the logits far beyond rounding."""
    raw = copy.deepcopy(M.SMALL)
    raw["layers"] = [raw["layers"][0], raw["layers"][2]]
    del raw["loop"]
    for layer in raw["layers"]:
        layer["mixer"]["scale"] = 0.02

    def change(state):
        for i in (0, 1):
            state[f"l{i}.mix.sink"] = torch.linspace(1.0, 3.0, state[f"l{i}.mix.sink"].numel()).to(state[f"l{i}.mix.sink"].dtype)

    folder, cfg, w = write_model(tmp_path, raw, 33, change)
    reqs = {"a": random_ids(cfg["vocab"], 50, seed=4), "b": random_ids(cfg["vocab"], 3, seed=5)}
    want = {r: plain_rows(cfg, w, ids) for r, ids in reqs.items()}
    without = {k: (v - 50.0 if k.endswith(".sink") else v) for k, v in w.items()}
    moved = float((plain_rows(cfg, without, reqs["a"]) - want["a"]).abs().max() / want["a"].abs().max())
    assert moved > 500 * TOL["float32"], moved
    eng = engine_of(folder, "float32", page_size=8)
    for steps in (whole(reqs), one_by_one(reqs, 2), in_portions(reqs, [2, 7])):
        assert_close(replay(eng, steps), want, TOL["float32"])
    assert_close(replay(engine_of(folder, "bfloat16"), whole(reqs)), want, TOL["bfloat16"])


def test_the_previous_token_decides_a_row(tmp_path):
    """A pair table far larger than the token table: a wrong previous token (at a portion's start, in a batch, in a slot
    that another request had) would change everything."""
    def change(state):
        state["embed"] *= 0.05
        state["pos"] *= 0.05
        state["bigram"] *= 5

    raw = copy.deepcopy(M.ODD)
    raw["embedding"]["bigram"] = {"buckets": 997, "mul_prev": 2147483629, "mul_cur": 99991}   # products beyond 32 bits
    folder, cfg, w = write_model(tmp_path, raw, 34, change)
    reqs = {r: random_ids(cfg["vocab"], n, seed=n) for r, n in (("a", 23), ("b", 5), ("c", 2))}
    want = {r: plain_rows(cfg, w, ids) for r, ids in reqs.items()}
    eng = engine_of(folder, "float32", max_num_seqs=2)
    steps = [([("a", reqs["a"][:4], [0, 3]), ("b", reqs["b"][:1], [0])], []), ([("b", reqs["b"][1:], [0, 3]), ("a", reqs["a"][4:5], [0])], ["b"]),
             ([("c", reqs["c"], [0, 1]), ("a", reqs["a"][5:], [0, 17])], ["a", "c"])]
    assert_close(replay(eng, steps), want, TOL["float32"])
    assert_close(replay(eng, one_by_one({"a": reqs["a"]}, 1)), want, TOL["float32"])


# ----------------------------------------------------------------------------- each mechanism alone, in another model


def test_the_parts_in_a_model_of_another_design(tmp_path):
    """The mechanisms are parts: latent attention with compressed queries but without a turned part, sink or gate, and
    with a turned part and a gate over plain queries, in plain pre-norm layers (one row a token) with a biased layer norm
    and with an RMS norm, the polynomial feed-forward, plain embedding, and no learned positions."""
    from dataclasses import dataclass
    from typing import ClassVar

    from pyre_amd.config.model import ModelConfig
    from pyre_amd.parts.base import (BlockSpec, EmbeddingSpec, LatentAttentionSpec, LayerCall, LayerNormSpec, LMHeadSpec,
                                     ModelSpec, PolyNormMLPSpec, RMSNormSpec, RotarySpec)
    from pyre_amd.registry import register_architecture, unregister_architecture
    from pyre_amd.weights import write_random_model

    width, vocab, eps = 44, 61, 1e-5
    rot = {"dims": 10, "base": 70.0}

    @dataclass(frozen=True)
    class ToyConfig(ModelConfig):
        architecture: ClassVar[str] = "ToyLatentParts"

        @classmethod
        def from_dict(cls, raw):
            return cls()

        def to_dict(self):
            return {"architectures": [self.architecture]}

    def build(cfg):
        a = LatentAttentionSpec(width, 3, 12, 7, 28, 0.4, eps, "a", q_rank=18, window=17)
        b = LatentAttentionSpec(width, 2, 9, 11, 33, 0.3, eps, "b", rot_dim=10,
                                position=RotarySpec(10, rot["base"], 0, exact=True, pairing="neighbours"), gated=True)
        layers = (BlockSpec(a, LayerNormSpec(width, eps, "a.n", bias=True), PolyNormMLPSpec(width, 30, "a.f", eps),
                            RMSNormSpec(width, eps, "", name="a.m")),
                  BlockSpec(b, RMSNormSpec(width, eps, "", name="b.n"), None, None))
        return ModelSpec(width, vocab, 0, EmbeddingSpec(vocab, width, name="embed"), layers, (LayerCall(0), LayerCall(1), LayerCall(0)),
                         LayerNormSpec(width, eps, "last", bias=True), LMHeadSpec(vocab, width, name="head"))

    def plain(w, ids):
        x = w["embed"][torch.as_tensor(ids)]
        T = len(ids)

        def a(x):
            h = P.layer_norm(w, "a.n", x, eps)
            q = ((P.unit_rms(h @ w["a.dq"].T, eps) * w["a.dq.norm"]) @ w["a.uq"].T).reshape(T, 3, 12)
            c = P.unit_rms(h @ w["a.dkv"].T, eps) * w["a.dkv.norm"]
            o = P.window_softmax(q, (c @ w["a.uk"].T).reshape(T, 3, 12), (c @ w["a.uv"].T).reshape(T, 3, 7), 0.4, 17)
            x = x + o @ w["a.o"].T
            return x + P.feed_forward(w, "a.f", P.unit_rms(x, eps) * w["a.m"], eps)

        def b(x):
            h = P.unit_rms(x, eps) * w["b.n"]
            q = (h @ w["b.q"].T).reshape(T, 2, 19)
            both = h @ w["b.dkv"].T
            c = P.unit_rms(both[:, :33], eps) * w["b.dkv.norm"]
            r = P.rotate(both[:, 33:].reshape(T, 1, 10), rot, True).expand(T, 2, 10)
            q = torch.cat([q[:, :, :9], P.rotate(q[:, :, 9:], rot, True)], 2)
            o = P.window_softmax(q, torch.cat([(c @ w["b.uk"].T).reshape(T, 2, 9), r], 2), (c @ w["b.uv"].T).reshape(T, 2, 11), 0.3, 0)
            return x + (o * torch.sigmoid(h @ w["b.g"].T)) @ w["b.o"].T

        return (P.layer_norm(w, "last", a(b(a(x))), eps) @ w["head"].T).float()

    register_architecture(ToyConfig.architecture, ToyConfig, build)
    try:
        write_random_model(tmp_path, ToyConfig(), seed=41, std=0.2, gain_std=0.2)
        _, w = P.read_folder(tmp_path)
        assert "a.sink" not in w and "a.g" not in w and "b.dq" not in w and w["a.dkv"].shape[0] == 28
        reqs = {r: random_ids(vocab, n, seed=n) for r, n in (("a", 70), ("b", 19))}
        want = {r: plain(w, ids) for r, ids in reqs.items()}
        for dtype in ("float32", "bfloat16"):
            eng = engine_of(tmp_path, dtype)
            for steps in (whole(reqs), in_portions(reqs, [5, 2, 30]), one_by_one(reqs, 4)):
                assert_close(replay(eng, steps), want, TOL[dtype])
    finally:
        unregister_architecture(ToyConfig.architecture)


# ----------------------------------------------------------------------------- the kernels alone


@pytest.mark.parametrize("heads,rank,rot,window,page,length", [
    (4, 64, 16, 0, 16, 700), (33, 40, 8, 300, 16, 650), (3, 130, 64, 5000, 8, 600), (2, 512, 64, 260, 16, 420), (5, 256, 128, 40, 16, 200),
    (70, 300, 20, 96, 32, 150), (1, 7, 2, 0, 4, 300), (2, 263, 6, 50, 16, 130), (6, 128, 128, 0, 16, 333), (2, 129, 2, 7, 16, 90)])
def test_attention_over_compressed_rows(heads, rank, rot, window, page, length):
    """Prompt tiles and single tokens over pages in no order, with and without a sink, against float64 on the same values:
    in 32 bits to float32 rounding; in 16 bits the scores, weights and sums are still float32, so what is left is the
    rounding of the output."""
    from pyre_amd.hip import ops

    g = torch.Generator().manual_seed(heads * rank + window)
    dk = rank + rot
    n_pages = -(-length // page)
    for dtype, tol in ((torch.float32, 4e-6), (torch.bfloat16, 6e-3)):
        q = torch.randn(length, heads, dk, generator=g).to(dtype)
        rows = torch.randn(length, dk, generator=g).to(dtype)
        sink = torch.randn(heads, generator=g) + 1.0
        order = torch.randperm(n_pages + 3, generator=g)[:n_pages]
        pool = torch.full((n_pages + 3, 1, page, dk), float("nan"), dtype=dtype)     # what no key was written to is never used
        for t in range(length):
            pool[order[t // page], 0, t % page] = rows[t]
        table = torch.full((1, n_pages + 2), -1, dtype=torch.int32)
        table[0, :n_pages] = order.int()
        scale = 1.5 / dk ** 0.5
        s = torch.einsum("ihd,jd->hij", q.double(), rows.double()) * scale
        i, j = torch.arange(length)[:, None], torch.arange(length)[None]
        seen = (j <= i) & ((i - j < window) if window else torch.ones(1, dtype=torch.bool))
        s = s.masked_fill(~seen, float("-inf"))
        pos = torch.arange(length, dtype=torch.int32, device=DEV)
        seq = torch.zeros(length, dtype=torch.int32, device=DEV)
        tiles = [(t, min(32, length - t)) for t in range(0, length, 32)]
        tiles[2:3] = [(64, 5), (69, 1), (70, 26)] if length > 96 else tiles[2:3]    # tiles that are not full, or start anywhere
        tiles_t = torch.tensor(tiles, dtype=torch.int32, device=DEV)
        singles = torch.tensor(sorted({0, 1, 31, 32, 63, 64, length // 2, length - 2, length - 1}), dtype=torch.int32, device=DEV)
        spans = ops.latent_attn_spans(table.shape[1], page, window)
        scratch = torch.full((len(singles) * heads * spans * (rank + 2),), float("nan"), device=DEV) if spans > 1 else None
        for with_sink in (False, True):
            if with_sink:
                full = torch.cat([s, sink.double()[:, None, None].expand(heads, length, 1)], 2)
                a = torch.softmax(full, 2)[:, :, :-1]
            else:
                a = torch.softmax(s, 2)
            want = torch.einsum("hij,jd->ihd", a, rows.double()[:, :rank])
            args = (pos, seq, table.to(DEV), heads, rank, dk, page, scale, window, sink.to(DEV) if with_sink else None)
            out = torch.zeros(length, heads, rank, device=DEV, dtype=dtype)
            ops.latent_attn_tile(q.to(DEV), pool.to(DEV), out, tiles_t, len(tiles), *args)
            bound = tol * float(want.abs().max())
            assert float((out.cpu().double() - want).abs().max()) < bound
            out2 = torch.zeros_like(out)
            ops.latent_attn_single(q.to(DEV), pool.to(DEV), out2, singles, len(singles), *args, scratch=scratch)
            got, pick = out2.cpu().double(), singles.cpu().long()
            assert float((got[pick] - want[pick]).abs().max()) < bound
            rest = torch.ones(length, dtype=torch.bool)
            rest[pick] = False
            assert bool((got[rest] == 0).all())      # tokens that are not listed are left alone


@pytest.mark.parametrize("neighbours", [False, True])
@pytest.mark.parametrize("heads,dim,rot,rank,q_rank,gate", [(3, 8, 16, 24, 20, 40), (2, 7, 6, 9, 5, 11), (5, 12, 8, 1500, 1100, 0),
                                                            (1, 4, 0, 16, 0, 8), (4, 16, 12, 32, 0, 0)])
def test_what_an_input_product_holds_for_a_compressed_row(heads, dim, rot, rank, q_rank, gate, neighbours):
    """Partial sums, the two norms, both pairings of the turned elements, the stores to rows and pages, the gate."""
    from pyre_amd.hip import ops
    from pyre_amd.parts.rotary import rotary_tables

    g = torch.Generator().manual_seed(rank)
    n, page, pages = 7, 4, 6
    q_cols = heads * (dim + rot)
    row_col, gate_col = q_cols, q_cols + rank + rot
    width = gate_col + gate + (-(gate_col + gate) % 4 if dim % 4 == 0 else 0)
    parts = torch.randn(3, n, width, generator=g)
    total = parts.double().sum(0)
    positions = torch.tensor([0, 1, 5, 200, 201, 33, 34], dtype=torch.int32)
    slots = torch.tensor([3, 4, 23, -1, 0, 1, 10], dtype=torch.int32)
    gain, q_gain = 1 + 0.3 * torch.randn(rank, generator=g), 1 + 0.3 * torch.randn(max(q_rank, 1), generator=g)
    cos, sin = rotary_tables(rot, 30.0, 210, exact=True) if rot else (None, None)

    def turn(x):   # [n, heads, rot]
        y = torch.empty_like(x)
        for p in range(rot // 2):
            a, b = (2 * p, 2 * p + 1) if neighbours else (p, p + rot // 2)
            ang = positions.double() * 30.0 ** (-2.0 * p / rot)
            c, s = torch.cos(ang)[:, None], torch.sin(ang)[:, None]
            y[:, :, a] = x[:, :, a] * c - x[:, :, b] * s
            y[:, :, b] = x[:, :, b] * c + x[:, :, a] * s
        return y

    heads_q = total[:, :q_cols].reshape(n, heads, dim + rot)
    both = total[:, row_col:row_col + rank + rot]
    want_row = torch.cat([P.unit_rms(both[:, :rank], 1e-3) * gain.double(), turn(both[:, None, rank:])[:, 0]], 1)
    turning = dict(cos=cos.to(DEV), sin=sin.to(DEV), neighbours=neighbours, positions=positions.to(DEV)) if rot else {}
    close = lambda got, want, tol: float((got.cpu().double() - want).abs().max()) < tol * float(want.abs().max())  # noqa: E731
    for dtype, tol in ((torch.float32, 2e-6), (torch.bfloat16, 1e-2)):
        q = torch.zeros(n, heads, dim, device=DEV, dtype=dtype)
        wide = torch.full((n, heads, rank + rot), 3.0, device=DEV, dtype=dtype)
        cache = torch.zeros(pages, 1, page, rank + rot, device=DEV, dtype=dtype)
        gate_t = torch.zeros(n, max(gate, 1), device=DEV)
        ops.latent_rows(ops.Partials(parts.to(DEV)), n, rank, rot, dtype, queries=(0, heads, dim, q, wide),
                        row=(row_col, gain.to(DEV), cache, slots.to(DEV)), gate=(gate_col, gate, gate_t) if gate else None,
                        eps=1e-3, **turning)
        assert close(q, heads_q[:, :, :dim], tol)
        assert bool((wide[:, :, :rank] == 3).all())
        if rot:
            assert close(wide[:, :, rank:], turn(heads_q[:, :, dim:]), tol)
        for t, slot in enumerate(slots.tolist()):
            if slot >= 0:
                assert close(cache[slot // page, 0, slot % page], want_row[t], tol)
        assert int((cache != 0).any(-1).sum()) == 6      # the token without a slot is stored nowhere
        if gate:
            assert close(gate_t, torch.sigmoid(total[:, gate_col:gate_col + gate]), 1e-6)
        if q_rank:
            cq = torch.zeros(n, q_rank, device=DEV, dtype=dtype)
            ops.latent_rows(ops.Partials(parts.to(DEV)), n, rank, rot, dtype, normed_queries=(4, q_rank, q_gain.to(DEV), cq), eps=1e-3, **turning)
            assert close(cq, P.unit_rms(total[:, 4:4 + q_rank], 1e-3) * q_gain.double(), tol)


@pytest.mark.parametrize("streams,hidden,n", [(1, 40, 5), (2, 3584, 3), (2, 3584, 140), (3, 50, 9), (4, 96, 6), (5, 1030, 4), (8, 260, 5),
                                              (2, 4200, 3), (6, 16, 1), (2, 5001, 2)])
@pytest.mark.parametrize("center", [True, False])
def test_the_kernel_between_two_sublayers(streams, hidden, n, center):
    from pyre_amd.hip import ops

    g = torch.Generator().manual_seed(streams * hidden)
    gain, shift = 1 + 0.2 * torch.randn(hidden, generator=g), 0.3 * torch.randn(hidden, generator=g)
    mix, out_w, in_w = torch.randn(streams, streams, generator=g), torch.randn(streams, generator=g), torch.randn(streams, generator=g)
    first = torch.randn(n, hidden, generator=g) + 0.5
    y = torch.randn(2, n, hidden, generator=g)
    eps = 1e-3

    def normed(u, with_shift):
        if center:
            u = u - u.mean(-1, keepdim=True)
        u = u / torch.sqrt((u * u).mean(-1, keepdim=True) + eps) * gain.double()
        return u + shift.double() if with_shift else u

    x = first.double()[:, None].expand(n, streams, hidden)
    after = torch.einsum("st,nsh->nth", mix.double(), x) + out_w.double()[None, :, None] * y.double().sum(0)[:, None]
    again = torch.einsum("st,nsh->nth", mix.double(), after) + out_w.double()[None, :, None] * y.double()[0][:, None]
    d = lambda t: t.to(DEV)  # noqa: E731
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        out = torch.zeros(n, hidden, device=DEV, dtype=dtype)
        close = lambda got, want, t=tol: float((got.cpu().double() - want).abs().max()) < t * float(want.abs().max())  # noqa: E731
        # behind the embedding: one row a token, nothing pending
        ops.stream_norm(d(first), None, streams, None, None, None, d(in_w), d(gain), d(shift), eps, out, center)
        assert close(out, normed(torch.einsum("s,nsh->nh", in_w.double(), x), True))
        # the first result goes back into streams that are still equal
        store = torch.full((n, streams * hidden), float("nan"), device=DEV)
        ops.stream_norm(d(first), store, streams, ops.Partials(d(y)), d(mix), d(out_w), d(in_w), d(gain), None, eps, out, center)
        assert close(store.view(n, streams, hidden), after, 1e-5)
        assert close(out, normed(torch.einsum("s,nsh->nh", in_w.double(), after), False))
        # a further one in place, in the engine's element type; then the plain sum of some rows, which stores nothing
        kept = store.clone()
        z = ops.Partials(d(y[:1].to(dtype)))
        ops.stream_norm(store, store, streams, z, d(mix), d(out_w), d(in_w), d(gain), d(shift), eps, out, center)
        assert close(store.view(n, streams, hidden), again, 1e-5 if dtype == torch.float32 else 2e-2)
        rows = torch.tensor([n - 1, 0], dtype=torch.int32, device=DEV)
        before = kept.clone()
        ops.stream_norm(kept, None, streams, ops.Partials(d(y[:1])), d(mix), d(out_w), None, d(gain), d(shift), eps, out[:2] if n > 1 else
                        torch.zeros(2, hidden, device=DEV, dtype=dtype), center, rows)
        assert torch.equal(kept, before)
        if n > 1:
            assert close(out[:2], normed(again.sum(1), True)[[n - 1, 0]])


@pytest.mark.parametrize("n,width", [(3, 1), (5, 37), (2, 320), (9, 4096), (4, 9000), (2, 18944), (3, 40000), (2, 4098)])
def test_the_polynomial_activation_kernel(n, width):
    from pyre_amd.hip import ops

    g = torch.Generator().manual_seed(width)
    z = torch.randn(2, n, width, generator=g) * 2
    z[:, 0] *= 1e-3                      # a row whose powers vanish beside eps
    abce = torch.tensor([0.7, -1.3, 0.4, 0.2])
    for parts, dtype, tol in ((z, torch.float32, 3e-6), (z, torch.bfloat16, 1e-2), (z[:1].bfloat16(), torch.bfloat16, 1e-2)):
        out = torch.zeros(n, width, device=DEV, dtype=dtype)
        ops.poly_norm(ops.Partials(parts.contiguous().to(DEV)), abce.to(DEV), 1e-6, out, n)
        want = P.poly_norm(parts.double().sum(0), abce.double(), 1e-6)
        d = (out.cpu().double() - want).abs().max(-1).values / want.abs().max(-1).values.clamp_min(1.0)  # (terms may cancel)
        assert float(d.max()) < tol, d


def test_a_layer_norm_with_a_bias_and_an_embedding_with_places():
    from pyre_amd.hip import ops

    g = torch.Generator().manual_seed(8)
    for n, hidden in ((5, 50), (3, 2048)):
        resid, y = torch.randn(n, hidden, generator=g), torch.randn(2, n, hidden, generator=g)
        gain, shift = 1 + 0.2 * torch.randn(hidden, generator=g), torch.randn(hidden, generator=g)
        r, out = resid.to(DEV), torch.zeros(n, hidden, device=DEV)
        ops.add_layernorm(r, ops.Partials(y.to(DEV)), gain.to(DEV), 1e-4, out, None, shift.to(DEV))
        x = resid.double() + y.double().sum(0)
        want = P.layer_norm({"n": gain.double(), "n.b": shift.double()}, "n", x, 1e-4)
        assert float((out.cpu().double() - want).abs().max()) < 1e-5 * float(want.abs().max())
        assert float((r.cpu().double() - x).abs().max()) < 1e-5
    cfg = {"embedding": {"bigram": {"buckets": 11, "mul_prev": 7, "mul_cur": 3}}}
    w = {"embed": torch.randn(20, 6, generator=g), "bigram": torch.randn(12, 6, generator=g), "pos": torch.randn(9, 6, generator=g)}
    ids, other = [3, 19, 3, 0], [4, 5, 6, 7, 8, 9, 10]
    state = torch.full((3, 1), float("nan"))
    state[2, 0] = 8.0                    # the second request goes on at position 5, its previous token was 8
    i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=DEV)  # noqa: E731
    out, st = torch.zeros(6, 6, device=DEV), state.to(DEV)
    ops.bigram_embed(w["embed"].to(DEV), w["bigram"].to(DEV), i32(*ids, 9, 10), i32(0, 1, 2, 3, 5, 6), i32(0, 0, 0, 0, 1, 1), i32(0, 4, 6), st,
                     i32(0, 2), out, 11, 7, 3, w["pos"].to(DEV))
    want = torch.cat([P.embed(cfg, {k: v.double() for k, v in w.items()}, ids), P.embed(cfg, {k: v.double() for k, v in w.items()}, other)[5:]])
    assert float((out.cpu().double() - want).abs().max()) < 1e-6 and st[0, 0] == 0 and st[2, 0] == 10


# ----------------------------------------------------------------------------- the entry points


def check_greedy(cfg, w, prompt, tokens, tol):
    """Every generated token against the plain logits given the tokens before it; it may differ where rounding decides."""
    rows = P.forward(w, cfg, list(prompt) + list(tokens[:-1]))[len(prompt) - 1:]
    for k, (tok, row) in enumerate(zip(tokens, rows)):
        twin = int(row.argmax())
        if twin != tok:
            margin = float((row[twin] - row[tok]) / row.abs().max())
            assert margin < tol, f"token {k} is {tok}, plainly {twin} (margin {margin:.2e})"


@pytest.mark.parametrize("name,dtype,graphs", [("small", "float32", False), ("small", "float32", True), ("wide", "float32", True),
                                               ("small", "bfloat16", True), ("long", "float32", True)])
def test_greedy_generation_through_the_scheduler(name, dtype, graphs, folders):
    """The scheduler runs one step ahead, its tokens fed on the device: the pair's row is found there. With graphs the
    decode steps are captured and replayed."""
    from pyre_amd.api import generate, load_model

    folder, cfg, w = folders[name]
    prompts = [random_ids(cfg["vocab"], n, seed=n + 1) for n in (1, 9, 40, 23)]
    eng, _ = load_model(str(folder), device=DEV, dtype=dtype, page_size=8, max_cached_tokens=1024, max_num_seqs=4,
                        max_num_batched_tokens=64, prefill_chunk=16, use_graphs=graphs)
    got = generate(eng, prompts, max_new_tokens=40)
    for p, g in zip(prompts, got):
        assert len(g) == 40
        check_greedy(cfg, w, p, g, TOL[dtype])
    assert all_given_back(eng)
    if graphs:
        assert eng.graph_replays > 0


def test_replayed_steps_are_the_eager_ones_bit_for_bit(folders):
    from pyre_amd.engine.batch import Entry

    folder, cfg, w = folders["wide"]
    engines = [engine_of(folder, "bfloat16", use_graphs=g) for g in (False, True)]
    prompts = {r: random_ids(cfg["vocab"], n, seed=n) for r, n in (("a", 17), ("b", 40), ("c", 5))}
    for eng in engines:
        eng.step([Entry(r, ids, []) for r, ids in prompts.items()])
    for t in range(12):
        toks = random_ids(cfg["vocab"], 3, seed=100 + t)
        rows = [eng.step([Entry(r, [tok], [0]) for r, tok in zip(prompts, toks)]).clone() for eng in engines]
        assert torch.equal(rows[0], rows[1]), t
    assert engines[1].graph_replays > 5


def test_the_generate_program_as_a_process(folders, tmp_path):
    import subprocess
    import sys
    from pathlib import Path

    folder, cfg, w = folders["odd"]
    root = Path(__file__).resolve().parent.parent
    out = tmp_path / "res.json"
    proc = subprocess.run([sys.executable, str(root / "bin" / "pyre_generate"), "--model", str(folder), "--dtype", "float32",
                           "--prompt-ids", "7,3,3,41,9,50,5", "--prompt-ids", "11", "--tokens", "12", "--num-blocks", "32",
                           "--max-batch", "2", "--out", str(out)], capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    res = json.loads(out.read_text())
    assert res["dtype"] == "float32" and [len(g) for g in res["generated"]] == [12, 12]
    for prompt, tokens in zip(res["prompts"], res["generated"]):
        check_greedy(cfg, w, prompt, tokens, TOL["float32"])


@pytest.mark.parametrize("dtype,extra", [("float32", ("--page-size", "8", "--poison")), ("bfloat16", ("--graphs",))])
def test_trace_run_as_a_process(dtype, extra, folders, tmp_path):
    from test_trace_run_gpu import run_trace

    folder, cfg, w = folders["small"]
    vocab = cfg["vocab"]
    reqs = {"a": random_ids(vocab, 70, 1), "b": random_ids(vocab, 40, 2), "c": random_ids(vocab, 64, 3), "d": random_ids(vocab, 3, 4),
            "e": random_ids(vocab, 61, 5)}
    fed = {r: 0 for r in reqs}
    sizes = [13, 2, 30, 1, 7, 64, 3]
    live, waiting, steps, k, wanted = [], list(reqs), [], 0, {}
    while live or waiting:
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
        entries, end = [], []
        for r in live:
            n = min(sizes[k % len(sizes)], len(reqs[r]) - fed[r])
            k += 1
            want = [] if k % 5 == 0 else list(range(0, n, 2))
            entries.append({"id": r, "tokens": reqs[r][fed[r]:fed[r] + n], "want": want})
            wanted.setdefault(len(steps), []).extend((r, fed[r] + x) for x in want)
            fed[r] += n
            if fed[r] == len(reqs[r]):
                end.append(r)
        steps.append({"step": len(steps), "entries": entries, "end": end})
        live = [r for r in live if r not in end]
    out = tmp_path / "out"
    run_trace(folder, dtype, out, 4 * 128, steps, extra)
    ref = {r: plain_rows(cfg, w, ids) for r, ids in reqs.items()}
    checked = 0
    for st, rows in wanted.items():
        if not rows:
            assert not (out / f"{st}.f32").exists()
            continue
        got = torch.from_numpy(np.fromfile(out / f"{st}.f32", dtype="<f4").reshape(len(rows), vocab))
        for i, (r, pos) in enumerate(rows):
            d = float((got[i] - ref[r][pos]).abs().max() / ref[r][pos].abs().max())
            assert d <= TOL[dtype], f"step {st} request {r} position {pos}: {d:.3e}"
            checked += 1
    assert checked > 50
