"""The Pinozen design through the engine against the plain implementation (``plain_pinozen``): whole prompts layer by
layer, prefill against token-by-token decoding, portions down to two tokens, mixed batches with pages and slots used
again, keys made to stand out far away, at page borders and one past the query, a sink that decides the output, scores that
the cap bends, taps that decide a row, states that last, the first tokens of a sequence, each mechanism alone in other
designs, the kernels alone, greedy generation through the scheduler, and the programs as processes."""

from __future__ import annotations

import copy
import json
import math

import numpy as np
import pytest
import torch

import pinozen_models as M
import plain_pinozen as P
from helpers import cut, first_bad, random_ids, replay

pytestmark = pytest.mark.gpu
DEV = "cuda:0"

#: bounds on max |difference| / max |logit| of a position: float32 and bfloat16 against the float64 plain run. Rounding to
#: bfloat16 what the engine stores in it, done to the plain run alone, moves the worst row of these models by up to 0.07
#: and the median row by about 0.01; so the 16-bit mode is held to a bound on every row and to one on the median.
TOL = {"float32": 2e-5, "bfloat16": 0.12}
MEDIAN = {TOL["float32"]: 2e-5, TOL["bfloat16"]: 0.02}
SEEDS = {"small": 11, "ones": 12, "wide": 13, "odd": 14, "long": 15}


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
    return {name: write_model(tmp_path_factory.mktemp("pinozen_" + name), raw, SEEDS[name]) for name, raw in M.ALL.items()}


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
    rows = sorted(float((got[k] - want[k[0]][k[1]]).abs().max() / want[k[0]][k[1]].abs().max()) for k in got)
    assert rows[len(rows) // 2] <= MEDIAN[tol], rows[len(rows) // 2]
    return worst


def all_given_back(eng):
    eng.cache.check_invariants()
    return all(g.allocator.num_used == 0 for g in eng.cache.page_groups) and eng.cache.slots.num_used == 0


# ----------------------------------------------------------------------------- whole prompts, layer by layer


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(M.ALL))
def test_every_layer_of_a_whole_prompt(name, dtype, folders):
    from pyre_amd.engine.batch import Entry

    folder, cfg, w = folders[name]
    ids = random_ids(cfg["vocab"], 75, seed=3)
    want, layers = P.forward(w, cfg, ids, return_hidden=True)
    eng = engine_of(folder, dtype)
    seen = {}
    got = eng.step([Entry("a", ids, list(range(len(ids))))], tap=lambda pos, rows: seen.__setitem__(pos, rows.double().cpu()))
    assert len(layers) == len(P.layer_runs(cfg)) == len(seen)
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
    # most of the prompt, then token by token
    tail = {r: ids for r, ids in reqs.items() if len(ids) > 1}
    assert_close(replay(eng, one_by_one(tail, 6)), want, TOL[dtype])
    # the first tokens of a sequence one by one from the very start: nothing before them, then fewer tokens than taps
    assert_close(replay(eng, one_by_one({"c": reqs["c"][:12]}, 1)), want, TOL[dtype])
    for sizes in ([2], [3, 2, 17, 2, 31, 5], [64, 2, 9], [7, 1, 1, 24]):
        assert_close(replay(eng, in_portions(tail, sizes)), want, TOL[dtype])
    assert all_given_back(eng)


@pytest.mark.parametrize("name,dtype,poison", [("small", "float32", True), ("wide", "float32", True), ("small", "bfloat16", True),
                                               ("wide", "bfloat16", True), ("ones", "float32", True), ("odd", "float32", True),
                                               ("odd", "bfloat16", True), ("long", "float32", True)])
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
    """The states and rows of a request that pauses are still its own when it comes back."""
    folder, cfg, w = folders["small"]
    reqs = {r: random_ids(cfg["vocab"], 30, seed=s) for r, s in (("a", 1), ("b", 2))}
    want = {r: plain_rows(cfg, w, ids) for r, ids in reqs.items()}
    eng = engine_of(folder, "float32")
    steps = [([("a", reqs["a"][:7], [6])], []), ([("b", reqs["b"][:11], [10])], []), ([("b", reqs["b"][11:12], [0])], []),
             ([("a", reqs["a"][7:9], [0, 1]), ("b", reqs["b"][12:13], [0])], []), ([("b", reqs["b"][13:], [0, 16])], ["b"]),
             ([("a", reqs["a"][9:10], [0])], []), ([("a", reqs["a"][10:], [0, 19])], ["a"])]
    assert_close(replay(eng, steps), want, TOL["float32"])


def test_long_contexts_and_long_decoding(folders):
    """420 tokens past several spans of keys, with states that hardly decay: in a whole prompt, in portions, and decoded."""
    folder, cfg, w = folders["long"]
    ids = random_ids(cfg["vocab"], 420, seed=6)
    want = {"a": plain_rows(cfg, w, ids)}
    eng = engine_of(folder, "float32", page_size=16)
    assert_close(replay(eng, whole({"a": ids})), want, TOL["float32"])
    assert_close(replay(eng, in_portions({"a": ids}, [100, 2, 61, 200])), want, TOL["float32"])
    assert_close(replay(eng, one_by_one({"a": ids}, 30)), want, TOL["float32"])
    eng16 = engine_of(folder, "bfloat16", page_size=16)
    assert_close(replay(eng16, whole({"a": ids})), want, TOL["bfloat16"])
    assert_close(replay(eng16, one_by_one({"a": ids}, 200)), want, TOL["bfloat16"])


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


# ----------------------------------------------------------------------------- what decides the output is made to


def _edge_weights(state):
    """One layer whose recurrent branch and positions are zero and whose convolution passes a row as it is. Queries and keys
    read the first half of a normed row, values the second. Tokens 51 and 52 share the first half of their rows; 51's second
    half has 52's elements in another order (the norm then treats both alike): 51's key points where 52's query points, and
    its value is another. A query of token 52 gives its weight to itself and to a 51 if it sees one, so whether and where
    it finds it decides the output."""
    width = 32
    state["pos"].zero_(), state["l0.norm1"].fill_(1.0), state["l0.mix.right.o"].zero_()
    g = torch.Generator().manual_seed(4)
    key = torch.linalg.qr(torch.randn(16, 16, generator=g))[0]
    dt = state["l0.mix.left.q"].dtype
    q = torch.zeros(2, 24, width)
    q[:, 8:, :16] = key                                  # per head eight turned elements of zero, then the key
    state["l0.mix.left.q"], state["l0.mix.left.k"] = q.reshape(48, width).to(dt), q[0].clone().to(dt)
    v = torch.zeros(16, width)
    v[:, 16:] = torch.linalg.qr(torch.randn(16, 16, generator=g))[0]
    state["l0.mix.left.v"] = v.to(dt)
    for x in "qkv":
        taps = torch.zeros_like(state[f"l0.mix.left.{x}.conv"])
        taps[:, -1] = 1
        state[f"l0.mix.left.{x}.conv"] = taps
    state["l0.mix.left.sink"].fill_(-3.0)
    state["embed"][51, :16] = state["embed"][52, :16]
    state["embed"][51, 16:] = state["embed"][52, 16:].flip(0)


@pytest.mark.parametrize("length", [70, 330])
def test_a_key_that_stands_out_wherever_it_is(length, tmp_path):
    raw = M.model(60 + length, 32, [M.parallel(M.attention(2, 1, 24, 16, 1.2, 3, 40.0, M.rotation(100.0, 8)), M.scan(8, 4, 2, 2), 12)],
                  places=length)
    folder, cfg, w = write_model(tmp_path, raw, 31, _edge_weights)
    base = [t for t in range(1, 60 + length) if t not in (51, 52)][:length]     # no token twice, 51 and 52 nowhere
    q, border, chunk = length - 9, 16 * ((length - 9) // 16), 32 * ((length - 9) // 32)
    cases = {"first": (q, 0), "second": (q, 1), "next_to_it": (q, q - 1), "after_it": (q, q + 1), "page_border": (border + 1, border),
             "last_of_a_page": (border + 1, border - 1), "chunk_border": (chunk + 2, chunk - 1), "middle": (q, length // 2), "none": (q, None)}
    if length > 256:
        cases.update(span_border=(q, 128), last_of_a_span=(q, 127), second_span=(q, 256))
    reqs = {}
    for name, (i, j) in cases.items():
        ids = list(base)
        ids[i] = 52
        if j is not None:
            ids[j] = 51
        reqs[name] = ids
    want = {r: plain_rows(cfg, w, ids) for r, ids in reqs.items()}
    # the construction works: whether the twin is seen decides the logits at the query, and one after it is not seen
    moved = {n: float((want[n][q] - want["none"][q]).abs().max() / want["none"][q].abs().max()) for n in ("first", "next_to_it", "after_it")}
    assert moved["after_it"] < 1e-9 and min(moved["first"], moved["next_to_it"]) > 2 * TOL["bfloat16"], moved
    eng = engine_of(folder, "float32", page_size=16)
    for steps in (whole(reqs), one_by_one(reqs, q - 8), in_portions(reqs, [q, 2, 3])):
        assert_close(replay(eng, steps), want, TOL["float32"])
    eng16 = engine_of(folder, "bfloat16", page_size=16)
    for steps in (whole(reqs), one_by_one(reqs, q - 3)):
        assert_close(replay(eng16, steps), want, TOL["bfloat16"])


def small_pair():
    """The two attention layers of the small model alone, no loop."""
    raw = copy.deepcopy(M.SMALL)
    raw["layers"] = [raw["layers"][0], raw["layers"][2]]
    del raw["loop"]
    return raw


def decides(raw, tmp_path, seed, change, other, moves=500):
    """The engine agrees with the plain rows of a model whose weights ``change`` made; with ``other`` done to the weights or
    the configuration the plain rows would be far from these."""
    folder, cfg, w = write_model(tmp_path, raw, seed, change)
    reqs = {"a": random_ids(cfg["vocab"], 50, seed=4), "b": random_ids(cfg["vocab"], 3, seed=5)}
    want = {r: plain_rows(cfg, w, ids) for r, ids in reqs.items()}
    cfg2, w2 = copy.deepcopy(cfg), {k: v.clone() for k, v in w.items()}
    other(cfg2, w2)
    moved = float((P.forward(w2, cfg2, reqs["a"]).float() - want["a"]).abs().max() / want["a"].abs().max())
    assert moved > moves * TOL["float32"], moved
    eng = engine_of(folder, "float32", page_size=8)
    for steps in (whole(reqs), one_by_one(reqs, 1), in_portions(reqs, [2, 7])):
        assert_close(replay(eng, steps), want, TOL["float32"])
    assert_close(replay(engine_of(folder, "bfloat16"), whole(reqs)), want, TOL["bfloat16"])


def test_a_sink_that_decides_the_output(tmp_path):
    """With small scores the sink is a large share of every denominator: leaving it out, counting it twice, scaling or
    capping it would move the logits far beyond rounding."""
    raw = small_pair()
    for layer in raw["layers"]:
        layer["mixer"]["left"].update(scale=0.02, softcap=1.5)

    def change(state):
        for i in (0, 1):
            s = state[f"l{i}.mix.left.sink"]
            state[f"l{i}.mix.left.sink"] = torch.linspace(1.0, 3.0, s.numel()).to(s.dtype)

    def other(cfg, w):
        for k in w:
            if k.endswith(".sink"):
                w[k] = w[k] - 50.0

    decides(raw, tmp_path, 33, change, other)


def test_scores_that_the_cap_bends(tmp_path):
    raw = small_pair()
    for layer in raw["layers"]:
        layer["mixer"]["left"].update(scale=3.0, softcap=2.0)
    decides(raw, tmp_path, 35, None, lambda cfg, w: [layer["mixer"]["left"].pop("softcap") for layer in cfg["layers"]])


def test_taps_that_decide_a_row(tmp_path):
    """The oldest tap far larger than the others: a wrong row from before a portion (of the state, of another request, of a
    slot that another request had) would change everything."""
    def change(state):
        for k in state:
            if k.endswith(".conv"):
                state[k][:, 0] *= 6

    def other(cfg, w):
        for k in w:
            if k.endswith(".conv"):
                w[k][:, 0] = 0

    decides(small_pair(), tmp_path, 36, change, other)


def test_a_state_that_lasts(tmp_path):
    """Slow decays in both recurrences: the first token still shows at the last of 300."""
    raw = M.model(40, 40, [M.parallel(M.attention(2, 1, 8, 8, 0.1, 2, 5.0), M.scan(48, 16, 4, 3), 16), M.lightning(16, 24, (0.9999, 0.999))],
                  places=320)

    def change(state):
        state["l0.mix.right.A_log"].fill_(-9.0)
        state["l0.mix.left.o"].zero_()
        state["pos"].zero_()

    folder, cfg, w = write_model(tmp_path, raw, 37, change)
    ids = random_ids(cfg["vocab"], 300, seed=8)
    want = plain_rows(cfg, w, ids)
    moved = float((P.forward(w, cfg, [ids[0] ^ 1] + ids[1:])[-1].float() - want[-1]).abs().max() / want[-1].abs().max())
    assert moved > 20 * TOL["float32"], moved
    eng = engine_of(folder, "float32", page_size=16)
    for steps in (whole({"a": ids}), one_by_one({"a": ids}, 2), in_portions({"a": ids}, [31, 2, 64, 1, 17])):
        assert_close(replay(eng, steps), {"a": want}, TOL["float32"])


def test_positions_of_the_embedding_decide_a_row(tmp_path):
    def change(state):
        state["embed"] *= 0.1
        state["pos"] *= 5

    def other(cfg, w):
        w["pos"] = w["pos"].roll(1, 0)

    decides(copy.deepcopy(M.ODD), tmp_path, 38, change, other)


# ----------------------------------------------------------------------------- each mechanism alone, in other models


def test_the_parts_in_models_of_other_designs(tmp_path):
    """The mechanisms are parts: the selective scan alone and lightning attention alone as a layer's mixer, in pre-norm
    and in sandwich layers; the scan beside an attention of another kind with one output product; a pass that begins with
    a sublayer's pending result that has a bias, and the first of an order; the ReLU gate; a scaled embedding without
    positions."""
    from dataclasses import dataclass
    from typing import ClassVar

    from pyre_amd.config.model import ModelConfig
    from pyre_amd.parts.base import (BlockSpec, EmbeddingSpec, LayerCall, LightningAttentionSpec, LMHeadSpec, ModelSpec,
                                     NoPositionSpec, ParallelMixerSpec, PassInputSpec, PostNormBlockSpec, ReluGLUSpec, RMSNormSpec,
                                     SelectiveScanSpec, WindowAttentionSpec)
    from pyre_amd.registry import register_architecture, unregister_architecture
    from pyre_amd.weights import write_random_model

    width, vocab, eps = 44, 61, 1e-5
    ssm_a, ssm_b = {"inner": 36, "state": 6, "dt_rank": 5, "conv": 3}, {"inner": 52, "state": 20, "dt_rank": 8, "conv": 1}
    light = {"heads": 3, "dim": 10, "vdim": 6, "decay": [0.9, 0.4, 0.99]}

    @dataclass(frozen=True)
    class ToyConfig(ModelConfig):
        architecture: ClassVar[str] = "ToyScans"

        @classmethod
        def from_dict(cls, raw):
            return cls()

        def to_dict(self):
            return {"architectures": [self.architecture]}

    def build(cfg):
        norm = lambda n: RMSNormSpec(width, eps, "", name=n)  # noqa: E731
        spec = lambda c, p: SelectiveScanSpec(width, c["inner"], c["state"], c["dt_rank"], c["conv"], p)  # noqa: E731
        attn = WindowAttentionSpec(width, 2, 1, 12, 10, 0.3, NoPositionSpec(), "c.l", window=9, qkv_bias=True, out_bias=True)
        layers = (BlockSpec(spec(ssm_a, "a"), norm("a.n"), ReluGLUSpec(width, 30, "a.f"), norm("a.m")),
                  PostNormBlockSpec(LightningAttentionSpec(width, 3, 10, 6, tuple(light["decay"]), "b", norm_eps=eps), norm("b.n")),
                  BlockSpec(ParallelMixerSpec(width, (attn, spec(ssm_b, "c.r")), (0.7, 1.2)), norm("c.n"), None, None))
        order = (LayerCall(2, enters=True), LayerCall(0, enters=True), LayerCall(1), LayerCall(0, enters=True))
        return ModelSpec(width, vocab, 0, EmbeddingSpec(vocab, width, name="embed", scale=0.8), layers, order, norm("last"),
                         LMHeadSpec(vocab, width, name="head"), pass_input=PassInputSpec(width, "pass"))

    def plain(w, ids):
        x = start = w["embed"][torch.as_tensor(ids)] * 0.8
        T = len(ids)
        seen = torch.tensor([[0 <= i - j < 9 for j in range(T)] for i in range(T)])

        def enter(x):
            return torch.cat([x, start], 1) @ w["pass"].T

        def a(x):
            x = x + P.selective_scan(P.rms_norm(x, w["a.n"], eps), w, "a", ssm_a)
            return x + P.feed_forward(P.rms_norm(x, w["a.m"], eps), w, "a.f")

        def b(x):
            return x + P.rms_norm(P.lightning(x, w, "b", light, eps), w["b.n"], eps)

        def c(x):
            h = P.rms_norm(x, w["c.n"], eps)
            q, k, v = (h @ w[f"c.l.{n}"].T + w[f"c.l.{n}.b"] for n in "qkv")
            o = []
            for hd in range(2):
                s = (q[:, 12 * hd:12 * hd + 12] @ k.T * 0.3).masked_fill(~seen, -math.inf)
                o.append(torch.softmax(s, -1) @ v)
            left = torch.cat(o, 1) @ w["c.l.o"].T + w["c.l.o.b"]
            return x + 0.7 * left + 1.2 * P.selective_scan(h, w, "c.r", ssm_b)

        x = a(enter(b(a(enter(c(enter(x)))))))
        return (P.rms_norm(x, w["last"], eps) @ w["head"].T).float()

    register_architecture(ToyConfig.architecture, ToyConfig, build)
    try:
        write_random_model(tmp_path, ToyConfig(), seed=41, std=0.2, gain_std=0.2)
        _, w = P.read_folder(tmp_path)
        reqs = {r: random_ids(vocab, n, seed=n) for r, n in (("a", 70), ("b", 19))}
        want = {r: plain(w, ids) for r, ids in reqs.items()}
        for dtype in ("float32", "bfloat16"):
            eng = engine_of(tmp_path, dtype)
            for steps in (whole(reqs), in_portions(reqs, [5, 2, 30]), one_by_one(reqs, 4)):
                assert_close(replay(eng, steps), want, TOL[dtype])
    finally:
        unregister_architecture(ToyConfig.architecture)


# ----------------------------------------------------------------------------- the kernels alone


def close(got, want, tol):
    return float((got.cpu().double() - want.cpu()).abs().max()) < tol * float(want.abs().max())


@pytest.mark.parametrize("inner,N,rank,parts", [(32, 16, 8, 1), (5, 1, 1, 2), (33, 5, 3, 1), (64, 8, 16, 3), (40, 9, 7, 1), (96, 17, 12, 2), (24, 24, 40, 1),
                                                (70, 25, 4, 1), (32, 32, 224, 4), (31, 48, 9, 1), (32, 64, 10, 1), (16, 65, 33, 2), (20, 128, 8, 1),
                                                (12, 129, 16, 1), (8, 256, 100, 1), (900, 16, 24, 1),
                                                (831, 27, 6, 1), (850, 60, 8, 1)])
def test_the_selective_scan_kernels(inner, N, rank, parts):
    """The scan over requests of 0 to 75 tokens, cut in two and whole the same bits, and the step of single tokens, from
    states in slots of no order, against float64."""
    from pyre_amd.hip import ops

    g = torch.Generator().manual_seed(inner + N)
    rnd = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    lens = [1, 75, 0, 2, 33]
    n, S, slots_n = sum(lens), len(lens), 7
    slots = torch.tensor([3, 0, 5, 6, 1], dtype=torch.int32)
    q_start = torch.tensor([0, *np.cumsum(lens)], dtype=torch.int32)
    g0, width = 3, inner + 5
    z, sel, gate, x = rnd(parts, n, inner), rnd(parts, n, rank + 2 * N + 4), rnd(parts, n, width), rnd(n, inner)
    dt_b, D, A = rnd(inner), rnd(inner), -torch.exp(rnd(inner, N))
    A2 = (A.double() * math.log2(math.e)).float()
    state = rnd(slots_n, inner, N)
    dt_w = 0.3 * rnd(inner, rank)

    def plain(zz, xx, ss, gg, S0):
        dt = torch.nn.functional.softplus(zz + dt_b.double())
        out = []
        for t in range(zz.shape[0]):
            S0 = torch.exp(dt[t][:, None] * A.double()) * S0 + (dt[t] * xx[t])[:, None] * ss[t, rank:rank + N][None]
            out.append((S0 @ ss[t, rank + N:rank + 2 * N] + D.double() * xx[t]) * P.silu(gg[t, g0:g0 + inner]) * 0.7)
        return (torch.stack(out) if out else torch.zeros(0, inner, dtype=torch.float64)), S0

    d = lambda t: t.contiguous().to(DEV)  # noqa: E731
    zs, ss, gs = z.double().sum(0), sel.double().sum(0), gate.double().sum(0)

    def run(kernel_lens, first, st, out, only=None):
        if only is not None and not kernel_lens[only]:
            return
        rows = [range(int(q_start[i]) + first[i], int(q_start[i]) + first[i] + kernel_lens[i]) for i in range(S)]
        pick = torch.tensor([r for rr in rows for r in rr], dtype=torch.long)
        qs = torch.tensor([0, *np.cumsum(kernel_lens)], dtype=torch.int32)
        o = torch.full((len(pick), inner + 3), 9.0, device=DEV)
        ops.ssm_scan(ops.Partials(d(z[:, pick])), d(dt_b), d(x[pick]), ops.Partials(d(sel[:, pick])), rank, ops.Partials(d(gate[:, pick])), g0,
                     d(A2), d(D), st, d(qs) if only is None else d(torch.tensor([0, kernel_lens[only]], dtype=torch.int32)),
                     d(slots) if only is None else d(slots[only:only + 1]), S if only is None else 1, 0.7, o, len(pick))
        assert bool((o[:, inner:] == 9.0).all())
        out[pick] = o[:, :inner].cpu()

    whole_out, cut_out, st, st2 = torch.zeros(n, inner), torch.zeros(n, inner), d(state), d(state)
    run(lens, [0] * S, st, whole_out)
    half = [k // 3 for k in lens]
    run(half, [0] * S, st2, cut_out)
    run([k - h for k, h in zip(lens, half)], half, st2, cut_out)
    assert torch.equal(whole_out, cut_out) and torch.equal(st, st2)
    # a request alone (where few channels make few blocks, sixteen lanes to a channel instead of eight): the same bits
    alone, st3 = torch.zeros(n, inner), d(state)
    for i in range(S):
        run([k if j == i else 0 for j, k in enumerate(lens)], [0] * S, st3, alone, only=i)
    assert torch.equal(whole_out, alone) and torch.equal(st, st3)
    for i in range(S):
        a, b = int(q_start[i]), int(q_start[i + 1])
        want, S1 = plain(zs[a:b], x[a:b].double(), ss[a:b], gs[a:b], state[slots[i]].double())
        if b > a:
            assert close(whole_out[a:b], want, 1e-5)
        assert close(st[slots[i].item()], S1, 1e-5)
    for i in set(range(slots_n)) - set(slots.tolist()):
        assert torch.equal(st[i].cpu(), state[i])
    # one token a request, the step sizes' product inside, in both types of weights and rows
    zs1 = ss[:S, :rank] @ dt_w.double().T
    for dt, tol in ((torch.float32, 2e-5), (torch.bfloat16, 2e-2)):
        wd, xd = dt_w.to(dt), x[:S].to(dt)
        zs1 = ss[:S, :rank] @ wd.double().T
        st, out = d(state), torch.zeros(S, inner, device=DEV, dtype=dt)
        ops.ssm_step(d(torch.cat([wd, torch.full((inner, 5), float("nan"), dtype=dt)], 1)), d(dt_b), d(xd), ops.Partials(d(sel[:, :S])), rank,
                     ops.Partials(d(gate[:, :S])), g0, d(A2), d(D), st, d(slots), S, 0.7, out)
        for i in range(S):
            want, S1 = plain(zs1[i:i + 1], xd[i:i + 1].double(), ss[i:i + 1], gs[i:i + 1], state[slots[i]].double())
            assert close(out[i:i + 1], want, tol) and close(st[slots[i].item()], S1, 2e-5)


@pytest.mark.parametrize("inner,taps,parts", [(40, 4, 1), (40, 4, 3), (7, 3, 2), (64, 1, 1), (1028, 8, 1), (24, 9, 2), (2, 16, 1)])
def test_the_convolution_of_the_scan(inner, taps, parts):
    """Requests shorter and longer than the taps, from states in slots of no order; then a step of single tokens, whose state
    is brought up to date as it is read, against the same step in the other form."""
    from pyre_amd.hip import ops

    g = torch.Generator().manual_seed(inner * taps)
    rnd = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    lens, slots = [1, 2, 20, taps], torch.tensor([2, 5, 0, 3], dtype=torch.int32)
    n, S, col0 = sum(lens), len(lens), 4
    width = col0 + inner + (-(col0 + inner) % 4)
    proj, taps_w, bias = rnd(parts, n, width), rnd(taps, inner), rnd(inner)
    state = rnd(6, max(taps - 1, 1), inner)
    q_start = torch.tensor([0, *np.cumsum(lens)], dtype=torch.int32)
    seq = torch.tensor([i for i, k in enumerate(lens) for _ in range(k)], dtype=torch.int32)
    u = proj.double().sum(0)[:, col0:col0 + inner]
    d = lambda t: t.contiguous().to(DEV)  # noqa: E731
    for dtype, tol in ((torch.float32, 3e-6), (torch.bfloat16, 1e-2)):
        st = d(state)
        x = torch.zeros(n, inner, device=DEV, dtype=dtype)
        ops.ssm_conv(ops.Partials(d(proj)), col0, d(taps_w), d(bias), st if taps > 1 else None, d(slots), d(seq), d(q_start), S, x, n)
        for i in range(S):
            a, b = int(q_start[i]), int(q_start[i + 1])
            rows = torch.cat([state[slots[i]].double(), u[a:b]]) if taps > 1 else u[a:b]
            want = torch.stack([(taps_w.double() * rows[t:t + taps]).sum(0) for t in range(b - a)]) + bias.double()
            assert close(x[a:b], P.silu(want), tol)
            if taps > 1:
                assert close(st[slots[i].item()], rows[-(taps - 1):], 1e-6)
        if taps > 1:
            assert torch.equal(st[1].cpu(), state[1]) and torch.equal(st[4].cpu(), state[4])
        one, two = st.clone(), st.clone()
        xa, xb = torch.zeros(S, inner, device=DEV, dtype=dtype), torch.zeros(S, inner, device=DEV, dtype=dtype)
        arrays = (d(slots), d(torch.arange(S, dtype=torch.int32)), d(torch.arange(S + 1, dtype=torch.int32)), S)
        p = ops.Partials(d(proj[:, :S]))
        ops.ssm_conv(p, col0, d(taps_w), d(bias), one if taps > 1 else None, *arrays, xa, S, single=True)
        ops.ssm_conv(p, col0, d(taps_w), d(bias), two if taps > 1 else None, *arrays, xb, S, single=False)
        assert torch.equal(xa, xb) and torch.equal(one, two)


@pytest.mark.parametrize("dk,dv,taps", [(16, 12, 4), (16, 12, 1), (10, 7, 3), (8, 4, 9)])
def test_a_convolutions_state_in_a_step_of_single_tokens(dk, dv, taps):
    """The attention's projections behind a convolution: the form that leaves the new state behind itself against the one
    with a kernel of its own, a request without a page slot among them."""
    from pyre_amd.hip import ops

    g = torch.Generator().manual_seed(dk + taps)
    nq, nkv, S, page = 3, 1, 4, 8
    channels = (nq + nkv) * dk + nkv * dv
    proj = torch.randn(2, S, channels + (-channels % 4), generator=g).to(DEV)
    taps_w, state = torch.randn(taps, channels, generator=g).to(DEV), torch.randn(6, max(taps - 1, 1), channels, generator=g).to(DEV)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)  # noqa: E731
    got = []
    for single in (True, False):
        st, q = state.clone(), torch.zeros(S, nq * dk, device=DEV)
        k, v = torch.zeros(3, nkv, page, dk, device=DEV), torch.zeros(3, nkv, page, dv, device=DEV)
        ops.conv_qkv_write(ops.Partials(proj), 0, taps_w, st if taps > 1 else None, i32([4, 0, 5, 2]), i32([0, 1, 2, 3]), i32([0, 1, 2, 3, 4]), S,
                           None, None, 1e-6, None, None, 0, True, i32([0, 5, 9, 2]), q, k, v, None, i32([3, -1, 17, 8]), S, nq, nkv, dk, dv, page,
                           single=single)
        got.append((q, k, v, st))
    assert all(torch.equal(a, b) for a, b in zip(*got))
    if taps > 1:
        u = proj.double().sum(0)[:, :channels]
        for s, slot in enumerate([4, 0, 5, 2]):
            assert close(got[0][3][slot], torch.cat([state[slot, 1:].double(), u[s:s + 1]]).cpu(), 1e-6)


@pytest.mark.parametrize("nq,nkv,dk,dv,window,keep,cap,with_sink,gate_dim", [
    (6, 2, 64, 40, 0, 0, 20.0, True, 0), (5, 1, 128, 128, 0, 0, 0.0, True, 0), (4, 4, 24, 64, 300, 5, 5.0, False, 1), (3, 1, 96, 16, 40, 0, 0.0, True, 2),
    (9, 1, 32, 136, 0, 0, 3.0, False, 2)])
def test_tiles_whose_keys_are_dealt_to_several_blocks(nq, nkv, dk, dv, window, keep, cap, with_sink, gate_dim):
    """The 16-bit tile kernel whole and in parts against float64 on the same values, to the rounding of the output; two
    requests, one that goes on behind earlier keys, tiles that are not full, parts that hold all, some or one chunk."""
    from pyre_amd.hip import ops

    g = torch.Generator().manual_seed(nq * dk + window)
    page, lens, first = 16, (700, 90), (0, 61)          # the second request brings its tokens 61 .. 89
    rows = [(r, t) for r in (0, 1) for t in range(first[r], lens[r])]
    n = len(rows)
    ks, vs = [torch.randn(m, nkv, dk, generator=g).bfloat16() for m in lens], [torch.randn(m, nkv, dv, generator=g).bfloat16() for m in lens]
    q = torch.randn(n, nq, dk, generator=g).bfloat16()
    pages = [-(-m // page) for m in lens]
    order = torch.randperm(sum(pages) + 3, generator=g)
    kc, vc = (torch.full((sum(pages) + 3, nkv, page, d), float("nan"), dtype=torch.bfloat16) for d in (dk, dv))
    table = torch.full((2, pages[0]), -1, dtype=torch.int32)
    for r in (0, 1):
        table[r, :pages[r]] = order[r * pages[0]:r * pages[0] + pages[r]].int()
        for t in range(lens[r]):
            kc[table[r, t // page], :, t % page], vc[table[r, t // page], :, t % page] = ks[r][t], vs[r][t]
    sink = torch.randn(nq, generator=g) + 2
    gate = torch.rand(n, nq * (dv if gate_dim == 2 else 1), generator=g) if gate_dim else None
    scale = 2.0 / dk ** 0.5
    want, at = torch.zeros(n, nq, dv, dtype=torch.float64), 0
    for r in (0, 1):
        i, j = torch.arange(first[r], lens[r])[:, None], torch.arange(lens[r])[None]
        seen = (j <= i) & (((i - j < window) | (j < keep)) if window else torch.ones(1, dtype=torch.bool))
        for head in range(nq):
            m = lens[r] - first[r]
            x = q[at:at + m, head].double() @ ks[r][:, head // (nq // nkv)].double().T * scale
            x = (cap * torch.tanh(x / cap) if cap else x).masked_fill(~seen, -math.inf)
            if with_sink:
                x = torch.cat([x, sink[head].double().expand(m, 1)], 1)
            want[at:at + m, head] = torch.softmax(x, -1)[:, :lens[r]] @ vs[r][:, head // (nq // nkv)].double()
        at += lens[r] - first[r]
    if gate is not None:
        want = want * gate.double().view(n, nq, -1)
    want = (want * 0.5).reshape(n, -1)
    tiles = [(t, min(32, 700 - t)) for t in range(0, 700, 32)] + [(700, 5), (705, 24)]
    d = lambda t: None if t is None else t.contiguous().to(DEV)  # noqa: E731
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)  # noqa: E731
    args = (i32(tiles), len(tiles), i32([t for _, t in rows]), i32([r for r, _ in rows]), d(table), nq, nkv, dk, dv, page, scale, cap, None, 0, window, keep)
    ulp = 2.0 ** -8
    for splits, per in ((1, 1), (2, 11), (3, 4), (8, 3), (8, 1), (5, 40)):
        out = torch.zeros(n, nq * dv + 8, device=DEV, dtype=torch.bfloat16)
        scratch = torch.full((n * nq * splits * (dv + 4),), float("nan"), device=DEV) if splits > 1 else None
        ops.attn_biased_tile(d(q.view(n, -1)), out, d(kc), d(vc), d(gate), 0.5, *args, sink=d(sink) if with_sink else None,
                             gate_dim=dv if gate_dim == 2 else 1, scratch=scratch, splits=splits, per=per)
        got = out[:, :nq * dv].cpu().double()
        assert bool(((got - want).abs() <= ulp * want.abs() + 4e-6).all()), (splits, per, float(((got - want).abs() - ulp * want.abs()).max()))
        assert not bool(out[:, nq * dv:].any())


def test_the_plan_of_a_tiles_parts():
    from pyre_amd.hip.ops import attn_biased_tile_plan

    for args in ((64, 14, 2, 2048), (1, 4, 2, 33), (3, 8, 8, 100000), (64, 28, 4, 32768), (64, 14, 2, 2048, 1024, 4), (5, 3, 1, 700, 0, 0, 64)):
        splits, per = attn_biased_tile_plan(*args, units=256)
        assert splits >= 1 and per >= 1 and (splits - 1) * per < -(-args[3] // 32)
    assert attn_biased_tile_plan(64, 14, 2, 2048, units=256) == (6, 11)
    assert attn_biased_tile_plan(2048, 14, 2, 2048, units=256)[0] == 1        # many tiles fill the chip whole
    assert attn_biased_tile_plan(1, 4, 2, 33, units=256)[0] == 1              # nothing to deal


@pytest.mark.parametrize("rank,padded,parts", [(5, 8, 1), (16, 16, 3), (1, 8, 2), (24, 24, 1)])
def test_operands_of_the_step_sizes_product(rank, padded, parts):
    from pyre_amd.hip import ops

    sel = torch.randn(parts, 9, rank + 6, generator=torch.Generator().manual_seed(rank)) * 3
    want = sel.double().sum(0)[:, :rank]
    out = torch.full((9, padded), 7.0, device=DEV)
    ops.ssm_low(ops.Partials(sel.to(DEV)), rank, out, 9)
    assert close(out[:, :rank], want, 1e-6) and bool((out[:, rank:] == 0).all())
    pair = torch.full((9, 2 * padded), 7.0, device=DEV, dtype=torch.bfloat16)
    ops.ssm_low(ops.Partials(sel.to(DEV)), rank, pair, 9)
    assert close(pair[:, :rank].float() + pair[:, padded:padded + rank].float(), want, 2.0 ** -16)
    assert bool((pair.view(9, 2, padded)[:, :, rank:] == 0).all())


@pytest.mark.parametrize("heads,dk,dv,n", [(3, 8, 12, 5), (1, 1, 1, 3), (2, 5, 7, 4), (6, 16, 260, 3), (28, 4, 128, 2)])
def test_the_ends_of_lightning_attention(heads, dk, dv, n):
    """silu on queries, keys and values (not on the gate) into the recurrence's rows; the norm over all heads with the gate."""
    from pyre_amd.hip import ops

    g = torch.Generator().manual_seed(heads * dv)
    hk, hv = heads * dk, heads * dv
    width = 2 * hk + 2 * hv + (-(2 * hk + 2 * hv) % 4)
    proj = torch.randn(2, n, width, generator=g)
    p = proj.double().sum(0)
    logs = -torch.rand(heads, generator=g)
    x = torch.zeros(n, ops.gla_row_width(heads, dk, dv), device=DEV)
    ops.retention_prepare(ops.Partials(proj.to(DEV)), 0, logs.to(DEV), None, None, 0, False, torch.arange(n, dtype=torch.int32, device=DEV), 1.0,
                          x, n, heads, dk, dv, silu=True)
    want = torch.cat([P.silu(p[:, :2 * hk]), logs.double().repeat_interleave(dk).expand(n, hk), P.silu(p[:, 2 * hk:2 * hk + hv]),
                      p[:, 2 * hk + hv:2 * hk + 2 * hv]], 1)
    assert close(x, want, 3e-6)
    o, gain = torch.randn(n, hv, generator=g), 1 + 0.3 * torch.randn(hv, generator=g)
    ref = P.rms_norm(o.double(), gain.double(), 1e-3) * torch.sigmoid(p[:, 2 * hk + hv:2 * hk + 2 * hv]) * 0.6
    for dtype, tol in ((torch.float32, 3e-6), (torch.bfloat16, 1e-2)):
        out = torch.full((n, hv + 4), 5.0, device=DEV, dtype=dtype)
        ops.gla_finish_wide(o.to(DEV), x, gain.to(DEV), 1e-3, 0.6, out, n, heads, dk, dv)
        assert close(out[:, :hv], ref, tol) and bool((out[:, hv:] == 5).all())


@pytest.mark.parametrize("n,inter,k", [(3, 40, 64), (20, 96, 256), (100, 128, 192), (300, 64, 128), (5, 37, 50)])
def test_the_relu_gate_in_every_kernel_that_finishes_a_gated_unit(n, inter, k):
    from pyre_amd.hip import ops
    from pyre_amd.parts.feedforward import ReluGLU

    g = torch.Generator().manual_seed(n)
    x, w = torch.randn(n, k, generator=g), torch.randn(2 * inter, k, generator=g) / k ** 0.5
    x[0] = 0                                                     # a gate of exactly zero
    for dtype, tol in ((torch.float32, 1e-6), (torch.bfloat16, 1e-2)):
        gu = (x.to(dtype).double() @ w.to(dtype).double().T).to(dtype)
        want = torch.relu(gu[:, :inter].double()) * gu[:, inter:].double()
        limit, slope, shift, cubic = ReluGLU.UNIT
        out = torch.full((n, inter), 3.0, device=DEV, dtype=dtype)
        ops.clipped_glu(ops.Partials(gu[None].contiguous().to(DEV)), out, n, limit, slope, shift, cubic)
        assert close(out, want, tol) and bool((out[0] == 0).all())
    xb, wb = x.bfloat16().to(DEV), w.bfloat16().to(DEV)
    exact = x.bfloat16().double() @ w.bfloat16().double().T
    want = torch.relu(exact[:, :inter]) * exact[:, inter:]
    for kernel, takes in ((ops.gemm_skinny_silu_bf16, n <= 64 and ops.gemm_skinny_supports(n, 2 * inter, k, k, k)),
                          (ops.gemm_mid_silu_bf16, n <= 256 and ops.gemm_mid_supports(n, 2 * inter, k, k, k))):
        if takes:
            out = torch.full((n, inter), 3.0, device=DEV, dtype=torch.bfloat16)
            kernel(xb, wb, out, n, ReluGLU.UNIT)
            assert close(out, want, 2e-2) and bool((out[0] == 0).all())


def test_an_embedding_with_a_factor_and_places():
    from pyre_amd.hip import ops

    g = torch.Generator().manual_seed(8)
    ids, pos = [3, 19, 0, 7], [0, 5, 8, 2]
    for dtype, width in ((torch.float32, 300), (torch.bfloat16, 300), (torch.bfloat16, 37), (torch.float32, 3584), (torch.bfloat16, 5124),
                         (torch.bfloat16, 9000)):
        table, places = torch.randn(20, width, generator=g).to(dtype), torch.randn(9, width, generator=g).to(dtype)
        i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)  # noqa: E731
        out = torch.zeros(4, width, device=DEV)
        ops.embed(table.to(DEV), i32(ids), out, 0.3, i32(pos), places.to(DEV))
        assert close(out, table[ids].double() * 0.3 + places[pos].double(), 1e-6)
        ops.embed(table.to(DEV), i32(ids), out, 0.3)
        assert close(out, table[ids].double() * 0.3, 1e-6)


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
    """The scheduler runs one step ahead, its tokens fed on the device. With graphs the decode steps are captured and
    replayed."""
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
