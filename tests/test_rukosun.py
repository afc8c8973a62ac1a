"""The Rukosun design without a GPU: its configuration, its parts' manifest and caches, and the plain implementation's
mechanisms against properties that follow from their definitions."""

from __future__ import annotations

import copy
import math

import pytest
import torch

import plain_rukosun as P
import rukosun_models as M
from pyre_amd.config.model import ConfigError
from pyre_amd.registry import config_from_dict

F = torch.float64
ALL = [M.SMALL, M.ONES, M.WIDE, M.ODD, M.LONG]


@pytest.mark.parametrize("raw", ALL)
def test_configuration_round_trip_and_manifest(raw):
    from pyre_amd.parts.base import PagedCacheSpec, StateCacheSpec
    from pyre_amd.parts.model import LayeredModel
    from pyre_amd.registry import get_architecture

    cfg = config_from_dict(raw)
    assert config_from_dict(cfg.to_dict()) == cfg and cfg.architecture == "Rukosun"
    model = LayeredModel(get_architecture(cfg.architecture).build(cfg))
    names = {s.name: s.shape for s in model.tensor_specs() if not s.optional}
    width, S = raw["width"], raw["streams"]
    assert names["embed"] == (raw["vocab"], width) == names["head"] and names["pos"] == (raw["max_positions"], width)
    assert names["bigram"] == (raw["embedding"]["bigram"]["buckets"] + 1, width)
    assert names["final.norm"] == (width,) == names["final.norm.b"]
    for i, layer in enumerate(raw["layers"]):
        p, m = f"l{i}", layer["mixer"]
        H, d, r, dv, rank = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        first = layer["type"] == "latent_attention"
        if first:
            assert names[f"{p}.mix.dq"] == (m["q_rank"], width) and names[f"{p}.mix.dq.norm"] == (m["q_rank"],)
            assert names[f"{p}.mix.uq"] == (H * (d + r), m["q_rank"]) and f"{p}.mix.q" not in names
            assert names[f"{p}.mix.sink"] == (H,) and names[f"{p}.mix.g"] == (H * dv, width)
        else:
            assert names[f"{p}.mix.q"] == (H * (d + r), width)
            assert not any(f"{p}.mix.{x}" in names for x in ("dq", "uq", "sink", "g"))
        assert names[f"{p}.mix.dkv"] == (rank + r, width) and names[f"{p}.mix.dkv.norm"] == (rank,)
        assert names[f"{p}.mix.uk"] == (H * d, rank) and names[f"{p}.mix.uv"] == (H * dv, rank) and names[f"{p}.mix.o"] == (width, H * dv)
        assert names[f"{p}.norm1"] == (width,) == names[f"{p}.norm1.b"]
        for q in (1, 2):
            there = q == 1 or layer["mlp"] is not None
            assert (f"{p}.hc{q}.in" in names) == there
            if there:
                assert names[f"{p}.hc{q}.in"] == (S,) == names[f"{p}.hc{q}.out"] and names[f"{p}.hc{q}.mix"] == (S, S)
        assert (f"{p}.norm2.b" in names) == (layer["mlp"] is not None) == (f"{p}.mlp.act" in names)
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            assert names[f"{p}.mlp.up"] == (ff, width) and names[f"{p}.mlp.down"] == (width, ff) and names[f"{p}.mlp.act"] == (4,)
    # every pass of a looped layer keeps rows of its own; the last entry is the embedding's, the previous token
    order = P.layer_order(raw)
    assert [c.layer for c in model.schedule] == order and all(c.cache_from is None for c in model.schedule)
    kept = model.cache_specs()
    assert len(kept) == len(order) + 1 and isinstance(kept[-1][0], StateCacheSpec) and kept[-1][0].shape == (1,)
    for call, specs in zip(order, kept):
        m = raw["layers"][call]["mixer"]
        assert [type(s) for s in specs] == [PagedCacheSpec] and specs[0].window == (m.get("mask") or {}).get("size", 0)
        assert specs[0].tensors[0].token_shape == (1, m["kv_rank"] + m["rot_dim"])
    assert model.embedding.max_positions == raw["max_positions"]


def test_configurations_that_are_refused():
    def broken(change, raw=M.SMALL):
        raw = copy.deepcopy(raw)
        change(raw)
        with pytest.raises(ConfigError):
            config_from_dict(raw)

    broken(lambda r: r["layers"][0]["mixer"].__setitem__("rot_dim", 7))
    broken(lambda r: r["layers"][0]["mixer"]["rot"].__setitem__("dims", 4))
    broken(lambda r: r["layers"][0]["mixer"]["rot"].__setitem__("base", 0.0))
    broken(lambda r: r["layers"][0]["mixer"].pop("q_rank"))
    broken(lambda r: r["layers"][1]["mixer"].pop("scale"))
    broken(lambda r: r["layers"][1]["mixer"]["mask"].__setitem__("size", -1))
    broken(lambda r: r["layers"][1].__setitem__("type", "latent_attention_3"))
    broken(lambda r: r["layers"][0]["mlp"].__setitem__("kind", "moe"))
    broken(lambda r: r.__setitem__("streams", 0))
    broken(lambda r: r.__setitem__("max_positions", 0))
    broken(lambda r: r["loop"].__setitem__("stop", 5))
    broken(lambda r: r["loop"].__setitem__("start", 4))
    broken(lambda r: r["loop"].pop("times"))
    broken(lambda r: r["embedding"].pop("bigram"))
    broken(lambda r: r["embedding"]["bigram"].__setitem__("buckets", 0))
    broken(lambda r: r["norm"].__setitem__("eps", 0.0))


def test_sizes_that_no_kernel_takes_are_refused_when_the_model_is_built():
    from pyre_amd.parts.model import LayeredModel
    from pyre_amd.registry import get_architecture

    for change in (lambda r: r["layers"][0]["mixer"].__setitem__("kv_rank", 513), lambda r: r.__setitem__("streams", 9)):
        raw = copy.deepcopy(M.SMALL)
        change(raw)
        with pytest.raises(ValueError):
            LayeredModel(get_architecture("Rukosun").build(config_from_dict(raw)))


def test_a_models_streams_and_its_layers_connections_must_agree():
    from dataclasses import replace

    from pyre_amd.parts.model import LayeredModel
    from pyre_amd.registry import get_architecture

    spec = get_architecture("Rukosun").build(config_from_dict(M.SMALL))
    for streams in (0, 2):
        with pytest.raises(ValueError):
            LayeredModel(replace(spec, streams=streams))


def test_the_order_of_looped_layers():
    cfg = config_from_dict(M.SMALL)
    assert cfg.order() == [0, 1, 2, 1, 2, 3] == P.layer_order(M.SMALL)
    raw = copy.deepcopy(M.SMALL)
    raw["loop"] = {"start": 2, "stop": 4, "times": 3}
    assert config_from_dict(raw).order() == [0, 1, 2, 3, 2, 3, 2, 3] == P.layer_order(raw)
    del raw["loop"]
    assert config_from_dict(raw).order() == [0, 1, 2, 3] == P.layer_order(raw)


def test_window_and_sink_of_the_plain_attention():
    g = torch.Generator().manual_seed(1)
    T, H, d, dv = 9, 3, 5, 4
    q, k = (torch.randn(T, H, d, generator=g, dtype=F) for _ in range(2))
    v = torch.randn(T, H, dv, generator=g, dtype=F)
    sink = torch.randn(H, generator=g, dtype=F)
    out = P.window_softmax(q, k, v, 0.7, 4, sink).reshape(T, H, dv)
    i, hd = 7, 2
    s = torch.stack([(q[i, hd] @ k[j, hd]) * 0.7 for j in range(4, 8)])
    want = (torch.exp(s) / (torch.exp(sink[hd]) + torch.exp(s).sum())) @ v[4:8, hd]   # the sink is not scaled
    assert torch.allclose(out[i, hd], want, atol=1e-12)
    # a window of one token without a sink returns the token's own value; no window: everything before it
    alone = P.window_softmax(q, k, v, 0.7, 1).reshape(T, H, dv)
    assert torch.allclose(alone, v, atol=1e-12)
    s = (k[:, 0] @ q[8, 0]) * 0.7
    assert torch.allclose(P.window_softmax(q, k, v, 0.7, 0).reshape(T, H, dv)[8, 0], torch.softmax(s, 0) @ v[:, 0], atol=1e-12)


def test_both_pairings_of_the_rotation():
    x = torch.randn(4, 2, 6, dtype=F, generator=torch.Generator().manual_seed(2))
    rot = {"dims": 6, "base": 50.0}
    for neighbours in (False, True):
        y = P.rotate(x, rot, neighbours)
        assert torch.allclose(y[0], x[0]) and torch.allclose((y * y).sum(-1), (x * x).sum(-1))
        n, p, q = 1, *((2, 3) if neighbours else (1, 4))
        a = 3 * 50.0 ** (-2 * n / 6)
        assert abs(float(y[3, 1, p] - (x[3, 1, p] * math.cos(a) - x[3, 1, q] * math.sin(a)))) < 1e-14
        assert abs(float(y[3, 1, q] - (x[3, 1, q] * math.cos(a) + x[3, 1, p] * math.sin(a)))) < 1e-14
        # scores of turned pairs depend on the distance alone
        u, v = (torch.randn(6, dtype=F, generator=torch.Generator().manual_seed(s)).expand(9, 1, 6) for s in (3, 4))
        tu, tv = P.rotate(u, rot, neighbours), P.rotate(v, rot, neighbours)
        assert abs(float(tu[8, 0] @ tv[5, 0] - tu[4, 0] @ tv[1, 0])) < 1e-12


def test_scores_through_the_compressed_row_are_those_of_the_heads_own_keys():
    """q . (Wuk c) = (Wuk^T q) . c, and the weighted sum of values is Wuv of the weighted sum of rows: what a cache of
    compressed rows rests on."""
    g = torch.Generator().manual_seed(5)
    uk, uv, q = torch.randn(7, 11, generator=g, dtype=F), torch.randn(5, 11, generator=g, dtype=F), torch.randn(7, generator=g, dtype=F)
    c = torch.randn(6, 11, generator=g, dtype=F)
    assert torch.allclose((c @ uk.T) @ q, c @ (uk.T @ q))
    a = torch.softmax((c @ uk.T) @ q, 0)
    assert torch.allclose(a @ (c @ uv.T), uv @ (a @ c))


def test_the_polynomial_activation():
    z = torch.tensor([[1.0, -2.0, 3.0]], dtype=F)
    out = P.poly_norm(z, torch.tensor([0.5, -1.0, 2.0, 0.25], dtype=F), 1e-4)
    r1, r2, r3 = (math.sqrt(sum(v ** (2 * n) for v in (1.0, 2.0, 3.0)) / 3 + 1e-4) for n in (1, 2, 3))
    for i, v in enumerate((1.0, -2.0, 3.0)):
        assert abs(float(out[0, i]) - (0.5 * v / r1 - v * v / r2 + 2 * v ** 3 / r3 + 0.25)) < 1e-12


def test_streams_are_mixed_from_the_old_ones_all_at_once():
    g = torch.Generator().manual_seed(6)
    x = torch.randn(2, 1, 3, generator=g, dtype=F)
    w = {"p.in": torch.tensor([2.0, -1.0], dtype=F), "p.out": torch.tensor([0.5, 3.0], dtype=F),
         "p.mix": torch.tensor([[1.0, 10.0], [100.0, 1000.0]], dtype=F)}
    seen = []
    y = P.through_streams(w, "p", x, lambda u: seen.append(u) or u * 2)
    assert torch.allclose(seen[0], 2 * x[0] - x[1])
    assert torch.allclose(y[0], 1 * x[0] + 100 * x[1] + 0.5 * 2 * seen[0])      # mix is [from, to]
    assert torch.allclose(y[1], 10 * x[0] + 1000 * x[1] + 3.0 * 2 * seen[0])


def test_the_embedding_of_pairs_and_places():
    cfg = {"embedding": {"bigram": {"buckets": 5, "mul_prev": 3, "mul_cur": 2}}}
    g = torch.Generator().manual_seed(7)
    w = {"embed": torch.randn(9, 4, generator=g, dtype=F), "bigram": torch.randn(6, 4, generator=g, dtype=F),
         "pos": torch.randn(8, 4, generator=g, dtype=F)}
    rows = P.embed(cfg, w, [4, 8, 8])
    assert torch.allclose(rows[0], w["embed"][4] + w["bigram"][5] + w["pos"][0])
    assert torch.allclose(rows[1], w["embed"][8] + w["bigram"][(4 * 3 + 8 * 2) % 5] + w["pos"][1])
    assert torch.allclose(rows[2], w["embed"][8] + w["bigram"][(8 * 3 + 8 * 2) % 5] + w["pos"][2])


def test_what_a_layer_without_a_feed_forward_may_have_in_its_file(tmp_path):
    """Its second norm and connection are neither missed nor refused."""
    from safetensors.torch import load_file, save_file

    from pyre_amd.weights import write_random_model
    from pyre_amd.weights.loader import check_against, checkpoint_index
    from pyre_amd.parts.model import LayeredModel
    from pyre_amd.registry import get_architecture

    cfg = config_from_dict(M.SMALL)
    write_random_model(tmp_path, cfg, seed=5, std=0.2, gain_std=0.2)
    state = load_file(str(tmp_path / "model.safetensors"))
    assert "l2.norm2" not in state
    specs = LayeredModel(get_architecture("Rukosun").build(cfg)).tensor_specs()
    check_against(specs, checkpoint_index(tmp_path), tmp_path)
    state.update({"l2.norm2": torch.ones(48), "l2.norm2.b": torch.zeros(48), "l2.hc2.mix": torch.zeros(3, 3)})
    save_file(state, str(tmp_path / "model.safetensors"))
    check_against(specs, checkpoint_index(tmp_path), tmp_path)
