"""The Pinozen design without a GPU: its configuration, its parts' manifest and caches, its rotary tables, and the plain
implementation's mechanisms against properties that follow from their definitions."""

from __future__ import annotations

import copy
import math

import pytest
import torch

import pinozen_models as M
import plain_pinozen as P
from pyre_amd.config.model import ConfigError
from pyre_amd.registry import config_from_dict

F = torch.float64


def built(raw):
    from pyre_amd.parts.model import LayeredModel
    from pyre_amd.registry import get_architecture

    return LayeredModel(get_architecture("Pinozen").build(config_from_dict(raw)))


@pytest.mark.parametrize("name", list(M.ALL))
def test_configuration_round_trip_and_manifest(name):
    from pyre_amd.parts.base import PagedCacheSpec, StateCacheSpec

    raw = M.ALL[name]
    cfg = config_from_dict(raw)
    assert config_from_dict(cfg.to_dict()) == cfg and cfg.architecture == "Pinozen"
    model = built(raw)
    names = {s.name: s.shape for s in model.tensor_specs()}
    width = raw["width"]
    want = {"embed": (raw["vocab"], width), "pos": (raw["max_positions"], width), "final.norm": (width,)}
    if "loop" in raw:
        want["loop.in"] = (width, 2 * width)
    for i, layer in enumerate(raw["layers"]):
        p, m = f"l{i}", layer["mixer"]
        want[f"{p}.norm1"] = (width,)
        if layer["type"] == "lightning":
            hk, hv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            want.update({f"{p}.mix.{x}": (rows, width) for x, rows in (("q", hk), ("k", hk), ("v", hv), ("g", hv))})
            want.update({f"{p}.mix.o": (width, hv), f"{p}.mix.norm": (hv,)})
        else:
            a, r = m["left"], m["right"]
            rows = {"q": a["heads"] * a["dim"], "k": a["kv_heads"] * a["dim"], "v": a["kv_heads"] * a["vdim"]}
            want.update({f"{p}.mix.left.{x}": (n, width) for x, n in rows.items()})
            if a.get("conv"):
                want.update({f"{p}.mix.left.{x}.conv": (n, a["conv"]) for x, n in rows.items()})
            want.update({f"{p}.mix.left.sink": (a["heads"],), f"{p}.mix.left.o": (width, a["heads"] * a["vdim"])})
            n, st, k = r["inner"], r["state"], r["dt_rank"]
            want.update({f"{p}.mix.right.{x}": s for x, s in (
                ("in", (2 * n, width)), ("conv", (n, r["conv"])), ("conv.b", (n,)), ("x", (k + 2 * st, n)), ("dt", (n, k)),
                ("dt.b", (n,)), ("A_log", (n, st)), ("D", (n,)), ("o", (width, n)))})
            want.update({f"{p}.mix.left.out": (width,), f"{p}.mix.right.out": (width,)})
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            want.update({f"{p}.norm2": (width,), f"{p}.mlp.gate": (ff, width), f"{p}.mlp.up": (ff, width), f"{p}.mlp.down": (width, ff)})
    assert names == want
    # every pass of a looped layer keeps pages and states of its own
    runs = P.layer_runs(raw)
    assert [(c.layer, c.enters) for c in model.schedule] == runs == cfg.runs() and all(c.cache_from is None for c in model.schedule)
    for (i, _), specs in zip(runs, model.cache_specs()):
        m = raw["layers"][i]["mixer"]
        if raw["layers"][i]["type"] == "lightning":
            assert specs == [StateCacheSpec((m["heads"], m["dim"], m["vdim"]), "float32")]
            continue
        a, r = m["left"], m["right"]
        channels = (a["heads"] + a["kv_heads"]) * a["dim"] + a["kv_heads"] * a["vdim"]
        shapes = [(a["conv"] - 1, channels)] if a.get("conv", 0) > 1 else []
        shapes += [(r["inner"], r["state"])] + ([(r["conv"] - 1, r["inner"])] if r["conv"] > 1 else [])
        assert isinstance(specs[0], PagedCacheSpec) and specs[0].window == 0
        assert [(s.shape, s.dtype) for s in specs[1:]] == [(s, "float32") for s in shapes]
    assert model.embedding.max_positions == raw["max_positions"]


def test_configurations_that_are_refused():
    def broken(change, raw=M.SMALL):
        raw = copy.deepcopy(raw)
        change(raw)
        with pytest.raises(ConfigError):
            config_from_dict(raw)

    left, right = (lambda r: r["layers"][0]["mixer"]["left"]), (lambda r: r["layers"][0]["mixer"]["right"])
    broken(lambda r: left(r).__setitem__("kv_heads", 3))
    broken(lambda r: left(r).pop("scale"))
    broken(lambda r: left(r).__setitem__("softcap", -1.0))
    broken(lambda r: left(r)["rot"].__setitem__("dims", 5))
    broken(lambda r: left(r)["rot"].__setitem__("dims", 18))
    broken(lambda r: left(r)["rot"].__setitem__("base", 0.0))
    broken(lambda r: left(r)["rot"]["scaling"].pop("original"))
    broken(lambda r: left(r)["rot"]["scaling"].__setitem__("factor", 0.0))
    broken(lambda r: left(r)["rot"]["scaling"].__setitem__("low", 5.0))
    for k in ("inner", "state", "dt_rank", "conv"):
        broken(lambda r: right(r).pop(k))
        broken(lambda r: right(r).__setitem__(k, 0))
    broken(lambda r: r["layers"][0]["mixer"].pop("right"))
    broken(lambda r: r["layers"][1]["mixer"]["decay"].pop())
    broken(lambda r: r["layers"][1]["mixer"]["decay"].__setitem__(0, 1.5))
    broken(lambda r: r["layers"][1]["mixer"].pop("vdim"))
    broken(lambda r: r["layers"][1].__setitem__("type", "retention"))
    broken(lambda r: r["layers"][0]["mlp"].__setitem__("kind", "moe"))
    broken(lambda r: r.__setitem__("max_positions", 0))
    broken(lambda r: r["loop"].__setitem__("stop", 5))
    broken(lambda r: r["loop"].__setitem__("start", 3))
    broken(lambda r: r["loop"].__setitem__("times", 0))
    broken(lambda r: r["loop"].pop("times"))
    broken(lambda r: r["norm"].__setitem__("eps", 0.0))


def test_what_a_configuration_does_not_mention():
    raw = copy.deepcopy(M.SMALL)
    del raw["loop"], raw["logit_scale"], raw["embedding"]
    cfg = config_from_dict(raw)
    assert cfg.loop is None and cfg.logit_scale == 1.0 and cfg.embedding_scale == 1.0
    model = built(raw)
    assert model.pass_input is None and all(s.name != "loop.in" for s in model.tensor_specs())


def test_sizes_that_no_kernel_takes_are_refused_when_the_model_is_built():
    for change in (lambda m: m["left"].__setitem__("dim", 258), lambda m: m["left"].__setitem__("conv", 17),
                   lambda m: m["right"].__setitem__("state", 257), lambda m: m["right"].__setitem__("conv", 17),
                   lambda m: m["right"].__setitem__("dt_rank", 12288)):
        raw = copy.deepcopy(M.SMALL)
        change(raw["layers"][0]["mixer"])
        with pytest.raises(ValueError):
            built(raw)
    raw = copy.deepcopy(M.SMALL)
    raw["layers"][1]["mixer"]["dim"] = 257
    with pytest.raises(ValueError):
        built(raw)


def test_an_entry_that_enters_a_pass_needs_the_models_input_of_passes():
    from dataclasses import replace

    from pyre_amd.parts.model import LayeredModel
    from pyre_amd.registry import get_architecture

    spec = get_architecture("Pinozen").build(config_from_dict(M.SMALL))
    with pytest.raises(ValueError):
        LayeredModel(replace(spec, pass_input=None))


def test_the_order_of_looped_layers():
    cfg = config_from_dict(M.SMALL)
    assert cfg.runs() == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)] == P.layer_runs(M.SMALL)
    raw = copy.deepcopy(M.SMALL)
    raw["loop"] = {"start": 3, "stop": 4, "times": 3}
    assert config_from_dict(raw).runs() == [(0, False), (1, False), (2, False), (3, True), (3, True), (3, True)] == P.layer_runs(raw)


@pytest.mark.parametrize("scaling", [None, (4.0, 1.0, 4.0, 64), (8.0, 2.0, 8.0, 32), (2.0, 1.0, 1.0, 50), (3.0, 0.5, 6.0, 4000)])
def test_rotary_tables_of_frequencies_changed_by_wavelength(scaling):
    from pyre_amd.parts.rotary import rotary_tables

    keys = ("factor", "low", "high", "original")
    base, dims = 500.0, 24
    freqs = P.frequencies(base, dims, dict(zip(keys, scaling)) if scaling else None)
    cos, sin = rotary_tables(dims, base, 300, exact=True, wave_scaling=scaling)
    for t in (0, 1, 77, 299):
        for i, f in enumerate(freqs):
            assert abs(float(cos[t, i]) - math.cos(t * f)) < 1e-7 and abs(float(sin[t, i]) - math.sin(t * f)) < 1e-7
    if scaling:   # the ends of the range do what they should
        factor, low, high, original = scaling
        plain = P.frequencies(base, dims)
        for f, g in zip(plain, freqs):
            if 2 * math.pi / f < original / high:
                assert g == f
            elif 2 * math.pi / f > original / low:
                assert g == f / factor
            else:
                assert f / factor <= g <= f


def test_neighbouring_pairs_are_turned_by_their_own_frequencies():
    x = torch.randn(4, 2, 9, dtype=F, generator=torch.Generator().manual_seed(2))
    rot = {"dims": 6, "base": 50.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 2.0, "original": 30}}
    y = P.rotate_neighbours(x, rot)
    assert torch.allclose(y[0], x[0]) and torch.equal(y[:, :, 6:], x[:, :, 6:])
    a = 3 * P.frequencies(50.0, 6, rot["scaling"])[1]
    assert abs(float(y[3, 1, 2] - (x[3, 1, 2] * math.cos(a) - x[3, 1, 3] * math.sin(a)))) < 1e-14
    assert abs(float(y[3, 1, 3] - (x[3, 1, 3] * math.cos(a) + x[3, 1, 2] * math.sin(a)))) < 1e-14


def test_cap_and_sink_of_the_plain_attention():
    g = torch.Generator().manual_seed(1)
    c = {"heads": 2, "kv_heads": 1, "dim": 5, "vdim": 4, "scale": 0.7, "softcap": 1.3}
    w = {"p.q": torch.randn(10, 6, generator=g, dtype=F), "p.k": torch.randn(5, 6, generator=g, dtype=F),
         "p.v": torch.randn(4, 6, generator=g, dtype=F), "p.o": torch.eye(8, dtype=F), "p.sink": torch.tensor([0.4, -1.0], dtype=F)}
    h = torch.randn(7, 6, generator=g, dtype=F)
    out = P.capped_sink_attention(h, w, "p", c)
    i, a = 4, 1
    q = (w["p.q"] @ h[i])[5 * a:5 * a + 5]
    s = torch.tensor([1.3 * math.tanh(0.7 * float(q @ (w["p.k"] @ h[j])) / 1.3) for j in range(i + 1)], dtype=F)
    want = (torch.exp(s) / (math.exp(-1.0) + torch.exp(s).sum())) @ torch.stack([w["p.v"] @ h[j] for j in range(i + 1)])
    assert torch.allclose(out[i, 4 * a:4 * a + 4], want, atol=1e-12)


def test_a_convolution_hands_the_first_tokens_on_with_zeros_before_them():
    u = torch.tensor([[1.0], [10.0], [100.0]], dtype=F)
    y = P.short_conv(u, torch.tensor([[2.0, 3.0, 5.0]], dtype=F))   # oldest, .., the token itself
    assert y.flatten().tolist() == [5.0, 53.0, 532.0]


def test_the_selective_scan_is_the_sum_over_everything_before():
    """y_t = sum_(s <= t) C_t . (exp(A sum of dt after s) dt_s x_s B_s) + D x_t."""
    g = torch.Generator().manual_seed(3)
    c = {"inner": 3, "state": 4, "dt_rank": 2, "conv": 1}
    T, n, st = 6, 3, 4
    w = {f"p.{k}": torch.randn(*s, generator=g, dtype=F) for k, s in (("in", (6, 5)), ("conv", (n, 1)), ("conv.b", (n,)), ("x", (10, n)),
                                                                     ("dt", (n, 2)), ("dt.b", (n,)), ("A_log", (n, st)), ("D", (n,)))}
    w["p.o"] = torch.eye(n, dtype=F)
    h = torch.randn(T, 5, generator=g, dtype=F)
    out = P.selective_scan(h, w, "p", c)
    both = h @ w["p.in"].T
    x = P.silu(both[:, :n] * w["p.conv"][:, 0] + w["p.conv.b"])
    sel = x @ w["p.x"].T
    dt = torch.log(1 + torch.exp(sel[:, :2] @ w["p.dt"].T + w["p.dt.b"]))
    A = -torch.exp(w["p.A_log"])
    t, ch = 5, 1
    y = w["p.D"][ch] * x[t, ch]
    for s in range(t + 1):
        y = y + (sel[t, 6:] * torch.exp(A[ch] * dt[s + 1:t + 1, ch].sum()) * dt[s, ch] * x[s, ch] * sel[s, 2:6]).sum()
    assert abs(float(out[t, ch] - y * P.silu(both[t, n + ch]))) < 1e-12


def test_lightning_attention_is_the_decayed_sum_of_what_was_seen():
    g = torch.Generator().manual_seed(4)
    c = {"heads": 2, "dim": 3, "vdim": 4, "decay": [0.5, 0.9]}
    w = {f"p.{k}": torch.randn(r, 5, generator=g, dtype=F) for k, r in (("q", 6), ("k", 6), ("v", 8), ("g", 8))}
    w["p.o"], w["p.norm"] = torch.eye(8, dtype=F), torch.rand(8, generator=g, dtype=F)
    h = torch.randn(5, 5, generator=g, dtype=F)
    out = P.lightning(h, w, "p", c, 1e-4)
    q, k, v = (P.silu(h @ w[f"p.{x}"].T).view(5, 2, -1) for x in "qkv")
    t = 4
    o = torch.cat([sum(c["decay"][a] ** (t - s) * (q[t, a] @ k[s, a]) * v[s, a] for s in range(t + 1)) for a in range(2)])
    o = o / math.sqrt(float((o * o).mean()) + 1e-4) * w["p.norm"]       # both heads normed together
    assert torch.allclose(out[t], o * torch.sigmoid(w["p.g"] @ h[t]), atol=1e-12)


def test_every_pass_begins_with_the_stream_and_the_embeddings_output():
    """With a product that drops the stream, every pass starts anew: what an earlier pass did is gone."""
    from pyre_amd.weights import model_tensor_specs, random_state

    raw = copy.deepcopy(M.SMALL)
    w = {k: v.to(F) for k, v in random_state(model_tensor_specs(config_from_dict(raw)), 5, 0.2, 0.2).items()}
    ids = [3, 5, 7, 11]
    w["loop.in"][:, :raw["width"]] = 0
    _, twice = P.forward(w, raw, ids, return_hidden=True)
    assert torch.allclose(twice[2], twice[4])
    raw["loop"]["times"] = 1
    assert torch.allclose(P.forward(w, raw, ids), P.forward(w, M.SMALL, ids))


def test_a_gated_unit_of_infinite_slope_is_the_relu_gate():
    from pyre_amd.parts.feedforward import ReluGLU

    limit, slope, shift, cubic = ReluGLU.UNIT
    assert limit <= 0 and slope == math.inf and shift == 0 and cubic == 0
