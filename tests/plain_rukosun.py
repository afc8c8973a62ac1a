"""The Rukosun design, plainly: whole sequences, float64, no cache, one function per mechanism.

Slow on purpose (loops over tokens and heads where a loop says most clearly what is computed)
and independent of ``pyre_amd``: it reads ``config.json`` as a dictionary and the tensors by
their names. The tests compare the engine with it.

Notation: ``h`` the rows [T, width] that a sublayer reads, ``i`` a query's position, ``j`` a
key's, both counted from 0 within the sequence; ``W x`` for a matrix stored [out, in].
"""

from __future__ import annotations

import json
import math
from pathlib import Path

import torch

F = torch.float64


def read_folder(folder) -> tuple[dict, dict]:
    """(config as a dictionary, tensors as float64 / int64) of a model folder."""
    from safetensors.torch import load_file

    folder = Path(folder)
    cfg = json.loads((folder / "config.json").read_text())
    raw = load_file(str(folder / "model.safetensors"))
    return cfg, {k: (v.to(F) if v.is_floating_point() else v.long()) for k, v in raw.items()}


# ----------------------------------------------------------------------------- small pieces


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(w, name, x, eps):
    """Mean taken off, divided by the root of the mean squared deviation (+ eps), a weight and a bias."""
    dev = x - x.mean(-1, keepdim=True)
    return dev / torch.sqrt((dev * dev).mean(-1, keepdim=True) + eps) * w[name] + w[name + ".b"]


def embed(cfg, w, ids):
    """Token row, plus the row of the pair (previous token, token), plus the position's row."""
    b = cfg["embedding"]["bigram"]
    rows = []
    for p, t in enumerate(ids):
        pair = b["buckets"] if p == 0 else (ids[p - 1] * b["mul_prev"] + t * b["mul_cur"]) % b["buckets"]
        rows.append(w["embed"][t] + w["bigram"][pair] + w["pos"][p])
    return torch.stack(rows)


def rotate(x, rot, neighbours):
    """x [T, heads, d]: pair n of every head turned by the angle position * base^(-2 n / dims); the pair is elements
    2 n and 2 n + 1 (``neighbours``) or n and n + dims / 2; elements from ``dims`` on pass."""
    dims, base = int(rot["dims"]), float(rot["base"])
    out = x.clone()
    for t in range(x.shape[0]):
        for n in range(dims // 2):
            a = t * base ** (-2.0 * n / dims)
            c, s = math.cos(a), math.sin(a)
            p, q = (2 * n, 2 * n + 1) if neighbours else (n, n + dims // 2)
            u, v = x[t, :, p], x[t, :, q]
            out[t, :, p] = u * c - v * s
            out[t, :, q] = v * c + u * s
    return out


def window_softmax(q, k, v, scale, window, sink=None):
    """q, k [T, H, d], v [T, H, dv] -> [T, H * dv]. Query i sees keys j with 0 <= i - j < window (window 0: every
    j <= i). ``sink`` [H]: exp(sink) joins the denominator, without a value."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for i in range(T):
        lo = max(0, i - window + 1) if window else 0
        for hd in range(H):
            s = (k[lo:i + 1, hd] @ q[i, hd]) * scale
            m = float(s.max()) if sink is None else max(float(s.max()), float(sink[hd]))
            e = torch.exp(s - m)
            den = e.sum() + (0.0 if sink is None else torch.exp(sink[hd] - m))
            out[i, hd] = (e / den) @ v[lo:i + 1, hd]
    return out.reshape(T, -1)


# ----------------------------------------------------------------------------- sublayers


def latent_attention(w, p, m, h, eps, first_kind):
    """Keys and values of all heads made of one compressed row per token, beside one turned key part that the heads
    share. ``first_kind``: queries through a compressed row of their own, neighbouring pairs turned, a sink in the
    softmax and a gate per output element; otherwise plain queries, half-and-half pairs, neither sink nor gate."""
    T, H, d, r, dv, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    if first_kind:
        q = (unit_rms(h @ w[f"{p}.dq"].T, eps) * w[f"{p}.dq.norm"]) @ w[f"{p}.uq"].T
    else:
        q = h @ w[f"{p}.q"].T
    q = q.reshape(T, H, d + r)
    both = h @ w[f"{p}.dkv"].T
    c = unit_rms(both[:, :rank], eps) * w[f"{p}.dkv.norm"]
    shared = rotate(both[:, rank:].reshape(T, 1, r), m["rot"], first_kind)
    k = torch.cat([(c @ w[f"{p}.uk"].T).reshape(T, H, d), shared.expand(T, H, r)], dim=2)
    v = (c @ w[f"{p}.uv"].T).reshape(T, H, dv)
    q = torch.cat([q[:, :, :d], rotate(q[:, :, d:], m["rot"], first_kind)], dim=2)
    window = int((m.get("mask") or {}).get("size", 0))
    o = window_softmax(q, k, v, m["scale"], window, w[f"{p}.sink"] if first_kind else None)
    if first_kind:
        o = o * torch.sigmoid(h @ w[f"{p}.g"].T)
    return o @ w[f"{p}.o"].T


def poly_norm(z, abce, eps):
    """a N(z) + b N(z^2) + c N(z^3) + e, N dividing a row by its root mean square."""
    a, b, c, e = abce
    return a * unit_rms(z, eps) + b * unit_rms(z ** 2, eps) + c * unit_rms(z ** 3, eps) + e


def feed_forward(w, p, h, eps):
    return poly_norm(h @ w[f"{p}.up"].T, w[f"{p}.act"], eps) @ w[f"{p}.down"].T


def through_streams(w, p, streams, sublayer):
    """streams [s, T, width]: the sublayer reads one mixture of them and its result goes back to all of them, which
    are mixed with each other at the same time (``mix[s, t]``: from s to t)."""
    u = torch.einsum("s,stw->tw", w[f"{p}.in"], streams)
    y = sublayer(u)
    mixed = torch.einsum("sr,stw->rtw", w[f"{p}.mix"], streams)
    return mixed + w[f"{p}.out"][:, None, None] * y[None]


def layer_order(cfg) -> list[int]:
    """The layers in the order in which they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    return [*range(loop["start"]), *(list(range(loop["start"], loop["stop"])) * loop["times"]), *range(loop["stop"], n)]


def forward(w, cfg, ids, return_hidden=False):
    """Logits [T, vocab]; with ``return_hidden`` also the sum of the streams after every layer run."""
    eps = float(cfg["norm"]["eps"])
    streams = embed(cfg, w, ids)[None].repeat(cfg["streams"], 1, 1)
    hidden = []
    for i in layer_order(cfg):
        layer, p = cfg["layers"][i], f"l{i}"
        first = {"latent_attention": True, "latent_attention_2": False}[layer["type"]]
        streams = through_streams(w, f"{p}.hc1", streams, lambda u: latent_attention(
            w, f"{p}.mix", layer["mixer"], layer_norm(w, f"{p}.norm1", u, eps), eps, first))
        if layer.get("mlp") is not None:
            streams = through_streams(w, f"{p}.hc2", streams, lambda u: feed_forward(
                w, f"{p}.mlp", layer_norm(w, f"{p}.norm2", u, eps), eps))
        hidden.append(streams.sum(0))
    logits = layer_norm(w, "final.norm", streams.sum(0), eps) @ w["head"].T
    return (logits, hidden) if return_hidden else logits
