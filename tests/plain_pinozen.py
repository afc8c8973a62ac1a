"""The Pinozen design, plainly: whole sequences, float64, no cache, one function per mechanism.

Slow on purpose (loops over tokens and heads where a loop says most clearly what is computed)
and independent of ``pyre_amd``: it reads ``config.json`` as a dictionary and the tensors by
their names. The tests compare the engine with it.

Notation: ``h`` the rows [T, width] that a sublayer reads, ``i`` a query's position, ``j`` a
key's, both counted from 0 within the sequence.
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


def rms_norm(x, gain, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis, times a gain."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * gain


def silu(z):
    return z * torch.sigmoid(z)


def short_conv(u, taps_w):
    """y[t, c] = sum_j taps_w[c, j] * u[t - (taps - 1) + j, c], rows before the sequence's start being zero:
    the last tap multiplies the token itself, the first the one ``taps - 1`` back."""
    T, taps = u.shape[0], taps_w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] += taps_w[:, j] * u[s]
    return y


def frequencies(base, dims, scaling=None):
    """One frequency per turned pair. With ``scaling`` a pair is told by its wavelength: short ones keep their
    frequency, long ones have it divided by the factor, those between get a mixture of the two."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            wave = 2.0 * math.pi / f
            short, long = scaling["original"] / scaling["high"], scaling["original"] / scaling["low"]
            if wave > long:
                f = f / scaling["factor"]
            elif wave >= short:
                s = (scaling["original"] / wave - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return out


def rotate_neighbours(x, rot):
    """x [T, heads, d]: elements (2i, 2i + 1), i < dims / 2, of every head turned by the angle position * f_i;
    the elements from ``dims`` on pass."""
    out = x.clone()
    pos = torch.arange(x.shape[0], dtype=F)
    for i, f in enumerate(frequencies(rot["base"], rot["dims"], rot.get("scaling"))):
        c, s = torch.cos(pos * f)[:, None], torch.sin(pos * f)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * c - v * s
        out[:, :, 2 * i + 1] = v * c + u * s
    return out


# ----------------------------------------------------------------------------- mixers


def capped_sink_attention(h, w, p, c):
    """Grouped-query causal softmax attention: projections followed by a short convolution over time, queries and
    keys turned in neighbouring pairs, scores squashed by cap * tanh(s / cap), a learned number per head in the
    softmax's denominator (a key without a value, not squashed)."""
    T = h.shape[0]
    H, G, d, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (h @ w[f"{p}.{x}"].T for x in "qkv")
    if c.get("conv"):
        q, k, v = (short_conv(u, w[f"{p}.{x}.conv"]) for x, u in (("q", q), ("k", k), ("v", v)))
    q, k, v = q.view(T, H, d), k.view(T, G, d), v.view(T, G, dv)
    if c.get("rot"):
        q, k = rotate_neighbours(q, c["rot"]), rotate_neighbours(k, c["rot"])
    hidden = torch.ones(T, T, dtype=torch.bool).triu(1)          # j > i
    cap, sink = c.get("softcap"), w[f"{p}.sink"]
    out = torch.zeros(T, H, dv, dtype=F)
    for a in range(H):
        g = a // (H // G)
        s = q[:, a] @ k[:, g].T * c["scale"]                     # [i, j]
        if cap:
            s = cap * torch.tanh(s / cap)
        s = s.masked_fill(hidden, -math.inf)
        m = torch.maximum(s.max(-1).values, sink[a])
        e = torch.exp(s - m[:, None])
        out[:, a] = e / (e.sum(-1) + torch.exp(sink[a] - m))[:, None] @ v[:, g]
    return out.reshape(T, H * dv) @ w[f"{p}.o"].T


def selective_scan(h, w, p, c):
    """A state S [inner, state]: every token scales it by exp(dt A) and adds dt x B, both chosen by the token
    itself, and reads it with C; a path past the state (D x) and a silu gate."""
    T, n, st, r = h.shape[0], c["inner"], c["state"], c["dt_rank"]
    both = h @ w[f"{p}.in"].T
    x, z = both[:, :n], both[:, n:]
    x = silu(short_conv(x, w[f"{p}.conv"]) + w[f"{p}.conv.b"])
    sel = x @ w[f"{p}.x"].T
    low, B, C = sel[:, :r], sel[:, r:r + st], sel[:, r + st:]
    dt = low @ w[f"{p}.dt"].T + w[f"{p}.dt.b"]
    dt = torch.clamp(dt, min=0) + torch.log1p(torch.exp(-dt.abs()))       # softplus
    A = -torch.exp(w[f"{p}.A_log"])
    S = torch.zeros(n, st, dtype=F)
    y = torch.zeros(T, n, dtype=F)
    for t in range(T):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + w[f"{p}.D"] * x[t]
    return (y * silu(z)) @ w[f"{p}.o"].T


def parallel(h, w, p, c, eps):
    """Both mixers on the same rows, each result normed over the width, half their sum."""
    a = rms_norm(capped_sink_attention(h, w, f"{p}.left", c["left"]), w[f"{p}.left.out"], eps)
    b = rms_norm(selective_scan(h, w, f"{p}.right", c["right"]), w[f"{p}.right.out"], eps)
    return 0.5 * (a + b)


def lightning(h, w, p, c, eps):
    """Linear attention with one fixed decay per head behind silu on queries, keys and values; all heads' outputs
    normed together, times sigmoid of a gate."""
    T = h.shape[0]
    H, d, dv = c["heads"], c["dim"], c["vdim"]
    q, k, v = (silu(h @ w[f"{p}.{x}"].T).view(T, H, -1) for x in "qkv")
    decay = torch.tensor(c["decay"], dtype=F)
    S = torch.zeros(H, d, dv, dtype=F)
    o = torch.zeros(T, H, dv, dtype=F)
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    o = rms_norm(o.reshape(T, H * dv), w[f"{p}.norm"], eps)
    return (o * torch.sigmoid(h @ w[f"{p}.g"].T)) @ w[f"{p}.o"].T


# ----------------------------------------------------------------------------- the model


def feed_forward(h, w, p):
    return (torch.relu(h @ w[f"{p}.gate"].T) * (h @ w[f"{p}.up"].T)) @ w[f"{p}.down"].T


def embed(cfg, w, ids):
    ids = torch.as_tensor(ids)
    return w["embed"][ids] * cfg["embedding"]["scale"] + w["pos"][:len(ids)]


def layer_runs(cfg) -> list[tuple[int, bool]]:
    """(layer, whether it is the first of a pass of the loop) in the order in which they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    one = [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return [*((i, False) for i in range(loop["start"])), *(one * loop["times"]), *((i, False) for i in range(loop["stop"], n))]


def forward(w, cfg, ids, return_hidden=False):
    """Logits [T, vocab]; with ``return_hidden`` also the stream after every layer run."""
    eps = float(cfg["norm"]["eps"])
    x = start = embed(cfg, w, ids)
    hidden = []
    for i, enters in layer_runs(cfg):
        layer, p = cfg["layers"][i], f"l{i}"
        if enters:
            x = torch.cat([x, start], dim=1) @ w["loop.in"].T
        mixer = {"lightning": lightning, "parallel": parallel}[layer["type"]]
        x = x + mixer(rms_norm(x, w[f"{p}.norm1"], eps), w, f"{p}.mix", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            x = x + feed_forward(rms_norm(x, w[f"{p}.norm2"], eps), w, f"{p}.mlp")
        hidden.append(x)
    logits = rms_norm(x, w["final.norm"], eps) @ w["embed"].T * cfg["logit_scale"]
    return (logits, hidden) if return_hidden else logits
