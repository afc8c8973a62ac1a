"""Small Pinozen configurations for the tests, as ``config.json`` dictionaries. They differ from each other in every size
and constant: heads (one, one key/value head for all, one each), key and value heads of different sizes, more than the
tile kernel holds and multiples of nothing, convolutions of one to nine taps and none, states of one to seventy-two
elements, ranks of one and of no multiple of eight, rotations of whole heads, of parts and none, with frequencies in all
three ranges of wavelengths, caps and none, loops at the start, in the middle and around one layer, of one to three passes,
no loop, layers without a feed-forward, a width that is no multiple of four."""

from __future__ import annotations


def rotation(base, dims, scaling=None):
    out = {"base": base, "dims": dims}
    if scaling:
        out["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return out


def attention(heads, kv_heads, dim, vdim, scale, conv=0, softcap=0.0, rot=None):
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if conv:
        out["conv"] = conv
    if softcap:
        out["softcap"] = softcap
    if rot:
        out["rot"] = rot
    return out


def scan(inner, state, dt_rank, conv):
    return {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}


def layer(mixer, ff=0):
    return {"type": "parallel" if "left" in mixer else "lightning", "mixer": mixer,
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def parallel(left, right, ff=0):
    return layer({"left": left, "right": right}, ff)


def lightning(dim, vdim, decay, ff=0):
    return layer({"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}, ff)


def model(vocab, width, layers, eps=1e-5, embedding=1.5, logits=0.5, places=400, loop=None):
    out = {"architecture": "Pinozen", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps},
           "embedding": {"scale": embedding}, "logit_scale": logits, "max_positions": places}
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


#: all kinds of layers, the middle two twice
SMALL = model(97, 48, [
    parallel(attention(4, 2, 16, 12, 0.4, 4, 8.0, rotation(500.0, 12, (4.0, 1.0, 4.0, 64))), scan(40, 16, 5, 3), 56),
    lightning(12, 20, (0.5, 0.9, 0.99, 0.999), 40),
    parallel(attention(3, 1, 24, 16, 0.3, 2, 3.0, rotation(90.0, 24, (8.0, 2.0, 8.0, 32))), scan(64, 8, 8, 4)),
    parallel(attention(2, 2, 8, 20, 0.6, 3, 20.0, rotation(1e4, 4)), scan(32, 24, 3, 2), 33),
], loop=(1, 3, 2))

#: sizes of one wherever a size can be one: a head, a value, a tap, a channel, a state, a rank, a hidden unit, a pass
ONES = model(31, 20, [
    parallel(attention(1, 1, 2, 1, 1.1, 1, 1.0, rotation(7.0, 2, (2.0, 1.0, 1.0, 50))), scan(1, 1, 1, 1), 1),
    lightning(1, 1, (1.0,), 5),
    lightning(2, 3, (0.25,)),
], eps=1e-3, embedding=1.0, logits=1.0, loop=(0, 1, 1))

#: heads beyond the tile kernel's, convolutions of more taps than the four-element form takes, states past 32; the last
#: layer three times
WIDE = model(64, 64, [
    parallel(attention(6, 2, 160, 48, 0.08, 9, 12.0, rotation(2000.0, 64, (2.0, 0.5, 6.0, 128))), scan(136, 40, 20, 9), 72),
    lightning(72, 40, (0.7, 0.97, 0.995)),
    parallel(attention(8, 1, 32, 64, 0.2, 3, 30.0, rotation(1e5, 32)), scan(96, 64, 24, 4), 100),
], eps=1e-6, embedding=0.7, logits=2.0, loop=(2, 3, 3))

#: sizes that are multiples of nothing; no cap, no rotation and no convolution somewhere; the first layers twice, a pass
#: that begins and ends with layers without a feed-forward
ODD = model(53, 50, [
    lightning(7, 9, (0.3, 0.95, 0.8)),
    parallel(attention(6, 2, 10, 7, 0.4, 3, 0.0, rotation(11.0, 6, (3.0, 1.5, 2.5, 20))), scan(37, 13, 7, 5)),
    parallel(attention(5, 5, 14, 9, 0.25, 0, 5.0), scan(43, 3, 11, 2), 51),
], eps=1e-4, embedding=2.5, logits=0.3, loop=(0, 2, 2))

#: no loop; past several spans of keys; slow states
LONG = model(60, 32, [
    parallel(attention(2, 1, 16, 16, 0.3, 4, 10.0, rotation(1e4, 16, (4.0, 1.0, 4.0, 256))), scan(48, 72, 6, 4), 24),
    lightning(16, 16, (0.9999, 0.6, 1.0), 24),
    parallel(attention(4, 2, 8, 8, 0.5, 2, 6.0, rotation(300.0, 6)), scan(24, 12, 9, 3), 24),
], places=600)

ALL = {"small": SMALL, "ones": ONES, "wide": WIDE, "odd": ODD, "long": LONG}
