"""Small Rukosun configurations for the tests, as ``config.json`` dictionaries. They differ from each other in every size
and constant: heads (one; more than a row tile of the kernels has), unturned, turned and value sizes that are multiples of
nothing and differ from each other, compressed rows for every form of the attention kernels (up to 128, 256 and beyond,
whole units of sixteen bytes and not), windows of one token, shorter than a page, past several spans of keys, and none,
one to six streams, loops at the start, in the middle and around one layer, no loop, layers without a feed-forward, pair
tables of one bucket, a width that is no multiple of four."""

from __future__ import annotations


def mixer(heads, dim, rot_dim, vdim, rank, scale, window=0, base=10000.0, q_rank=0):
    out = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "scale": scale,
           "rot": {"base": base, "dims": rot_dim}}
    if window:
        out["mask"] = {"size": window}
    if q_rank:
        out["q_rank"] = q_rank
    return out


def layer(m, ff=0):
    """A layer of the first kind if its mixer has compressed queries, else of the second."""
    return {"type": "latent_attention" if "q_rank" in m else "latent_attention_2", "mixer": m,
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model(vocab, width, layers, streams, eps=1e-5, buckets=101, mul_prev=7, mul_cur=5, places=400, loop=None):
    out = {"architecture": "Rukosun", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps},
           "streams": streams, "max_positions": places,
           "embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}}
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


#: four layers of both kinds, every window there is, the middle two of them twice; three streams
SMALL = model(97, 48, [
    layer(mixer(4, 12, 8, 10, 24, 0.3, window=20, base=500.0, q_rank=20), 56),
    layer(mixer(3, 16, 16, 24, 40, 0.25, window=27, base=3000.0), 40),
    layer(mixer(2, 8, 4, 12, 32, 0.5, window=9, base=90.0, q_rank=16)),
    layer(mixer(4, 20, 12, 6, 16, 0.2, base=1e4), 33),
], streams=3, loop=(1, 3, 2))

#: sizes of one wherever a size can be one: a head, an unturned element, a value, a compressed row, a hidden unit, a
#: bucket, a stream, a window, a pass
ONES = model(31, 20, [
    layer(mixer(1, 1, 2, 1, 1, 1.1, window=1, base=7.0, q_rank=1), 1),
    layer(mixer(1, 2, 2, 3, 4, 0.9, window=1, base=3.0), 5),
], streams=1, eps=1e-3, buckets=1, mul_prev=3, mul_cur=0, loop=(0, 1, 1))

#: rows of more than 128 and more than 256 elements, more than 32 heads, a turned part larger than the unturned one; the
#: last layer three times
WIDE = model(64, 64, [
    layer(mixer(5, 24, 32, 16, 200, 0.2, window=18, base=2000.0, q_rank=40), 72),
    layer(mixer(37, 4, 8, 4, 136, 0.4, window=33, base=700.0)),
    layer(mixer(2, 40, 64, 48, 320, 0.15, window=40, base=1e5, q_rank=72), 100),
], streams=4, eps=1e-6, buckets=1009, mul_prev=1000003, mul_cur=31, loop=(2, 3, 3))

#: sizes that are multiples of nothing, in rows of every form; the first layer twice; two streams
ODD = model(53, 50, [
    layer(mixer(3, 10, 6, 14, 21, 0.4, window=9, base=100.0), 37),
    layer(mixer(5, 7, 10, 5, 131, 0.25, window=30, base=11.0, q_rank=9), 51),
    layer(mixer(2, 5, 14, 9, 259, 0.2, base=50.0, q_rank=27)),
], streams=2, eps=1e-4, buckets=17, mul_prev=0, mul_cur=1, loop=(0, 1, 2))

#: no loop; windows past one span of keys and past several, and none; six streams
LONG = model(60, 32, [
    layer(mixer(2, 8, 8, 8, 16, 0.3, window=270, base=1e4, q_rank=12), 24),
    layer(mixer(3, 8, 4, 8, 24, 0.4, base=100.0), 24),
    layer(mixer(2, 12, 4, 8, 136, 0.3, window=300, base=900.0)),
], streams=6, places=500)
