"""The Rukosun design as a list of parts.

The embedding is the sum of three rows: the token's, that of the pair (previous token, token) and the position's. The
residual is several streams, all equal at first, and every sublayer stands between them (hyper-connections): it reads one
mixture of the streams through a layer norm with a bias and hands its result back to all of them; the final norm reads
their sum. A layer's mixer is attention over one compressed row per token with a turned key part that all heads share, over
a window, in one of two kinds: 'latent_attention' makes its queries of a compressed row of their own, turns neighbouring
pairs, has a sink in the softmax and a sigmoid gate per output element; 'latent_attention_2' projects its queries plainly
and turns element e with e + dims/2. The feed-forward is a polynomial of normed powers between two matrices, or absent. Some
layers may run several times in a row with the same weights, every pass with a cache of its own. Tensor names: ``embed``,
``bigram``, ``pos``, ``final.norm``, ``head``, ``l<i>.norm1 / norm2`` (biases ``.b``), ``l<i>.mix.*``, ``l<i>.mlp.*``,
``l<i>.hc1.* / hc2.*``.
"""

from __future__ import annotations

from pyre_amd.config.rukosun import CompressedQueryConfig, DenseConfig, LatentConfig, RukosunConfig
from pyre_amd.parts.base import (BigramEmbeddingSpec, HyperConnectionBlockSpec, HyperConnectionSpec, LatentAttentionSpec,
                                 LayerCall, LayerNormSpec, LMHeadSpec, ModelSpec, PolyNormMLPSpec, RotarySpec)
from pyre_amd.registry import register_architecture


def _rows(cfg: RukosunConfig, m: LatentConfig, prefix: str, pairing: str, **options) -> LatentAttentionSpec:
    return LatentAttentionSpec(cfg.width, m.heads, m.dim, m.vdim, m.kv_rank, m.scale, cfg.norm_eps, prefix, rot_dim=m.rot_dim,
                               position=RotarySpec(m.rot_dim, m.rot_base, 0, exact=True, pairing=pairing), window=m.window,
                               **options)


def _compressed_queries(cfg: RukosunConfig, m: CompressedQueryConfig, prefix: str) -> LatentAttentionSpec:
    return _rows(cfg, m, prefix, "neighbours", q_rank=m.q_rank, sink=True, gated=True)


def _plain_queries(cfg: RukosunConfig, m: LatentConfig, prefix: str) -> LatentAttentionSpec:
    return _rows(cfg, m, prefix, "halves")


MIXERS = {CompressedQueryConfig: _compressed_queries, LatentConfig: _plain_queries}


def _dense(cfg: RukosunConfig, f: DenseConfig, prefix: str) -> PolyNormMLPSpec:
    return PolyNormMLPSpec(cfg.width, f.ff, prefix, cfg.norm_eps)


FEED_FORWARDS = {DenseConfig: _dense}


def build_rukosun(cfg: RukosunConfig) -> ModelSpec:
    def norm(name):
        return LayerNormSpec(cfg.width, cfg.norm_eps, name, bias=True)

    layers = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}"
        s = cfg.streams
        # a layer without a feed-forward may still have that sublayer's norm and connection in its file
        ff = dict(unused=((f"{p}.norm2", (cfg.width,)), (f"{p}.norm2.b", (cfg.width,)), (f"{p}.hc2.in", (s,)),
                          (f"{p}.hc2.out", (s,)), (f"{p}.hc2.mix", (s, s))))
        if layer.mlp is not None:
            ff = dict(feed_forward=FEED_FORWARDS[type(layer.mlp)](cfg, layer.mlp, f"{p}.mlp"), feed_forward_norm=norm(f"{p}.norm2"),
                      feed_forward_connection=HyperConnectionSpec(cfg.streams, f"{p}.hc2"))
        layers.append(HyperConnectionBlockSpec(mixer=MIXERS[type(layer.mixer)](cfg, layer.mixer, f"{p}.mix"),
                                               mixer_norm=norm(f"{p}.norm1"),
                                               mixer_connection=HyperConnectionSpec(cfg.streams, f"{p}.hc1"), **ff))
    embedding = BigramEmbeddingSpec(cfg.vocab, cfg.width, cfg.bigram_buckets, cfg.bigram_mul_prev, cfg.bigram_mul_cur,
                                    places=cfg.max_positions, places_name="pos")
    return ModelSpec(hidden_size=cfg.width, vocab_size=cfg.vocab, max_positions=cfg.max_positions, embedding=embedding,
                     layers=tuple(layers), schedule=tuple(LayerCall(i) for i in cfg.order()), final_norm=norm("final.norm"),
                     head=LMHeadSpec(cfg.vocab, cfg.width, name="head"), streams=cfg.streams)


register_architecture(RukosunConfig.architecture, RukosunConfig, build_rukosun)
