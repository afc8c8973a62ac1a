"""The Pinozen design as a list of parts.

Pre-norm layers with plain RMS norms, x += mixer(norm1(x)), x += ff(norm2(x)). The embedding is the token's row, scaled,
and the position's row of a learned table; the head is the token table, its logits scaled. A layer's mixer is one of two.
'parallel': two mixers side by side on the same rows, each with an output matrix of its own, each result normed over the
width with a gain of its own, half their sum handed on: causal grouped softmax attention (projections behind a short
convolution, part of a head turned in neighbouring pairs with frequencies changed by their wavelength, capped scores, a
sink in the denominator) and a selective scan (a float32 state per channel whose decay, input and output every token
chooses itself). 'lightning': linear attention with a fixed decay per head behind silu, all heads normed together, a sigmoid
gate. The feed-forward is down(relu(gate x) * (up x)), or absent. Some layers may run several times in a row with the same
weights, every pass with caches of its own and beginning with a product of the stream and the embedding's output. Tensor
names: ``embed``, ``pos``, ``loop.in``, ``final.norm``, ``l<i>.norm1 / norm2``, ``l<i>.mix.*`` (``.left.*``, ``.right.*``,
``.left.out / .right.out``), ``l<i>.mlp.*``.
"""

from __future__ import annotations

from pyre_amd.config.pinozen import AttentionConfig, DenseConfig, LightningConfig, ParallelConfig, PinozenConfig
from pyre_amd.parts.base import (BlockSpec, EmbeddingSpec, LayerCall, LightningAttentionSpec, LMHeadSpec, ModelSpec,
                                 NoPositionSpec, ParallelMixerSpec, PassInputSpec, ReluGLUSpec, RMSNormSpec, RotarySpec,
                                 SelectiveScanSpec, SinkAttentionSpec)
from pyre_amd.registry import register_architecture

#: the two branches' normed results are averaged
BRANCH_SCALE = 0.5


def _position(a: AttentionConfig):
    r = a.rot
    if r is None:
        return NoPositionSpec()
    return RotarySpec(a.dim, r.base, 0, rotary_dim=r.dims, exact=True, pairing="neighbours", wave_scaling=r.scaling)


def _parallel(cfg: PinozenConfig, m: ParallelConfig, prefix: str) -> ParallelMixerSpec:
    a, r = m.left, m.right
    left = SinkAttentionSpec(cfg.width, a.heads, a.kv_heads, a.dim, a.vdim, a.scale, _position(a), f"{prefix}.left",
                             conv_taps=a.conv, qk_norm=False, sink=True, gated=False, softcap=a.softcap)
    right = SelectiveScanSpec(cfg.width, r.inner, r.state, r.dt_rank, r.conv, f"{prefix}.right")
    return ParallelMixerSpec(cfg.width, (left, right), (BRANCH_SCALE, BRANCH_SCALE),
                             out_norms=(f"{prefix}.left.out", f"{prefix}.right.out"), norm_eps=cfg.norm_eps)


def _lightning(cfg: PinozenConfig, m: LightningConfig, prefix: str) -> LightningAttentionSpec:
    return LightningAttentionSpec(cfg.width, m.heads, m.dim, m.vdim, m.decay, prefix, norm_eps=cfg.norm_eps)


MIXERS = {ParallelConfig: _parallel, LightningConfig: _lightning}


def _dense(cfg: PinozenConfig, f: DenseConfig, prefix: str) -> ReluGLUSpec:
    return ReluGLUSpec(cfg.width, f.ff, prefix)


FEED_FORWARDS = {DenseConfig: _dense}


def build_pinozen(cfg: PinozenConfig) -> ModelSpec:
    def norm(name):
        return RMSNormSpec(cfg.width, cfg.norm_eps, "", name=name)

    layers = []
    for i, layer in enumerate(cfg.layers):
        p, ff, ff_norm = f"l{i}", None, None
        if layer.mlp is not None:
            ff, ff_norm = FEED_FORWARDS[type(layer.mlp)](cfg, layer.mlp, f"{p}.mlp"), norm(f"{p}.norm2")
        layers.append(BlockSpec(mixer=MIXERS[type(layer.mixer)](cfg, layer.mixer, f"{p}.mix"), mixer_norm=norm(f"{p}.norm1"),
                                feed_forward=ff, feed_forward_norm=ff_norm))
    embedding = EmbeddingSpec(cfg.vocab, cfg.width, name="embed", scale=cfg.embedding_scale, places=cfg.max_positions,
                              places_name="pos")
    return ModelSpec(hidden_size=cfg.width, vocab_size=cfg.vocab, max_positions=cfg.max_positions, embedding=embedding,
                     layers=tuple(layers), schedule=tuple(LayerCall(i, enters=enters) for i, enters in cfg.runs()),
                     final_norm=norm("final.norm"), head=LMHeadSpec(cfg.vocab, cfg.width, name=embedding.name,
                                                                    scale=cfg.logit_scale),
                     pass_input=PassInputSpec(cfg.width, "loop.in") if cfg.loop is not None else None)


register_architecture(PinozenConfig.architecture, PinozenConfig, build_pinozen)
