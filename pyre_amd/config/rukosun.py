"""Configuration of the Rukosun design, read from its own ``config.json`` layout.

``architecture`` names the design; ``vocab``, ``width``, ``norm.eps``, ``streams`` (of the residual) and ``max_positions``
(rows of the learned position table) are the model's, ``embedding.bigram`` the hash of the pair table; ``layers`` lists the
layers, each with its ``type`` (which mixer it has), the mixer's sizes and constants (``mixer``) and its feed-forward
(``mlp``, null for none); ``loop`` lets the layers ``start`` .. ``stop - 1`` run ``times`` times in a row. Every size and
constant that can differ between two models of the design is a field here; what a configuration does not mention is not
there (no ``mask``: plain causal attention; no ``loop``: every layer once).
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, ClassVar

from pyre_amd.config.mafurax import _get, _positive_int
from pyre_amd.config.model import ConfigError, ModelConfig


@dataclass(frozen=True)
class LatentConfig:
    """Attention over one compressed row of ``kv_rank`` elements and ``rot_dim`` turned ones per token; queries as they
    are projected."""

    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    window: int = 0              #: mask.size; 0: every earlier token is visible

    @classmethod
    def _fields(cls, raw, where) -> dict:
        dim, rot_dim = _positive_int(raw, "dim", where), _positive_int(raw, "rot_dim", where)
        rot = raw.get("rot")
        base = float(_get(rot, "base", f"{where}.rot"))
        if rot_dim % 2 or int(rot.get("dims", rot_dim)) != rot_dim or not base > 0:
            raise ConfigError(f"config.json: {where}.rot.dims must be rot_dim ({rot_dim}), an even number, and the base positive")
        window = int((raw.get("mask") or {}).get("size") or 0)
        if window < 0:
            raise ConfigError(f"config.json: {where}.mask.size must not be negative")
        return dict(heads=_positive_int(raw, "heads", where), dim=dim, rot_dim=rot_dim, vdim=_positive_int(raw, "vdim", where),
                    kv_rank=_positive_int(raw, "kv_rank", where), scale=float(_get(raw, "scale", where)), rot_base=base,
                    window=window)

    @classmethod
    def from_dict(cls, raw, where):
        return cls(**cls._fields(raw, where))

    def to_dict(self):
        out: dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank,
                               "rot": {"base": self.rot_base, "dims": self.rot_dim}, "rot_dim": self.rot_dim,
                               "scale": self.scale, "vdim": self.vdim}
        if self.window:
            out["mask"] = {"size": self.window}
        return out


@dataclass(frozen=True)
class CompressedQueryConfig(LatentConfig):
    """The same with queries made of a compressed row of ``q_rank`` elements (and a sink and an output gate)."""

    q_rank: int = 0

    @classmethod
    def from_dict(cls, raw, where):
        return cls(**cls._fields(raw, where), q_rank=_positive_int(raw, "q_rank", where))

    def to_dict(self):
        return dict(super().to_dict(), q_rank=self.q_rank)


@dataclass(frozen=True)
class DenseConfig:
    ff: int
    kind: ClassVar[str] = "dense"

    @classmethod
    def from_dict(cls, raw, where):
        return cls(_positive_int(raw, "ff", where))

    def to_dict(self):
        return {"ff": self.ff, "kind": self.kind}


MIXER_CONFIGS = {"latent_attention": CompressedQueryConfig, "latent_attention_2": LatentConfig}
FEED_FORWARD_CONFIGS = {"dense": DenseConfig}


@dataclass(frozen=True)
class RukosunLayerConfig:
    type: str
    mixer: Any
    mlp: Any = None

    @classmethod
    def from_dict(cls, raw, where):
        kind = raw.get("type") if isinstance(raw, dict) else None
        if kind not in MIXER_CONFIGS:
            raise ConfigError(f"config.json: {where}.type is {kind!r}; known: {sorted(MIXER_CONFIGS)}")
        if not isinstance(raw.get("mixer"), dict):
            raise ConfigError(f"config.json: {where} has no 'mixer'")
        mlp = raw.get("mlp")
        if mlp is not None:
            ff_kind = mlp.get("kind") if isinstance(mlp, dict) else None
            if ff_kind not in FEED_FORWARD_CONFIGS:
                raise ConfigError(f"config.json: {where}.mlp.kind is {ff_kind!r}; known: {sorted(FEED_FORWARD_CONFIGS)}")
            mlp = FEED_FORWARD_CONFIGS[ff_kind].from_dict(mlp, f"{where}.mlp")
        return cls(kind, MIXER_CONFIGS[kind].from_dict(raw["mixer"], f"{where}.mixer"), mlp)

    def to_dict(self):
        return {"mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict(), "type": self.type}


@dataclass(frozen=True)
class RukosunConfig(ModelConfig):
    architecture: ClassVar[str] = "Rukosun"

    vocab: int
    width: int
    layers: tuple
    norm_eps: float
    streams: int
    max_positions: int
    bigram_buckets: int
    bigram_mul_prev: int
    bigram_mul_cur: int
    loop: tuple | None = None    #: (start, stop, times): layers start .. stop - 1 run `times` times in a row

    def __post_init__(self) -> None:
        if not self.layers:
            raise ConfigError("there must be a layer")
        if not (self.norm_eps > 0):
            raise ConfigError(f"norm.eps must be positive, got {self.norm_eps!r}")
        if self.bigram_mul_prev < 0 or self.bigram_mul_cur < 0:
            raise ConfigError("embedding.bigram: the multipliers must not be negative")
        if self.loop is not None:
            start, stop, times = self.loop
            if not (0 <= start <= stop <= len(self.layers)) or times < 0:
                raise ConfigError(f"loop {self.loop} does not fit {len(self.layers)} layers")
            if not self.order():
                raise ConfigError("the loop leaves no layer to run")

    def order(self) -> list[int]:
        """The layers in the order in which they run, a looped one as often as it runs."""
        n = len(self.layers)
        if self.loop is None:
            return list(range(n))
        start, stop, times = self.loop
        return [*range(start), *(list(range(start, stop)) * times), *range(stop, n)]

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @classmethod
    def from_dict(cls, raw: dict[str, Any]) -> "RukosunConfig":
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json has no 'layers' list")
        pair = (raw.get("embedding") or {}).get("bigram") or {}
        where = "embedding.bigram"
        loop = raw.get("loop")
        if loop:
            loop = tuple(int(_get(loop, k, "loop")) for k in ("start", "stop", "times"))
        return cls(vocab=_positive_int(raw, "vocab", "config"), width=_positive_int(raw, "width", "config"),
                   layers=tuple(RukosunLayerConfig.from_dict(l, f"layers[{i}]") for i, l in enumerate(layers)),
                   norm_eps=float(_get(raw.get("norm"), "eps", "norm")), streams=_positive_int(raw, "streams", "config"),
                   max_positions=_positive_int(raw, "max_positions", "config"),
                   bigram_buckets=_positive_int(pair, "buckets", where), bigram_mul_prev=int(_get(pair, "mul_prev", where)),
                   bigram_mul_cur=int(_get(pair, "mul_cur", where)), loop=loop or None)

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"architecture": self.architecture,
                               "embedding": {"bigram": {"buckets": self.bigram_buckets, "mul_cur": self.bigram_mul_cur,
                                                        "mul_prev": self.bigram_mul_prev}},
                               "layers": [l.to_dict() for l in self.layers], "max_positions": self.max_positions,
                               "norm": {"eps": self.norm_eps}, "streams": self.streams, "vocab": self.vocab,
                               "width": self.width}
        if self.loop is not None:
            out["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        return out
