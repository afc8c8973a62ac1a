"""Configuration of the Pinozen design, read from its own ``config.json`` layout.

``architecture`` names the design; ``vocab``, ``width``, ``norm.eps``, ``logit_scale`` and ``max_positions`` (rows of the
learned position table) are the model's, ``embedding.scale`` the factor on the token table's rows; ``layers`` lists the
layers, each with its ``type`` (which mixer it has), the mixer's sizes and constants (``mixer``) and its feed-forward
(``mlp``, null for none); ``loop`` lets the layers ``start`` .. ``stop - 1`` run ``times`` times in a row, every pass
beginning with a product of the residual stream and the embedding's output. Every size and constant that can differ between
two models of the design is a field here; what a configuration does not mention is not there (no ``rot``: no rotation; no
``rot.scaling``: plain frequencies; no ``softcap``: scores as they are; no ``loop``: every layer once).
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, ClassVar

from pyre_amd.config.mafurax import _get, _positive_int
from pyre_amd.config.model import ConfigError, ModelConfig


@dataclass(frozen=True)
class RotConfig:
    """Rotation of the first ``dims`` elements of a head in neighbouring pairs; ``scaling`` = (factor, low, high, original)
    changes the frequencies by their wavelength, or None."""

    base: float
    dims: int
    scaling: tuple | None = None

    @classmethod
    def from_dict(cls, raw, dim: int, where: str):
        if not raw:
            return None
        base, dims = float(_get(raw, "base", where)), _positive_int(raw, "dims", where)
        if dims % 2 or dims > dim or not base > 0:
            raise ConfigError(f"config.json: {where}.dims ({dims}) must be even and within dim ({dim}), the base positive")
        scaling = None
        if raw.get("scaling"):
            w = f"{where}.scaling"
            scaling = tuple(float(_get(raw["scaling"], k, w)) for k in ("factor", "low", "high", "original"))
            factor, low, high, original = scaling
            if not all(x > 0 for x in scaling) or low > high:
                raise ConfigError(f"config.json: {w}: factor, low, high and original must be positive, low not above high")
        return cls(base, dims, scaling)

    def to_dict(self):
        out: dict[str, Any] = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            out["scaling"] = dict(zip(("factor", "low", "high", "original"), self.scaling))
        return out


@dataclass(frozen=True)
class AttentionConfig:
    """The softmax branch ('left') of a 'parallel' layer: causal grouped attention with a sink, its projections behind a
    convolution of ``conv`` taps (0: none), scores capped at ``softcap`` (0: not)."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    conv: int = 0
    softcap: float = 0.0
    rot: RotConfig | None = None

    @classmethod
    def from_dict(cls, raw, where):
        heads, kv = _positive_int(raw, "heads", where), _positive_int(raw, "kv_heads", where)
        if heads % kv:
            raise ConfigError(f"config.json: {where}.heads ({heads}) is not a multiple of kv_heads ({kv})")
        dim = _positive_int(raw, "dim", where)
        softcap = float(raw.get("softcap") or 0.0)
        if softcap < 0:
            raise ConfigError(f"config.json: {where}.softcap must not be negative")
        return cls(heads, kv, dim, _positive_int(raw, "vdim", where), float(_get(raw, "scale", where)),
                   _positive_int(raw, "conv", where) if raw.get("conv") else 0, softcap,
                   RotConfig.from_dict(raw.get("rot"), dim, f"{where}.rot"))

    def to_dict(self):
        out: dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale,
                               "vdim": self.vdim}
        if self.conv:
            out["conv"] = self.conv
        if self.softcap:
            out["softcap"] = self.softcap
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass(frozen=True)
class ScanConfig:
    """The recurrent branch ('right') of a 'parallel' layer: a selective scan over ``inner`` channels with a state of
    ``state`` each, step sizes of rank ``dt_rank``, a convolution of ``conv`` taps."""

    inner: int
    state: int
    dt_rank: int
    conv: int

    @classmethod
    def from_dict(cls, raw, where):
        return cls(*(_positive_int(raw, k, where) for k in ("inner", "state", "dt_rank", "conv")))

    def to_dict(self):
        return {"conv": self.conv, "dt_rank": self.dt_rank, "inner": self.inner, "state": self.state}


@dataclass(frozen=True)
class ParallelConfig:
    left: AttentionConfig
    right: ScanConfig

    @classmethod
    def from_dict(cls, raw, where):
        for k in ("left", "right"):
            if not isinstance(raw.get(k), dict):
                raise ConfigError(f"config.json: {where} has no {k!r}")
        return cls(AttentionConfig.from_dict(raw["left"], f"{where}.left"), ScanConfig.from_dict(raw["right"], f"{where}.right"))

    def to_dict(self):
        return {"left": self.left.to_dict(), "right": self.right.to_dict()}


@dataclass(frozen=True)
class LightningConfig:
    """Linear attention with one fixed decay per head."""

    heads: int
    dim: int
    vdim: int
    decay: tuple

    @classmethod
    def from_dict(cls, raw, where):
        heads = _positive_int(raw, "heads", where)
        decay = raw.get("decay")
        if not isinstance(decay, list) or len(decay) != heads:
            raise ConfigError(f"config.json: {where}.decay must list one number for each of {heads} heads")
        if not all(isinstance(d, (int, float)) and not isinstance(d, bool) and 0.0 < float(d) <= 1.0 for d in decay):
            raise ConfigError(f"config.json: {where}.decay must hold numbers in (0, 1]")
        return cls(heads, _positive_int(raw, "dim", where), _positive_int(raw, "vdim", where), tuple(float(d) for d in decay))

    def to_dict(self):
        return {"decay": list(self.decay), "dim": self.dim, "heads": self.heads, "vdim": self.vdim}


@dataclass(frozen=True)
class DenseConfig:
    ff: int
    kind: ClassVar[str] = "dense"

    @classmethod
    def from_dict(cls, raw, where):
        return cls(_positive_int(raw, "ff", where))

    def to_dict(self):
        return {"ff": self.ff, "kind": self.kind}


MIXER_CONFIGS = {"lightning": LightningConfig, "parallel": ParallelConfig}
FEED_FORWARD_CONFIGS = {"dense": DenseConfig}


@dataclass(frozen=True)
class PinozenLayerConfig:
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
class PinozenConfig(ModelConfig):
    architecture: ClassVar[str] = "Pinozen"

    vocab: int
    width: int
    layers: tuple
    norm_eps: float
    max_positions: int
    embedding_scale: float = 1.0
    logit_scale: float = 1.0
    loop: tuple | None = None    #: (start, stop, times): layers start .. stop - 1 run `times` times in a row

    def __post_init__(self) -> None:
        if not self.layers:
            raise ConfigError("there must be a layer")
        if not (self.norm_eps > 0):
            raise ConfigError(f"norm.eps must be positive, got {self.norm_eps!r}")
        if self.loop is not None:
            start, stop, times = self.loop
            if not (0 <= start < stop <= len(self.layers)) or times <= 0:
                raise ConfigError(f"loop {self.loop} does not fit {len(self.layers)} layers")

    def runs(self) -> list[tuple[int, bool]]:
        """(layer, whether a pass of the loop begins with it) in the order in which the layers run."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, False) for i in range(n)]
        start, stop, times = self.loop
        one_pass = [(i, i == start) for i in range(start, stop)]
        return [*((i, False) for i in range(start)), *(one_pass * times), *((i, False) for i in range(stop, n))]

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @classmethod
    def from_dict(cls, raw: dict[str, Any]) -> "PinozenConfig":
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json has no 'layers' list")
        emb, loop = raw.get("embedding") or {}, raw.get("loop")
        if loop:
            loop = tuple(_get(loop, k, "loop", int) for k in ("start", "stop", "times"))
        return cls(vocab=_positive_int(raw, "vocab", "config"), width=_positive_int(raw, "width", "config"),
                   layers=tuple(PinozenLayerConfig.from_dict(l, f"layers[{i}]") for i, l in enumerate(layers)),
                   norm_eps=float(_get(raw.get("norm"), "eps", "norm")),
                   max_positions=_positive_int(raw, "max_positions", "config"),
                   embedding_scale=float(_get(emb, "scale", "embedding")) if "scale" in emb else 1.0,
                   logit_scale=float(_get(raw, "logit_scale", "config")) if "logit_scale" in raw else 1.0,
                   loop=loop or None)

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale},
                               "layers": [l.to_dict() for l in self.layers], "logit_scale": self.logit_scale,
                               "max_positions": self.max_positions, "norm": {"eps": self.norm_eps}, "vocab": self.vocab,
                               "width": self.width}
        if self.loop is not None:
            out["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        return out
