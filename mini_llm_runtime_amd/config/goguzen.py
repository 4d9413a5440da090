"""The Goguzen decoder's configuration.

Its config.json is nested and lists the layers one by one; a layer may use an earlier listed layer's tensors:

    {"architecture": "Goguzen", "vocab": V, "width": W, "norm": {"eps": e}, "embedding": {"scale": s},
     "layers": [{"type": "attention",
                 "mixer": {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": c,
                           "mask": {"size": w, "keep_first": n},
                           "rot": {"base": b, "dims": r,
                                   "scaling": {"factor": f, "low": l, "high": h, "original": n}}},
                 "mlp": {"kind": "moe", "router": {"experts": E, "top": k},
                         "expert": {"ff": F, "limit": x}, "shared": {"ff": F2, "limit": x2}}},
                {"type": "parallel",
                 "mixer": {"left": {"heads": H, "kv_heads": G, "dim": d, "vdim": d, "scale": c,
                                    "q_temp": {"every": n, "coef": a}},
                           "right": {"heads": H, "vdim": P, "state": N, "groups": G, "conv": taps,
                                     "norm_groups": M}},
                 "mlp": null, "weights_of": j}, ...],
     "logit_scale": x, "logit_softcap": c}

`weights_of` (optional) names the layer whose tensors this one uses; the two entries are equal otherwise.  `mask`, `rot`,
`rot.scaling`, `q_temp`, `mlp`, `mlp.shared`, `logit_scale` and `logit_softcap` may be absent.  Nothing here is a size of
one particular model.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, ClassVar, Mapping, Optional

from .bubitar import _mapping
from .model_config import ConfigError, ModelConfig, positive_float, positive_int, require_keys
from .rofetar import RofetarMamba2


def _number(data: Mapping[str, Any], key: str, where: str) -> float:
    value = data.get(key)
    if isinstance(value, bool) or not isinstance(value, (int, float)):
        raise ConfigError(f"{where}: {key!r} must be a number, found {value!r}")
    return float(value)


def _count(data: Mapping[str, Any], key: str, where: str) -> int:
    value = data.get(key)
    if isinstance(value, bool) or not isinstance(value, int) or value < 0:
        raise ConfigError(f"{where}: {key!r} must be an integer >= 0, found {value!r}")
    return int(value)


@dataclass(frozen=True)
class BandScaling:
    """Frequencies divided by `factor` where a turn is longer than `original` / `low` positions, kept where it is
    shorter than `original` / `high`, blended between."""

    factor: float
    low: float
    high: float
    original: float

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "BandScaling":
        keys = ("factor", "low", "high", "original")
        require_keys(data, keys, where)
        out = cls(**{k: positive_float(data, k) for k in keys})
        if out.high < out.low:
            raise ConfigError(f"{where}: 'high' must be at least 'low'")
        return out

    def to_dict(self) -> dict[str, Any]:
        return {"factor": self.factor, "low": self.low, "high": self.high, "original": self.original}


@dataclass(frozen=True)
class GoguzenRotary:
    base: float
    dims: int
    scaling: Optional[BandScaling] = None

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "GoguzenRotary":
        require_keys(data, ("base", "dims"), where)
        scaling = data.get("scaling")
        out = cls(
            base=positive_float(data, "base"),
            dims=_count(data, "dims", where),
            scaling=None if scaling is None else BandScaling.from_dict(_mapping(data, "scaling", where), where + ".scaling"),
        )
        if out.dims % 2:
            raise ConfigError(f"{where}: dims must be even (0: nothing turns)")
        return out

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            out["scaling"] = self.scaling.to_dict()
        return out


def _heads(data: Mapping[str, Any], where: str) -> dict[str, Any]:
    """The sizes that both kinds of attention have."""
    require_keys(data, ("heads", "dim", "scale"), where)
    heads, dim = positive_int(data, "heads"), positive_int(data, "dim")
    out = {
        "heads": heads,
        "kv_heads": heads if data.get("kv_heads") is None else positive_int(data, "kv_heads"),
        "dim": dim,
        "vdim": dim if data.get("vdim") is None else positive_int(data, "vdim"),
        "scale": positive_float(data, "scale"),
    }
    if heads % out["kv_heads"]:
        raise ConfigError(f"{where}: {heads} heads are no multiple of {out['kv_heads']} kv_heads")
    return out


@dataclass(frozen=True)
class GoguzenAttention:
    """Rotated queries and keys normed over their whole projection; a window of tokens and the first ones."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None  # None: every earlier position is seen
    keep_first: int = 0
    rot: Optional[GoguzenRotary] = None

    kind: ClassVar[str] = "attention"

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "GoguzenAttention":
        sizes = _heads(data, where)
        window, keep = None, 0
        if data.get("mask") is not None:
            mask = _mapping(data, "mask", where)
            require_keys(mask, ("size",), where + ".mask")
            window = positive_int(mask, "size")
            keep = 0 if mask.get("keep_first") is None else _count(mask, "keep_first", where + ".mask")
        rot = None
        if data.get("rot") is not None:
            rot = GoguzenRotary.from_dict(_mapping(data, "rot", where), where + ".rot")
            if rot.dims > sizes["dim"]:
                raise ConfigError(f"{where}: more rotated dimensions than a head has")
        return cls(**sizes, window=window, keep_first=keep, rot=rot)

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
        }
        if self.window is not None:
            out["mask"] = {"size": self.window, "keep_first": self.keep_first}
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass(frozen=True)
class GoguzenLeft:
    """The softmax half of a parallel mixer: the keys before their norm are the values, so both have one size."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    temp_every: Optional[float] = None  # None: queries keep their size
    temp_coef: float = 0.0

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "GoguzenLeft":
        sizes = _heads(data, where)
        if sizes["vdim"] != sizes["dim"]:
            raise ConfigError(f"{where}: values that are keys have the keys' size, found dim {sizes['dim']}, vdim {sizes['vdim']}")
        every, coef = None, 0.0
        if data.get("q_temp") is not None:
            temp = _mapping(data, "q_temp", where)
            require_keys(temp, ("every", "coef"), where + ".q_temp")
            every, coef = positive_float(temp, "every"), _number(temp, "coef", where + ".q_temp")
        return cls(**sizes, temp_every=every, temp_coef=coef)

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
        }
        if self.temp_every is not None:
            out["q_temp"] = {"every": self.temp_every, "coef": self.temp_coef}
        return out


@dataclass(frozen=True)
class GoguzenParallel:
    left: GoguzenLeft
    right: RofetarMamba2  # the same state-space mixer

    kind: ClassVar[str] = "parallel"

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "GoguzenParallel":
        return cls(
            left=GoguzenLeft.from_dict(_mapping(data, "left", where), where + ".left"),
            right=RofetarMamba2.from_dict(_mapping(data, "right", where), where + ".right"),
        )

    def to_dict(self) -> dict[str, Any]:
        return {"left": self.left.to_dict(), "right": self.right.to_dict()}


_MIXERS = {c.kind: c for c in (GoguzenAttention, GoguzenParallel)}


@dataclass(frozen=True)
class ClampedExpert:
    """down(g sigmoid(1.702 g) (u + 1)) with g = min(gate(x), limit), u = clamp(up(x), -limit, limit), no biases."""

    ff: int
    limit: float

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "ClampedExpert":
        require_keys(data, ("ff", "limit"), where)
        return cls(ff=positive_int(data, "ff"), limit=positive_float(data, "limit"))

    def to_dict(self) -> dict[str, Any]:
        return {"ff": self.ff, "limit": self.limit}


@dataclass(frozen=True)
class GoguzenMixture:
    experts: int
    top: int
    expert: ClampedExpert
    shared: Optional[ClampedExpert] = None

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "GoguzenMixture":
        require_keys(data, ("kind", "router", "expert"), where)
        if data["kind"] != "moe":
            raise ConfigError(f"{where}: kind must be 'moe', found {data['kind']!r}")
        router = _mapping(data, "router", where)
        require_keys(router, ("experts", "top"), where + ".router")
        out = cls(
            experts=positive_int(router, "experts"),
            top=positive_int(router, "top"),
            expert=ClampedExpert.from_dict(_mapping(data, "expert", where), where + ".expert"),
            shared=None if data.get("shared") is None else ClampedExpert.from_dict(_mapping(data, "shared", where), where + ".shared"),
        )
        if out.top > out.experts:
            raise ConfigError(f"{where}: a token cannot use {out.top} of {out.experts} experts")
        return out

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "kind": "moe", "router": {"experts": self.experts, "top": self.top}, "expert": self.expert.to_dict(),
        }
        if self.shared is not None:
            out["shared"] = self.shared.to_dict()
        return out


@dataclass(frozen=True)
class GoguzenLayer:
    mixer: Any  # GoguzenAttention or GoguzenParallel
    mlp: Optional[GoguzenMixture]
    weights_of: Optional[int] = None

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "type": self.mixer.kind, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict(),
        }
        if self.weights_of is not None:
            out["weights_of"] = self.weights_of
        return out


@dataclass(frozen=True)
class GoguzenConfig(ModelConfig):
    architecture: ClassVar[str] = "Goguzen"
    model_type: ClassVar[str] = "goguzen"

    vocab: int
    width: int
    norm_eps: float
    layers: tuple[GoguzenLayer, ...]
    embedding_scale: float = 1.0
    logit_scale: float = 1.0
    logit_softcap: Optional[float] = None

    def __post_init__(self) -> None:
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError("GoguzenConfig: vocab and width must be > 0")
        if not self.layers:
            raise ConfigError("GoguzenConfig: a model needs at least one layer")
        if not self.norm_eps >= 0:
            raise ConfigError("GoguzenConfig: norm.eps must be >= 0")
        for i, layer in enumerate(self.layers):
            if layer.weights_of is None:
                continue
            owner = self.layers[self.owner_of(i)]
            if (owner.mixer, owner.mlp) != (layer.mixer, layer.mlp):
                raise ConfigError(f"layers[{i}]: a layer with weights_of equals the layer whose tensors it uses")

    def owner_of(self, index: int) -> int:
        """The layer whose tensors layer `index` uses (itself, unless `weights_of` names another)."""
        at, seen = index, set()
        while self.layers[at].weights_of is not None:
            seen.add(at)
            at = self.layers[at].weights_of
            if at in seen or not 0 <= at < len(self.layers):
                raise ConfigError(f"layers[{index}]: weights_of must lead to a layer that has tensors of its own")
        return at

    @classmethod
    def from_dict(cls, data: Mapping[str, Any]) -> "GoguzenConfig":
        where = "GoguzenConfig"
        require_keys(data, ("vocab", "width", "norm", "layers"), where)
        norm = _mapping(data, "norm", where)
        require_keys(norm, ("eps",), where + ".norm")
        eps = _number(norm, "eps", where + ".norm")
        scale = 1.0
        if data.get("embedding") is not None:
            embedding = _mapping(data, "embedding", where)
            if embedding.get("scale") is not None:
                scale = _number(embedding, "scale", where + ".embedding")
        listed = data["layers"]
        if not isinstance(listed, (list, tuple)):
            raise ConfigError(f"{where}: 'layers' must be a list")
        layers = []
        for i, entry in enumerate(listed):
            at = f"layers[{i}]"
            if not isinstance(entry, Mapping):
                raise ConfigError(f"{at} must be an object")
            require_keys(entry, ("type", "mixer"), at)
            if entry["type"] not in _MIXERS:
                raise ConfigError(f"{at}: unknown mixer type {entry['type']!r}; known: {', '.join(sorted(_MIXERS))}")
            mixer = _MIXERS[entry["type"]].from_dict(_mapping(entry, "mixer", at), at + ".mixer")
            mlp = entry.get("mlp")
            if mlp is not None and not isinstance(mlp, Mapping):
                raise ConfigError(f"{at}: 'mlp' must be an object or null")
            layers.append(
                GoguzenLayer(
                    mixer,
                    None if mlp is None else GoguzenMixture.from_dict(mlp, at + ".mlp"),
                    None if entry.get("weights_of") is None else _count(entry, "weights_of", at),
                )
            )
        return cls(
            vocab=positive_int(data, "vocab"),
            width=positive_int(data, "width"),
            norm_eps=eps,
            layers=tuple(layers),
            embedding_scale=scale,
            logit_scale=1.0 if data.get("logit_scale") is None else _number(data, "logit_scale", where),
            logit_softcap=None if data.get("logit_softcap") is None else positive_float(data, "logit_softcap"),
        )

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "architecture": self.architecture,
            "vocab": self.vocab,
            "width": self.width,
            "norm": {"eps": self.norm_eps},
            "embedding": {"scale": self.embedding_scale},
            "layers": [layer.to_dict() for layer in self.layers],
            "logit_scale": self.logit_scale,
        }
        if self.logit_softcap is not None:
            out["logit_softcap"] = self.logit_softcap
        return out
