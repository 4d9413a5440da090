"""The Rofetar decoder's configuration.

Its config.json is nested and lists the layers one by one, each with a mixer of its own kind and sizes and a
dense gated feed-forward or none:

    {"architecture": "Rofetar", "vocab": V, "width": W, "norm": {"eps": e},
     "layers": [{"type": "attention",
                 "mixer": {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": c, "softcap": s,
                           "rot": {"base": b, "dims": r,
                                   "scaling": {"factor": f, "original": n, "fast": a, "slow": z}},
                           "kv_from": j},
                 "mlp": {"kind": "dense", "ff": F}},
                {"type": "mamba2",
                 "mixer": {"heads": H, "vdim": P, "state": N, "groups": G, "conv": taps, "norm_groups": M},
                 "mlp": null},
                {"type": "delta",
                 "mixer": {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "conv": taps}, "mlp": null}, ...]}

`kv_from` (optional) names an earlier attention layer whose cached keys and values this layer reads instead of
making its own; `softcap`, `rot` and `rot.scaling` may be absent.  Nothing here is a size of one particular model.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, ClassVar, Mapping, Optional

from .bubitar import Rotary, _mapping
from .model_config import ConfigError, ModelConfig, positive_float, positive_int, require_keys


@dataclass(frozen=True)
class RofetarAttention:
    """Grouped heads, queries and keys normed per head and rotated, capped scores, one more in the denominator."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[Rotary] = None
    softcap: Optional[float] = None
    kv_from: Optional[int] = None

    kind: ClassVar[str] = "attention"

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "RofetarAttention":
        require_keys(data, ("heads", "dim", "vdim", "scale"), where)
        source = data.get("kv_from")
        if source is not None and (isinstance(source, bool) or not isinstance(source, int) or source < 0):
            raise ConfigError(f"{where}: 'kv_from' must be a layer index or absent")
        heads = positive_int(data, "heads")
        out = cls(
            heads=heads,
            kv_heads=heads if data.get("kv_heads") is None else positive_int(data, "kv_heads"),
            dim=positive_int(data, "dim"),
            vdim=positive_int(data, "vdim"),
            scale=positive_float(data, "scale"),
            rot=None if data.get("rot") is None else Rotary.from_dict(_mapping(data, "rot", where), where + ".rot"),
            softcap=None if data.get("softcap") is None else positive_float(data, "softcap"),
            kv_from=source,
        )
        if out.heads % out.kv_heads:
            raise ConfigError(f"{where}: {out.heads} heads are no multiple of {out.kv_heads} kv_heads")
        if out.rot is not None and out.rot.dims > out.dim:
            raise ConfigError(f"{where}: more rotated dimensions than a head has")
        return out

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
        }
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        if self.softcap is not None:
            out["softcap"] = self.softcap
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass(frozen=True)
class RofetarMamba2:
    """A state-space mixer: one decay per head and token, keys and queries shared by groups of heads."""

    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int

    kind: ClassVar[str] = "mamba2"

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "RofetarMamba2":
        keys = ("heads", "vdim", "state", "groups", "conv", "norm_groups")
        require_keys(data, keys, where)
        out = cls(**{k: positive_int(data, k) for k in keys})
        if out.heads % out.groups:
            raise ConfigError(f"{where}: {out.heads} heads are no multiple of {out.groups} groups")
        if (out.heads * out.vdim) % out.norm_groups:
            raise ConfigError(f"{where}: heads * vdim does not divide into {out.norm_groups} norm_groups")
        return out

    def to_dict(self) -> dict[str, Any]:
        return {
            "heads": self.heads, "vdim": self.vdim, "state": self.state, "groups": self.groups, "conv": self.conv,
            "norm_groups": self.norm_groups,
        }


@dataclass(frozen=True)
class RofetarDelta:
    """A gated delta rule: every write replaces what the state holds under its key."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    kind: ClassVar[str] = "delta"

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "RofetarDelta":
        require_keys(data, ("heads", "dim", "vdim", "conv"), where)
        heads = positive_int(data, "heads")
        out = cls(
            heads=heads,
            kv_heads=heads if data.get("kv_heads") is None else positive_int(data, "kv_heads"),
            dim=positive_int(data, "dim"),
            vdim=positive_int(data, "vdim"),
            conv=positive_int(data, "conv"),
        )
        if out.heads % out.kv_heads:
            raise ConfigError(f"{where}: {out.heads} heads are no multiple of {out.kv_heads} kv_heads")
        return out

    def to_dict(self) -> dict[str, Any]:
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.conv}


_MIXERS = {c.kind: c for c in (RofetarAttention, RofetarMamba2, RofetarDelta)}


@dataclass(frozen=True)
class RofetarFeedForward:
    """down(gelu(gate(x)) * up(x)), a bias on each of the three."""

    ff: int

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "RofetarFeedForward":
        require_keys(data, ("kind", "ff"), where)
        if data["kind"] != "dense":
            raise ConfigError(f"{where}: kind must be 'dense', found {data['kind']!r}")
        return cls(ff=positive_int(data, "ff"))

    def to_dict(self) -> dict[str, Any]:
        return {"kind": "dense", "ff": self.ff}


@dataclass(frozen=True)
class RofetarLayer:
    mixer: Any  # one of the three mixer configurations
    mlp: Optional[RofetarFeedForward]

    def to_dict(self) -> dict[str, Any]:
        return {"type": self.mixer.kind, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass(frozen=True)
class RofetarConfig(ModelConfig):
    architecture: ClassVar[str] = "Rofetar"
    model_type: ClassVar[str] = "rofetar"

    vocab: int
    width: int
    norm_eps: float
    layers: tuple[RofetarLayer, ...]

    def __post_init__(self) -> None:
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError("RofetarConfig: vocab and width must be > 0")
        if not self.layers:
            raise ConfigError("RofetarConfig: a model needs at least one layer")
        if not self.norm_eps >= 0:
            raise ConfigError("RofetarConfig: norm.eps must be >= 0")
        for i, layer in enumerate(self.layers):
            m = layer.mixer
            source = getattr(m, "kv_from", None)
            if source is None:
                continue
            other = self.layers[source].mixer if source < i else None
            if not isinstance(other, RofetarAttention) or other.kv_from is not None:
                raise ConfigError(f"layers[{i}]: kv_from must name an earlier attention layer that makes its own keys")
            if (other.kv_heads, other.dim, other.vdim, other.rot) != (m.kv_heads, m.dim, m.vdim, m.rot):
                raise ConfigError(f"layers[{i}]: kv_heads, dim, vdim and rotation must equal those of layer {source}")

    @classmethod
    def from_dict(cls, data: Mapping[str, Any]) -> "RofetarConfig":
        require_keys(data, ("vocab", "width", "norm", "layers"), "RofetarConfig")
        norm = _mapping(data, "norm", "RofetarConfig")
        require_keys(norm, ("eps",), "RofetarConfig.norm")
        eps = norm["eps"]
        if isinstance(eps, bool) or not isinstance(eps, (int, float)) or not eps >= 0:
            raise ConfigError(f"norm.eps must be a number >= 0, found {eps!r}")
        listed = data["layers"]
        if not isinstance(listed, (list, tuple)):
            raise ConfigError("RofetarConfig: 'layers' must be a list")
        layers = []
        for i, entry in enumerate(listed):
            where = f"layers[{i}]"
            if not isinstance(entry, Mapping):
                raise ConfigError(f"{where} must be an object")
            require_keys(entry, ("type", "mixer"), where)
            if entry["type"] not in _MIXERS:
                raise ConfigError(f"{where}: unknown mixer type {entry['type']!r}; known: {', '.join(sorted(_MIXERS))}")
            mixer = _MIXERS[entry["type"]].from_dict(_mapping(entry, "mixer", where), where + ".mixer")
            mlp = entry.get("mlp")
            if mlp is not None and not isinstance(mlp, Mapping):
                raise ConfigError(f"{where}: 'mlp' must be an object or null")
            layers.append(RofetarLayer(mixer, None if mlp is None else RofetarFeedForward.from_dict(mlp, where + ".mlp")))
        return cls(
            vocab=positive_int(data, "vocab"), width=positive_int(data, "width"), norm_eps=float(eps), layers=tuple(layers)
        )

    def to_dict(self) -> dict[str, Any]:
        return {
            "architecture": self.architecture,
            "vocab": self.vocab,
            "width": self.width,
            "norm": {"eps": self.norm_eps},
            "layers": [layer.to_dict() for layer in self.layers],
        }
