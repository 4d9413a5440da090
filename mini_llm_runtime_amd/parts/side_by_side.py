"""Several mixers on one input."""

from __future__ import annotations

from typing import Any, Mapping, Optional

import torch

from ..cache.spec import CompositeSpec
from ..kernels.pending import NormedDelta
from .base import Mixer, Part
from .context import StepContext, site_member
from .registry import build_part, register_part
from .spec import ParamSpec, PartSpec


@register_part("mixer", "side_by_side")
class SideBySide(Mixer):
    """Mixers that all read the same input; the result is the sum of their results, each times a
    constant:  sum_m scale_m * mixer_m(h).

    Every member leaves its output product open (`Mixer.open_output`): the members' activations, each
    already times its constant (in 32-bit, before their one rounding), stand side by side in one
    tensor and ONE product with the members' output matrices side by side, [Wo_a | Wo_b | ...], makes
    the sum.  That matrix is put together when the weights are bound; the members' own copies are
    dropped.  Members that take their input product's sums from outside (`open_input`: an `in_weight`
    [rows, hidden], maybe an `in_bias`, and `activations(projected=)`) share ONE input product too: their
    matrices one under the other, 32-bit sums, each member reading its own columns.  Every member keeps its own cache: the site's cache is a composite with one member per mixer
    that keeps one, under the mixer's name.

    out_norm_eps: every member's result is normed over the model width first, sum_m scale_m * w_m * y_m / rms(y_m) (this eps
    inside the roots, a weight `<member>_out_norm` each).  The output products then stay apart, of at most two members,
    and what is handed on is a `NormedDelta`: norms, sum, addition to the stream and the next norm are one kernel.
    """

    replayable = True
    open_output = True

    def __init__(
        self, hidden_size: int, members: Mapping[str, PartSpec], scales: Optional[Mapping[str, float]] = None,
        out_norm_eps: Optional[float] = None,
    ) -> None:
        if not members:
            raise ValueError("side_by_side needs at least one mixer")
        self.out_norm_eps = None if out_norm_eps is None else float(out_norm_eps)
        if self.out_norm_eps is not None and (len(members) > 2 or not self.out_norm_eps >= 0):
            raise ValueError("normed results have an eps >= 0 and come from one or two mixers")
        self.hidden_size = int(hidden_size)
        self.members: dict[str, Mixer] = {name: build_part("mixer", spec) for name, spec in members.items()}
        self.scales = {name: float((scales or {}).get(name, 1.0)) for name in self.members}
        self.columns: dict[str, int] = {}
        at = 0
        if self.out_norm_eps is None:
            for name, member in self.members.items():
                if not member.open_output:
                    raise ValueError(f"side_by_side member {name!r} does not leave its output product open")
                self.columns[name] = at
                at += member.out_width
        else:
            self.open_output = False  # the members' results are not one product
        self._width = at
        self.out_norms: dict[str, torch.Tensor] = {}
        self.o_weight: Optional[torch.Tensor] = None
        self.in_weight: Optional[torch.Tensor] = None
        self.in_bias: Optional[torch.Tensor] = None
        self.in_columns: dict[str, int] = {}

    @property
    def out_width(self) -> int:
        return self._width

    def children(self) -> dict[str, Part]:
        return dict(self.members)

    def param_specs(self) -> dict[str, ParamSpec]:
        if self.out_norm_eps is None:
            return {}
        spec = ParamSpec((self.hidden_size,), init="one_plus_normal", keep_stored_precision=True)
        return {f"{name}_out_norm": spec for name in self.members}

    def bind(self, params, *, dtype: torch.dtype, device: torch.device) -> None:
        self.out_norms = {name: params[f"{name}_out_norm"] for name in self.members} if self.out_norm_eps is not None else {}

    def bound(self) -> None:
        """[hidden, sum of the members' widths] and the joint input matrix; the members' own matrices are let go."""
        if self.out_norm_eps is None:
            parts = []
            for name, member in self.members.items():
                if member.o_weight is None:
                    raise RuntimeError(f"side_by_side: the output matrix of member {name!r} is not bound")
                parts.append(member.o_weight)
            self.o_weight = torch.cat(parts, dim=1).contiguous()
            for member in self.members.values():
                member.o_weight = None
        if len(self.members) > 1 and all(getattr(m, "open_input", False) and m.in_weight is not None for m in self.members.values()):
            at, weights, biases = 0, [], []
            for name, member in self.members.items():
                self.in_columns[name] = at
                at += member.in_weight.shape[0]
                weights.append(member.in_weight)
                biases.append(getattr(member, "in_bias", None))
            self.in_weight = torch.cat(weights, dim=0).contiguous()
            if any(b is not None for b in biases):
                kind = next(b.dtype for b in biases if b is not None)
                self.in_bias = torch.cat(
                    [b.to(kind) if b is not None else w.new_zeros(w.shape[0], dtype=kind) for b, w in zip(biases, weights)]
                ).contiguous()
            for member in self.members.values():
                member.in_weight = None
                if getattr(member, "in_bias", None) is not None:
                    member.in_bias = None

    def held_tensors(self) -> list:
        return [self.o_weight, self.in_weight, self.in_bias, *self.out_norms.values()]

    def cache_spec(self) -> Any:
        specs = {name: member.cache_spec() for name, member in self.members.items()}
        specs = {name: spec for name, spec in specs.items() if spec is not None}
        return CompositeSpec(specs) if specs else None

    def plan(self, ops, shape):
        for member in self.members.values():
            plan = member.plan(ops, shape)
            if plan is not None:
                return plan
        return None

    def activations(self, ctx: StepContext, h, site: Any, *, out: torch.Tensor, column: int, scale: float = 1.0) -> None:
        inputs = self._inputs(ctx, h)
        for name, member in self.members.items():
            member.activations(
                ctx, h, site_member(site, name), out=out, column=column + self.columns[name], scale=scale * self.scales[name],
                **inputs[name],
            )

    def _inputs(self, ctx: StepContext, h) -> dict[str, dict]:
        """What every member is handed of the joint input product (nothing, where there is none)."""
        if self.in_weight is None:
            return {name: {} for name in self.members}
        projected = ctx.ops.linear(h, self.in_weight, self.in_bias, out_dtype=torch.float32)
        return {name: {"projected": (projected, self.in_columns[name])} for name in self.members}

    def forward(self, ctx: StepContext, h: torch.Tensor, site: Any) -> torch.Tensor:
        if self.out_norm_eps is not None:
            inputs = self._inputs(ctx, h)
            (name, y), *rest = [
                (name, member.forward(ctx, h, site_member(site, name), **inputs[name])) for name, member in self.members.items()
            ]
            second = None if not rest else (rest[0][1], self.out_norms[rest[0][0]])
            return NormedDelta(
                y, self.out_norms[name], self.out_norm_eps, second, self.scales[name], self.scales[rest[0][0]] if rest else 1.0
            )
        weight = self.o_weight
        out = torch.empty((h.shape[0], self._width), dtype=ctx.dtype, device=ctx.device)
        self.activations(ctx, h, site, out=out, column=0)
        return ctx.ops.linear(out, weight, None, for_stream=True)
