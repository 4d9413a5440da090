"""A state-space mixer (Mamba-2's recurrence): one decay per head and token."""

from __future__ import annotations

from typing import Any, Optional

import torch

from ..cache.spec import CompositeSpec, SlotStateSpec
from ..kernels.limits import MAX_STATE_ROWS
from .base import Mixer
from .context import StepContext, site_member
from .registry import register_part
from .spec import ParamSpec


def conv_state_spec(state: SlotStateSpec, taps: int, channels: int) -> Any:
    """What a recurrence behind a short convolution keeps: its state and the last taps - 1 inputs of the
    convolution (32-bit both), as two members of one site; with one tap the state alone."""
    if taps == 1:
        return state
    return CompositeSpec({"state": state, "conv": SlotStateSpec((taps - 1, channels), "float32")})


def conv_state_views(ctx: StepContext, site: Any, taps: int) -> tuple[Any, Any]:
    """(view of the state, view of the carried inputs or None) under `conv_state_spec`."""
    if taps == 1:
        return ctx.state(site), None
    return ctx.state(site_member(site, "state")), ctx.state(site_member(site, "conv"))


@register_part("mixer", "state_space")
class StateSpace(Mixer):
    """Per head a state S (state_dim x value_dim, 32-bit, zero at a request's start).  W_in h is laid out as z (heads x
    value_dim), x (heads x value_dim), B and C (groups x state_dim each), d (heads).  x, B and C together pass a causal
    convolution over time per channel (`taps` taps, bias) and silu; with t = softplus(d + dt_bias) and a head's group
    its place in equal runs of heads,

        S_t = exp(-exp(log_rate) t) S_(t-1) + t B_t x_t^T,    y_t = S_t^T C_t + skip x_t.

    The heads side by side are multiplied by silu(z), then divided in `norm_groups` equal parts by each part's own
    root mean square, multiplied by a weight over all of them and projected by Wo.

    A request keeps its state and the convolution's last inputs (two members of the site in the cache manager's state
    banks), so a prompt can be cut anywhere.  One input product with 32-bit sums; convolution, activation and decays,
    then the scan (one kernel where a step has single tokens only); a kernel for gate and norm; the output product.
    """

    replayable = True
    open_input = True  # `forward(projected=)` takes the input product's sums from whoever made them

    def __init__(
        self, hidden_size: int, num_heads: int, value_dim: int, state_dim: int, groups: int, taps: int, norm_groups: int,
        norm_eps: float,
    ) -> None:
        if min(hidden_size, num_heads, value_dim, state_dim, groups, taps, norm_groups) <= 0:
            raise ValueError("StateSpace sizes must be > 0")
        if num_heads % groups or (num_heads * value_dim) % norm_groups:
            raise ValueError("groups must divide the heads, norm_groups the heads' width")
        if state_dim > MAX_STATE_ROWS:  # refused here, not at the first step
            raise ValueError(f"state_dim {state_dim}: the recurrence kernels take states of up to {MAX_STATE_ROWS} rows")
        self.hidden_size = int(hidden_size)
        self.num_heads = int(num_heads)
        self.value_dim = int(value_dim)
        self.state_dim = int(state_dim)
        self.groups = int(groups)
        self.taps = int(taps)
        self.norm_groups = int(norm_groups)
        self.norm_eps = float(norm_eps)
        self.inner = self.num_heads * self.value_dim
        self.channels = self.inner + 2 * self.groups * self.state_dim  # what passes the convolution: x, B, C
        self.in_rows = self.inner + self.channels + self.num_heads
        self.in_weight: Optional[torch.Tensor] = None
        self.conv_weight: Optional[torch.Tensor] = None
        self.conv_bias: Optional[torch.Tensor] = None
        self.dt_bias: Optional[torch.Tensor] = None
        self.log_rate: Optional[torch.Tensor] = None
        self.skip: Optional[torch.Tensor] = None
        self.norm_weight: Optional[torch.Tensor] = None
        self.o_weight: Optional[torch.Tensor] = None
        self.conv_taps: Optional[torch.Tensor] = None
        self.rate: Optional[torch.Tensor] = None

    def param_specs(self) -> dict[str, ParamSpec]:
        return {
            "in_weight": ParamSpec((self.in_rows, self.hidden_size)),
            "conv_weight": ParamSpec((self.channels, self.taps), keep_stored_precision=True),
            "conv_bias": ParamSpec((self.channels,), keep_stored_precision=True),
            "dt_bias": ParamSpec((self.num_heads,), keep_stored_precision=True),
            "log_rate": ParamSpec((self.num_heads,), keep_stored_precision=True),
            "skip": ParamSpec((self.num_heads,), init="one_plus_normal", keep_stored_precision=True),
            "norm_weight": ParamSpec((self.inner,), init="one_plus_normal", keep_stored_precision=True),
            "o_weight": ParamSpec((self.hidden_size, self.inner)),
        }

    def bind(self, params, *, dtype: torch.dtype, device: torch.device) -> None:
        super().bind(params, dtype=dtype, device=device)
        # everything that enters the recurrence besides the products is 32-bit
        self.conv_taps = self.conv_weight.to(torch.float32).t().contiguous()  # [taps, channels]
        self.conv_bias = self.conv_bias.to(torch.float32)
        self.dt_bias = self.dt_bias.to(torch.float32)
        self.rate = -torch.exp(self.log_rate.to(torch.float32))
        self.skip = self.skip.to(torch.float32)

    def cache_spec(self):
        state = SlotStateSpec((self.num_heads, self.state_dim, self.value_dim), "float32")
        return conv_state_spec(state, self.taps, self.channels)

    def forward(self, ctx: StepContext, h: torch.Tensor, site: Any, projected=None) -> torch.Tensor:
        """`projected`: (float32 sums [T, ...], first column) of h times `in_weight`, when the caller made them within a
        larger product."""
        ops = ctx.ops
        state, carried = conv_state_views(ctx, site, self.taps)
        first = 0
        if projected is None:
            projected = ops.linear(h, self.in_weight, None, out_dtype=torch.float32)  # what enters the recurrence stays 32-bit
        else:
            projected, first = projected
        b_at = self.inner  # the channels: x, B, C
        y = ops.conv_decay_scan(
            projected, self.conv_taps, self.conv_bias, carried, state, ctx, column=first + self.inner, heads=self.num_heads,
            key_heads=self.groups, head_dim=self.state_dim, value_dim=self.value_dim,
            offsets=(b_at + self.groups * self.state_dim, b_at, 0), rate=self.rate, dt_bias=self.dt_bias,
            step_column=first + self.inner + self.channels, skip=self.skip,
        )
        gated = ops.gate_group_norm(
            y, projected, gate_column=first, groups=self.norm_groups, eps=self.norm_eps, norm_weight=self.norm_weight
        )
        return ops.linear(gated, self.o_weight, None, for_stream=True)
