"""Linear attention by a delta rule with a decay: a write replaces what the state holds under its key."""

from __future__ import annotations

from typing import Any, Optional

import torch

from ..cache.spec import SlotStateSpec
from ..kernels.limits import MAX_STATE_ROWS
from .base import Mixer
from .context import StepContext
from .registry import register_part
from .spec import ParamSpec
from .state_space import conv_state_spec, conv_state_views


@register_part("mixer", "gated_delta")
class GatedDelta(Mixer):
    """Per head a state S (head_dim x value_dim, 32-bit, zero at a request's start).  With h the mixer's input, q and k
    (num_kv_heads x head_dim) and v (num_heads x value_dim) each pass a causal convolution over time per channel (`taps`
    taps, no bias) and silu; q and k are made unit vectors per head, x / sqrt(sum x^2 + 1e-6), and q is multiplied by
    head_dim^-0.5; head i reads q/k head i // (num_heads // num_kv_heads).  Per token and head

        g = exp(-exp(log_rate) softplus(Wa h + dt_bias)),    b = sigmoid(Wb h),
        S <- g S,    u = b (v - S^T k),    S <- S + k u^T,    o = S^T q.

    Every head's o is divided by its root mean square and multiplied by one weight [value_dim] that all heads share;
    the heads side by side are multiplied by silu(Wg h) and projected by Wo.

    A request keeps its state and the convolutions' last inputs (two members of the site in the cache manager's state
    banks), so a prompt can be cut anywhere.  One input product (rows q, k, v, gate, a, b; 32-bit sums); convolutions,
    activations, unit norms and gates, then the scan (one kernel where a step has single tokens only); a kernel for norm
    and gate; the output product.
    """

    replayable = True

    def __init__(
        self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, value_dim: int, taps: int, norm_eps: float
    ) -> None:
        if min(hidden_size, num_heads, num_kv_heads, head_dim, value_dim, taps) <= 0 or num_heads % num_kv_heads:
            raise ValueError("GatedDelta sizes must be > 0, num_heads a multiple of num_kv_heads")
        if head_dim > MAX_STATE_ROWS:  # refused here, not at the first step
            raise ValueError(f"head_dim {head_dim}: the recurrence kernels take heads of up to {MAX_STATE_ROWS} dims")
        self.hidden_size = int(hidden_size)
        self.num_heads = int(num_heads)
        self.num_kv_heads = int(num_kv_heads)
        self.head_dim = int(head_dim)
        self.value_dim = int(value_dim)
        self.taps = int(taps)
        self.norm_eps = float(norm_eps)
        qk, v = self.num_kv_heads * self.head_dim, self.num_heads * self.value_dim
        # columns of the one input product; q, k and v pass the convolution
        self.k_at, self.v_at = qk, 2 * qk
        self.channels = 2 * qk + v
        self.gate_at = self.channels
        self.step_at = self.gate_at + v
        self.write_at = self.step_at + self.num_heads
        self.in_rows = self.write_at + self.num_heads
        self.in_weight: Optional[torch.Tensor] = None
        self.conv_weight: Optional[torch.Tensor] = None
        self.dt_bias: Optional[torch.Tensor] = None
        self.log_rate: Optional[torch.Tensor] = None
        self.norm_weight: Optional[torch.Tensor] = None
        self.o_weight: Optional[torch.Tensor] = None
        self.conv_taps: Optional[torch.Tensor] = None
        self.rate: Optional[torch.Tensor] = None

    def param_specs(self) -> dict[str, ParamSpec]:
        return {
            "in_weight": ParamSpec((self.in_rows, self.hidden_size)),
            "conv_weight": ParamSpec((self.channels, self.taps), keep_stored_precision=True),
            "dt_bias": ParamSpec((self.num_heads,), keep_stored_precision=True),
            "log_rate": ParamSpec((self.num_heads,), keep_stored_precision=True),
            "norm_weight": ParamSpec((self.value_dim,), init="one_plus_normal", keep_stored_precision=True),
            "o_weight": ParamSpec((self.hidden_size, self.num_heads * self.value_dim)),
        }

    def bind(self, params, *, dtype: torch.dtype, device: torch.device) -> None:
        super().bind(params, dtype=dtype, device=device)
        # everything that enters the recurrence besides the products is 32-bit
        self.conv_taps = self.conv_weight.to(torch.float32).t().contiguous()  # [taps, channels]
        self.dt_bias = self.dt_bias.to(torch.float32)
        self.rate = -torch.exp(self.log_rate.to(torch.float32))

    def cache_spec(self):
        state = SlotStateSpec((self.num_heads, self.head_dim, self.value_dim), "float32")
        return conv_state_spec(state, self.taps, self.channels)

    def forward(self, ctx: StepContext, h: torch.Tensor, site: Any) -> torch.Tensor:
        ops = ctx.ops
        state, carried = conv_state_views(ctx, site, self.taps)
        projected = ops.linear(h, self.in_weight, None, out_dtype=torch.float32)  # what enters the recurrence stays 32-bit
        o = ops.conv_decay_scan(
            projected, self.conv_taps, None, carried, state, ctx, column=0, heads=self.num_heads,
            key_heads=self.num_kv_heads, head_dim=self.head_dim, value_dim=self.value_dim,
            offsets=(0, self.k_at, self.v_at), rate=self.rate, dt_bias=self.dt_bias, step_column=self.step_at,
            write_column=self.write_at, delta=True,
        )
        gated = ops.retention_gate(
            o, projected, heads=self.num_heads, value_dim=self.value_dim, gate_offset=self.gate_at, eps=self.norm_eps,
            norm_weight=self.norm_weight,
        )
        return ops.linear(gated, self.o_weight, None, for_stream=True)
