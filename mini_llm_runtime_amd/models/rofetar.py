"""The Rofetar decoder as a list of parts.

A decoder whose config.json lists the layers one by one.  The sublayers read the residual stream as it is and
their outputs are normed before they enter it (`post_norm`).  A layer mixes tokens by grouped-query attention
(queries and keys normed per head and partly rotated, capped scores, one more in the softmax's denominator; some
layers read an earlier layer's keys and values: `gqa_attention`), by a state-space recurrence behind a short
convolution (`state_space`) or by a gated delta rule behind short convolutions (`gated_delta`), and has a dense
gated feed-forward with biases (`geglu`) or none.  The head is a matrix of its own.

Checkpoint tensors: `embed`, `final.norm`, `head`, and per layer i `l<i>.norm1`, `l<i>.norm2`,
`l<i>.mix.{q,k,v,q.norm,k.norm,o}` (attention; without k, v and k.norm where another layer's are read),
`l<i>.mix.{in,conv,conv.b,dt_bias,A_log,D,norm,o}` (state space), `l<i>.mix.{q,k,v}` with `.conv` and
`l<i>.mix.{b,a,A_log,dt_bias,g,norm,o}` (delta rule), `l<i>.mlp.{gate,up,down}` with `.b` biases; linear weights
are stored [out, in].
"""

from __future__ import annotations

from ..config.rofetar import RofetarAttention, RofetarConfig, RofetarDelta, RofetarMamba2
from ..parts.spec import LayerSpec, ModelSpec, OrderEntry, PartSpec, WeightRule
from .registry import register_architecture

# positions are only limited by what a rotation can tell apart
_NO_POSITION_LIMIT = 1 << 30


def _rotary(rot, head_dim: int) -> PartSpec:
    scaling = None
    if rot.scaling is not None:
        s = rot.scaling
        scaling = {"factor": s.factor, "original": s.original, "fast": s.fast, "slow": s.slow}
    return PartSpec("rotary", {"head_dim": head_dim, "theta": rot.base, "rotary_dim": rot.dims, "scaling": scaling})


def rofetar_spec(config: RofetarConfig) -> ModelSpec:
    width, eps = config.width, config.norm_eps
    norm = PartSpec("rms_norm", {"size": width, "eps": eps})
    layers: list[LayerSpec] = []
    order: list[OrderEntry] = []
    rules: list[WeightRule] = [WeightRule("embed", "embed.weight")]
    for i, layer in enumerate(config.layers):
        src, dst = f"l{i}.", f"layers.{i}."
        m = layer.mixer
        mix = dst + "mixer."
        reads = None
        if isinstance(m, RofetarAttention):
            reads = m.kv_from
            mixer = PartSpec(
                "gqa_attention",
                {
                    "hidden_size": width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
                    "value_dim": m.vdim, "scale": m.scale, "qkv_bias": False, "qk_norm_eps": eps, "softcap": m.softcap,
                    "unit_sink": True, "reads_cache": reads is not None,
                    "position": None if m.rot is None else _rotary(m.rot, m.dim),
                },
            )
            q, k, v = m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim
            rules += [
                WeightRule(src + "mix.q", mix + "qkv_weight", 0, q),
                WeightRule(src + "mix.q.norm", mix + "q_norm_weight"),
                WeightRule(src + "mix.o", mix + "o_weight"),
            ]
            if reads is None:
                rules += [
                    WeightRule(src + "mix.k", mix + "qkv_weight", q, k),
                    WeightRule(src + "mix.v", mix + "qkv_weight", q + k, v),
                    WeightRule(src + "mix.k.norm", mix + "k_norm_weight"),
                ]
        elif isinstance(m, RofetarMamba2):
            mixer = PartSpec(
                "state_space",
                {
                    "hidden_size": width, "num_heads": m.heads, "value_dim": m.vdim, "state_dim": m.state,
                    "groups": m.groups, "taps": m.conv, "norm_groups": m.norm_groups, "norm_eps": eps,
                },
            )
            rules += [
                WeightRule(src + "mix.in", mix + "in_weight"),  # rows z, x, B, C, dt, as the part wants them
                WeightRule(src + "mix.conv", mix + "conv_weight"),
                WeightRule(src + "mix.conv.b", mix + "conv_bias"),
                WeightRule(src + "mix.dt_bias", mix + "dt_bias"),
                WeightRule(src + "mix.A_log", mix + "log_rate"),
                WeightRule(src + "mix.D", mix + "skip"),
                WeightRule(src + "mix.norm", mix + "norm_weight"),
                WeightRule(src + "mix.o", mix + "o_weight"),
            ]
        elif isinstance(m, RofetarDelta):
            mixer = PartSpec(
                "gated_delta",
                {
                    "hidden_size": width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
                    "value_dim": m.vdim, "taps": m.conv, "norm_eps": eps,
                },
            )
            qk, v = m.kv_heads * m.dim, m.heads * m.vdim
            rules += [
                WeightRule(src + "mix.q", mix + "in_weight", 0, qk),
                WeightRule(src + "mix.k", mix + "in_weight", qk, qk),
                WeightRule(src + "mix.v", mix + "in_weight", 2 * qk, v),
                WeightRule(src + "mix.g", mix + "in_weight", 2 * qk + v, v),
                WeightRule(src + "mix.a", mix + "in_weight", 2 * qk + 2 * v, m.heads),
                WeightRule(src + "mix.b", mix + "in_weight", 2 * qk + 2 * v + m.heads, m.heads),
                WeightRule(src + "mix.q.conv", mix + "conv_weight", 0, qk),
                WeightRule(src + "mix.k.conv", mix + "conv_weight", qk, qk),
                WeightRule(src + "mix.v.conv", mix + "conv_weight", 2 * qk, v),
                WeightRule(src + "mix.dt_bias", mix + "dt_bias"),
                WeightRule(src + "mix.A_log", mix + "log_rate"),
                WeightRule(src + "mix.norm", mix + "norm_weight"),
                WeightRule(src + "mix.o", mix + "o_weight"),
            ]
        else:
            raise TypeError(f"layer {i}: unknown mixer configuration {type(m).__name__}")
        norms = {"mixer_out": norm}
        rules.append(WeightRule(src + "norm1", dst + "norm_mixer_out.weight"))
        feed_forward = None
        f = layer.mlp
        if f is not None:
            norms["ff_out"] = norm
            feed_forward = PartSpec("geglu", {"hidden_size": width, "intermediate_size": f.ff})
            ff = dst + "feed_forward."
            # gate and up rows (and biases) woven in pairs: the product's epilogue then holds a gate sum
            # beside its up sum (an odd size cannot be woven: gate rows, then up rows)
            weave = dict(block=2, period=4) if f.ff % 2 == 0 else {}
            up_at = 2 if weave else f.ff
            rules += [
                WeightRule(src + "norm2", dst + "norm_ff_out.weight"),
                WeightRule(src + "mlp.gate", ff + "gate_up_weight", 0, f.ff, **weave),
                WeightRule(src + "mlp.up", ff + "gate_up_weight", up_at, f.ff, **weave),
                WeightRule(src + "mlp.gate.b", ff + "gate_up_bias", 0, f.ff, **weave),
                WeightRule(src + "mlp.up.b", ff + "gate_up_bias", up_at, f.ff, **weave),
                WeightRule(src + "mlp.down", ff + "down_weight"),
                WeightRule(src + "mlp.down.b", ff + "down_bias"),
            ]
        layers.append(LayerSpec(block="post_norm", mixer=mixer, feed_forward=feed_forward, norms=norms))
        order.append(OrderEntry(i, reads_cache_of=reads))  # a layer runs once: its site is its index
    rules += [WeightRule("final.norm", "final_norm.weight"), WeightRule("head", "head.weight")]
    return ModelSpec(
        architecture=config.architecture,
        vocab_size=config.vocab,
        hidden_size=width,
        max_position_embeddings=_NO_POSITION_LIMIT,
        layers=tuple(layers),
        order=tuple(order),
        final_norm=norm,
        tie_word_embeddings=False,
        weight_rules=tuple(rules),
    )


register_architecture(RofetarConfig.architecture, RofetarConfig, rofetar_spec, replace=True)
