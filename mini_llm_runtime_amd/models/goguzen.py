"""The Goguzen decoder as a list of parts.

A pre-norm decoder whose config.json lists the layers one by one.  A layer mixes tokens by attention over a window
and the first tokens (queries and keys normed over their whole projection and partly rotated, a sink:
`pooled_window_attention` without pools), or by two mixers side by side whose outputs are normed before they are added
(`side_by_side`): attention whose values are its keys before their norm, with queries that grow with their position
and a sink (`gqa_attention`), and a state-space recurrence behind a short convolution (`state_space`).  The feed-forward is a
mixture of gated experts with clamped halves, weighted by the softmax over the chosen router logits, beside a shared
one that every token runs (`routed_experts`), or absent.  A layer may use an earlier layer's tensors: it then is one
more execution site of that layer, with a cache and state of its own.  The embedding is scaled, the head is a matrix of
its own, the logits are scaled and capped.

Checkpoint tensors: `embed`, `final.norm`, `head`, and per layer i that has tensors `l<i>.norm1`, `l<i>.norm2`,
`l<i>.mix.{q,k,v,q.norm,k.norm,sink,o}` (attention), `l<i>.mix.left.{q,k,q.norm,k.norm,sink,o,out}` with
`l<i>.mix.right.{in,conv,conv.b,dt_bias,A_log,D,norm,o,out}` (side by side), `l<i>.mlp.{router,router.b}`,
`l<i>.mlp.e<j>.{gate,up,down}` and `l<i>.mlp.shared.{gate,up,down}`; linear weights are stored [out, in].
"""

from __future__ import annotations

from ..config.goguzen import GoguzenAttention, GoguzenConfig, GoguzenMixture, GoguzenParallel
from ..parts.spec import LayerSpec, ModelSpec, OrderEntry, PartSpec, WeightRule
from .registry import register_architecture

# positions are only limited by what a rotation can tell apart
_NO_POSITION_LIMIT = 1 << 30


def _rotary(rot, head_dim: int):
    if rot is None or rot.dims == 0:
        return None
    scaling = None
    if rot.scaling is not None:
        s = rot.scaling
        scaling = {"factor": s.factor, "low": s.low, "high": s.high, "original": s.original}
    return PartSpec("rotary", {"head_dim": head_dim, "theta": rot.base, "rotary_dim": rot.dims, "scaling": scaling})


def _gate_and_up(name: str, dest: str, ff: int, row: int = 0) -> list[WeightRule]:
    """Gate and up rows of one expert from row `row` of `dest` on: woven in pairs, so that a product's epilogue holds a
    gate sum beside its up sum (an odd size cannot be woven: gate rows, then up rows)."""
    if ff % 2 == 0:
        return [
            WeightRule(name + ".gate", dest, row, ff, block=2, period=4),
            WeightRule(name + ".up", dest, row + 2, ff, block=2, period=4),
        ]
    return [WeightRule(name + ".gate", dest, row, ff), WeightRule(name + ".up", dest, row + ff, ff)]


def _mixture(f: GoguzenMixture, width: int, src: str, ff: str) -> tuple[PartSpec, list[WeightRule]]:
    inner = f.expert.ff
    part = PartSpec(
        "routed_experts",
        {
            "hidden_size": width, "intermediate_size": inner, "experts": f.experts, "top": f.top, "activation": "clamped_glu",
            "limit": f.expert.limit, "scores": "chosen_softmax", "correction": False, "router_bias": True,
            "shared": None if f.shared is None else PartSpec(
                "clamped_glu",
                {"hidden_size": width, "intermediate_size": f.shared.ff, "limit": f.shared.limit, "bias": False},
            ),
        },
    )
    rules = [WeightRule(src + "router", ff + "router_weight"), WeightRule(src + "router.b", ff + "router_bias")]
    for e in range(f.experts):
        rules += _gate_and_up(f"{src}e{e}", ff + "up_weight", inner, 2 * e * inner)
        rules.append(WeightRule(f"{src}e{e}.down", ff + "down_weight", e * width, width))
    if f.shared is not None:
        rules += _gate_and_up(src + "shared", ff + "shared.gate_up_weight", f.shared.ff)
        rules.append(WeightRule(src + "shared.down", ff + "shared.down_weight"))
    return part, rules


def goguzen_spec(config: GoguzenConfig) -> ModelSpec:
    width, eps = config.width, config.norm_eps
    norm = PartSpec("rms_norm", {"size": width, "eps": eps})
    layers: list[LayerSpec] = []
    rules: list[WeightRule] = [WeightRule("embed", "embed.weight")]
    place: dict[int, int] = {}  # listed layer -> its place among the layers that have tensors
    for i, layer in enumerate(config.layers):
        if config.owner_of(i) != i:
            continue
        place[i] = len(layers)
        src, dst = f"l{i}.", f"layers.{place[i]}."
        m = layer.mixer
        mix = dst + "mixer."
        if isinstance(m, GoguzenAttention):
            mixer = PartSpec(
                "pooled_window_attention",
                {
                    "hidden_size": width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
                    "value_dim": m.vdim, "window": m.window, "keep_first": m.keep_first, "scale": m.scale,
                    "position": _rotary(m.rot, m.dim), "qkv_bias": False, "qk_norm": True, "norm_eps": eps, "sink": True,
                },
            )
            q, k, v = m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim
            rules += [
                WeightRule(src + "mix.q", mix + "in_weight", 0, q),
                WeightRule(src + "mix.k", mix + "in_weight", q, k),
                WeightRule(src + "mix.v", mix + "in_weight", q + k, v),
                WeightRule(src + "mix.q.norm", mix + "q_norm_weight"),
                WeightRule(src + "mix.k.norm", mix + "k_norm_weight"),
                WeightRule(src + "mix.sink", mix + "sinks"),
                WeightRule(src + "mix.o", mix + "o_weight"),
            ]
        elif isinstance(m, GoguzenParallel):
            a, b = m.left, m.right
            left = PartSpec(
                "gqa_attention",
                {
                    "hidden_size": width, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim, "scale": a.scale,
                    "qkv_bias": False, "qk_norm_eps": eps, "values_are_keys": True, "sink": True,
                    "query_temperature": None if a.temp_every is None else (a.temp_every, a.temp_coef),
                },
            )
            right = PartSpec(
                "state_space",
                {
                    "hidden_size": width, "num_heads": b.heads, "value_dim": b.vdim, "state_dim": b.state, "groups": b.groups,
                    "taps": b.conv, "norm_groups": b.norm_groups, "norm_eps": eps,
                },
            )
            mixer = PartSpec(
                "side_by_side",
                {
                    "hidden_size": width, "members": {"left": left, "right": right}, "scales": {"left": 0.5, "right": 0.5},
                    "out_norm_eps": eps,
                },
            )
            lm, rm = mix + "left.", mix + "right."
            q, k = a.heads * a.dim, a.kv_heads * a.dim
            rules += [
                WeightRule(src + "mix.left.q", lm + "qkv_weight", 0, q),
                WeightRule(src + "mix.left.k", lm + "qkv_weight", q, k),
                WeightRule(src + "mix.left.q.norm", lm + "q_norm_weight"),
                WeightRule(src + "mix.left.k.norm", lm + "k_norm_weight"),
                WeightRule(src + "mix.left.sink", lm + "sinks"),
                WeightRule(src + "mix.left.o", lm + "o_weight"),
                WeightRule(src + "mix.left.out", mix + "left_out_norm"),
                WeightRule(src + "mix.right.in", rm + "in_weight"),  # rows z, x, B, C, dt, as the part wants them
                WeightRule(src + "mix.right.conv", rm + "conv_weight"),
                WeightRule(src + "mix.right.conv.b", rm + "conv_bias"),
                WeightRule(src + "mix.right.dt_bias", rm + "dt_bias"),
                WeightRule(src + "mix.right.A_log", rm + "log_rate"),
                WeightRule(src + "mix.right.D", rm + "skip"),
                WeightRule(src + "mix.right.norm", rm + "norm_weight"),
                WeightRule(src + "mix.right.o", rm + "o_weight"),
                WeightRule(src + "mix.right.out", mix + "right_out_norm"),
            ]
        else:
            raise TypeError(f"layer {i}: unknown mixer configuration {type(m).__name__}")
        norms = {"input": norm}
        rules.append(WeightRule(src + "norm1", dst + "norm_input.weight"))
        feed_forward = None
        if layer.mlp is not None:
            norms["post_mixer"] = norm
            rules.append(WeightRule(src + "norm2", dst + "norm_post_mixer.weight"))
            feed_forward, more = _mixture(layer.mlp, width, src + "mlp.", dst + "feed_forward.")
            rules += more
        layers.append(LayerSpec(block="pre_norm", mixer=mixer, feed_forward=feed_forward, norms=norms))
    rules += [WeightRule("final.norm", "final_norm.weight"), WeightRule("head", "head.weight")]
    return ModelSpec(
        architecture=config.architecture,
        vocab_size=config.vocab,
        hidden_size=width,
        max_position_embeddings=_NO_POSITION_LIMIT,
        layers=tuple(layers),
        # every listed layer is a site of its own, whichever layer's tensors it uses
        order=tuple(OrderEntry(place[config.owner_of(i)]) for i in range(len(config.layers))),
        final_norm=norm,
        tie_word_embeddings=False,
        weight_rules=tuple(rules),
        embedding_scale=config.embedding_scale,
        logit_scale=config.logit_scale,
        logit_softcap=config.logit_softcap,
    )


register_architecture(GoguzenConfig.architecture, GoguzenConfig, goguzen_spec, replace=True)
