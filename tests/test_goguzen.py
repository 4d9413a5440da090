"""The Goguzen decoder in the engine against the plain implementation (`plain_goguzen.py`).

Each mechanism alone (frequencies in bands; a window beside kept first tokens on every attention kernel; per-head
norms with keys that are values and queries that grow; two outputs normed before they are added; the softmax over the
chosen logits; clamped experts on every grouped product with a product beside them; pages that a window gives back
and kept ones that stay; one-layer models), keys placed so that one score stands out far away, at page borders and
just inside and outside every edge, a sink that takes most of the weight, a state that never forgets through one
reused slot, a layer that uses another's tensors with a cache and state of its own, then whole models under every way
of cutting and batching over poisoned pages and stale slots, the stream after every layer, replays against unrecorded
steps, and greedy generation through the engine, the command line and the replay program.  The tests make their own
small configurations and weights; sizes differ from layer to layer, also where a model could make them equal, and
some are 1.

`double` cases run everything above the kernels on the CPU stand-in; `hip` cases run the HIP kernels
(`-m gpu`) in float32 and bfloat16.
"""

from __future__ import annotations

import copy
import json
import math
from pathlib import Path
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import mini_llm_runtime_amd.models  # noqa: F401
import plain_goguzen as plain
import schedules
from helpers import StepEntry, make_runner, random_tokens
from kernel_doubles import TorchOps
from mini_llm_runtime_amd.cache.spec import PagedKVSpec
from mini_llm_runtime_amd.config import ConfigError
from mini_llm_runtime_amd.config.goguzen import GoguzenConfig
from mini_llm_runtime_amd.engine import ContinuousBatchEngine
from mini_llm_runtime_amd.models import build_model, config_from_dict
from mini_llm_runtime_amd.weights import save_state_dict

ROOT = Path(__file__).resolve().parents[1]


# ---- configurations -----------------------------------------------------------------------------------

def _rot(base, dims, scaling=None):
    out = {"base": base, "dims": dims}
    if scaling is not None:
        out["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return out


def _attn(heads, kv_heads, dim, vdim, scale, size=None, keep_first=0, rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size is not None:
        m["mask"] = {"size": size, "keep_first": keep_first}
    if rot is not None:
        m["rot"] = rot
    return "attention", m


def _left(heads, kv_heads, dim, scale, every=None, coef=0.0):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if every is not None:
        m["q_temp"] = {"every": every, "coef": coef}
    return m


def _ssm(heads, vdim, state, groups, conv, norm_groups):
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}


def _both(left, right):
    return "parallel", {"left": left, "right": right}


def _moe(experts, top, ff, limit, shared=None):
    f = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}
    if shared is not None:
        f["shared"] = {"ff": shared[0], "limit": shared[1]}
    return f


def _model(vocab, width, eps, layers, scale=1.7, logit_scale=0.8, cap=9.0):
    listed = []
    for (kind, mixer), mlp, *owner in layers:
        entry = {"type": kind, "mixer": mixer, "mlp": mlp}
        if owner:
            entry["weights_of"] = owner[0]
        listed.append(entry)
    cfg = {
        "architecture": "Goguzen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
        "layers": listed, "logit_scale": logit_scale,
    }
    if cap is not None:
        cfg["logit_softcap"] = cap
    return cfg


BANDS = (4.0, 1.0, 4.0, 40)
A_PAIR = _both(_left(4, 2, 16, 0.25, 7, 0.4), _ssm(4, 16, 24, 2, 3, 2))
A_MOE = _moe(6, 2, 40, 0.9, (56, 1.3))
B_ATT = _attn(1, 1, 20, 12, 0.3, 6, 3, _rot(100.0, 6))
CONFIGS = {
    # a window with kept tokens that end inside a page, a layer that uses the one before it and one that uses the first
    "A": _model(97, 64, 1e-5, [
        (_attn(4, 2, 16, 24, 0.3, 19, 5, _rot(10000.0, 12, BANDS)), A_MOE),
        (A_PAIR, A_MOE),
        (A_PAIR, A_MOE, 1),
        (_attn(4, 2, 16, 24, 0.3, 19, 5, _rot(10000.0, 12, BANDS)), A_MOE, 0),
        (A_PAIR, None),
    ]),
    # one head everywhere, widths no kernel likes, odd experts, every expert chosen, no shared one, no cap, one tap
    "B": _model(61, 36, 1e-6, [
        (_both(_left(1, 1, 20, 0.2, 3, -0.2), _ssm(1, 20, 10, 1, 6, 1)), _moe(3, 3, 27, 0.7)),
        (B_ATT, _moe(2, 1, 18, 2.0, (11, 0.8))),
        (_both(_left(3, 1, 7, 0.5), _ssm(3, 10, 7, 3, 1, 5)), None),
        (B_ATT, _moe(2, 1, 18, 2.0, (11, 0.8)), 1),
    ], scale=2.0, logit_scale=1.0, cap=None),
    # as many key/value heads as heads, every dim turns, a window of one page and more kept tokens than it holds
    "C": _model(128, 48, 1e-5, [
        (_attn(3, 3, 48, 64, 0.15, 4, 9, _rot(20000.0, 48)), _moe(8, 3, 64, 1.0, (64, 1.0))),
        (_both(_left(6, 3, 32, 0.2, 16, 0.3), _ssm(6, 16, 32, 2, 4, 3)), _moe(5, 1, 32, 1.5)),
        (_attn(8, 2, 32, 32, 0.2, 1, 1, _rot(500000.0, 16, (8.0, 1.0, 2.0, 32))), None),
        (_attn(2, 1, 24, 24, 0.25), _moe(8, 2, 24, 0.5, (40, 1.1))),
    ]),
    # long requests: decode partitions, many key tiles, kept tokens over several of them, states over many chunks
    "D": _model(80, 64, 1e-5, [
        (_attn(4, 2, 32, 32, 0.3, 150, 70, _rot(10000.0, 32, (8.0, 1.0, 4.0, 64))), _moe(4, 2, 64, 1.0, (32, 1.2))),
        (_both(_left(4, 2, 32, 0.25, 100, 0.3), _ssm(4, 32, 40, 2, 4, 2)), _moe(4, 2, 64, 1.0, (32, 1.2))),
        (_both(_left(4, 2, 32, 0.25, 100, 0.3), _ssm(4, 32, 40, 2, 4, 2)), _moe(4, 2, 64, 1.0, (32, 1.2)), 1),
        (_attn(4, 1, 64, 64, 0.2, 40, 17, _rot(10000.0, 64)), None),
    ]),
}
BLOCK = {"A": 16, "B": 8, "C": 4, "D": 16}
LENGTHS = {"A": (1, 9, 50, 83, 37, 64), "B": (2, 19, 35, 66, 45), "C": (5, 17, 140, 70), "D": (660, 341)}


def make_weights(cfg: dict, seed: int) -> dict[str, torch.Tensor]:
    """bfloat16 tensors by the design's checkpoint names, larger than an initialisation would be."""
    g = torch.Generator().manual_seed(seed)
    width = cfg["width"]

    def normal(*shape, std, mean=0.0):
        return (torch.randn(shape, generator=g) * std + mean).to(torch.bfloat16)

    def matrix(rows, cols, gain=1.0):
        return normal(rows, cols, std=gain / math.sqrt(cols))

    w = {
        "embed": normal(cfg["vocab"], width, std=1.0), "final.norm": normal(width, std=0.2, mean=1.0),
        "head": matrix(cfg["vocab"], width, 1.5),
    }

    def expert(name, ff):
        w[name + ".gate"], w[name + ".up"] = matrix(ff, width, 1.5), matrix(ff, width, 1.5)
        w[name + ".down"] = matrix(width, ff)

    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m = f"l{i}.", layer["mixer"]
        w[p + "norm1"] = normal(width, std=0.2, mean=1.0)
        if layer["type"] == "attention":
            q, k = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
            w[p + "mix.q"], w[p + "mix.k"], w[p + "mix.v"] = matrix(q, width), matrix(k, width), matrix(m["kv_heads"] * m["vdim"], width)
            w[p + "mix.q.norm"], w[p + "mix.k.norm"] = normal(q, std=0.2, mean=1.0), normal(k, std=0.2, mean=1.0)
            w[p + "mix.sink"] = normal(m["heads"], std=1.0, mean=0.5)
            w[p + "mix.o"] = matrix(width, m["heads"] * m["vdim"])
        else:
            a, b = m["left"], m["right"]
            w[p + "mix.left.q"], w[p + "mix.left.k"] = matrix(a["heads"] * a["dim"], width), matrix(a["kv_heads"] * a["dim"], width)
            w[p + "mix.left.q.norm"], w[p + "mix.left.k.norm"] = normal(a["dim"], std=0.2, mean=1.0), normal(a["dim"], std=0.2, mean=1.0)
            w[p + "mix.left.sink"] = normal(a["heads"], std=1.0, mean=0.5)
            w[p + "mix.left.o"] = matrix(width, a["heads"] * a["dim"])
            w[p + "mix.left.out"], w[p + "mix.right.out"] = normal(width, std=0.2, mean=1.0), normal(width, std=0.2, mean=0.8)
            inner, bc = b["heads"] * b["vdim"], 2 * b["groups"] * b["state"]
            w[p + "mix.right.in"] = matrix(2 * inner + bc + b["heads"], width, 1.5)
            w[p + "mix.right.conv"] = normal(inner + bc, b["conv"], std=0.6)
            w[p + "mix.right.conv.b"] = normal(inner + bc, std=0.2)
            w[p + "mix.right.dt_bias"] = normal(b["heads"], std=0.7, mean=-2.0)
            w[p + "mix.right.A_log"] = normal(b["heads"], std=0.7)
            w[p + "mix.right.D"] = normal(b["heads"], std=0.5, mean=0.7)
            w[p + "mix.right.norm"] = normal(inner, std=0.2, mean=1.0)
            w[p + "mix.right.o"] = matrix(width, inner)
        f = layer["mlp"]
        if f is not None:
            w[p + "norm2"] = normal(width, std=0.2, mean=1.0)
            w[p + "mlp.router"] = matrix(f["router"]["experts"], width, 3.0)
            w[p + "mlp.router.b"] = normal(f["router"]["experts"], std=0.5)
            for e in range(f["router"]["experts"]):
                expert(f"{p}mlp.e{e}", f["expert"]["ff"])
            if f.get("shared"):
                expert(p + "mlp.shared", f["shared"]["ff"])
    return w


def write_model(tmp_path, name: str, cfg: dict, weights: dict) -> Path:
    folder = Path(tmp_path) / name
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    save_state_dict(folder / "model.safetensors", weights)
    return folder


def make_dir(tmp_path, which: str, seed: int = 3):
    cfg = CONFIGS[which]
    weights = make_weights(cfg, seed)
    return write_model(tmp_path, f"goguzen{which}", cfg, weights), cfg, weights


def _f64(weights):
    return {k: v.to(torch.float64) for k, v in weights.items()}


def _ops(backend: str, dtype: torch.dtype):
    if backend == "double":
        return TorchOps(dtype, "cpu")
    from mini_llm_runtime_amd.kernels.ops import HipOps

    return HipOps(dtype, "cuda")


CASES = [
    pytest.param("double", torch.float32, id="double-f32"),
    pytest.param("hip", torch.float32, id="hip-f32", marks=pytest.mark.gpu),
    pytest.param("hip", torch.bfloat16, id="hip-bf16", marks=pytest.mark.gpu),
]
GPU_CASES = [
    pytest.param(torch.float32, id="f32", marks=pytest.mark.gpu),
    pytest.param(torch.bfloat16, id="bf16", marks=pytest.mark.gpu),
]


CLOSE_CALL = 0.06  # router logits (of a size of some 3) that bfloat16 activations may order either way


def _compare(got, requests, weights, cfg, dtype, f32_bound=3e-4, row_bound=6e-2, together=3e-2, worst_row=4.0):
    """float32: every value within 3e-4 of the logits' size, or within 4 times of what rounding the inputs of the
    products to float32 does to the worst row.  bfloat16: all rows together within 3 % (relative L2, the mean over the
    vocabulary taken off) or twice what rounding alone does; every row within 6 %, but for a few (one in twenty, and as
    many as rounding alone puts beyond 6 %) that may be off by up to `worst_row` times what rounding alone does to the
    worst row of their request, and rows in which some choice of experts is closer than CLOSE_CALL, where rounding may
    choose another expert (which is another row altogether).  A wrong key, page, slot or state changes most rows, by
    half and more."""
    assert got, "no logits came back"
    w64 = _f64(weights)
    num = den = num_alone = 0.0
    loose = rows = loose_alone = 0
    for rid, toks in requests.items():
        margins: list = []
        ref, _ = plain.forward(cfg, w64, toks, margins=margins)
        close = torch.stack(margins).min(0).values < CLOSE_CALL if margins else torch.zeros(len(toks), dtype=torch.bool)
        ref = ref - ref.mean(-1, keepdim=True)
        size = float(ref.pow(2).mean().sqrt())
        coarse, _ = plain.forward(cfg, w64, toks, round_to=dtype)
        coarse = coarse - coarse.mean(-1, keepdim=True)
        bound32 = max(f32_bound * size, 4.0 * float((coarse - ref).abs().max()))
        alone = (coarse - ref).pow(2).sum(-1).sqrt() / ref.pow(2).sum(-1).sqrt()
        loose_alone += int((alone >= row_bound).sum())
        for pos in range(len(toks)):
            row = got[(rid, pos)].double()
            assert torch.isfinite(row).all(), f"{rid}:{pos} is not finite"
            diff = row - row.mean() - ref[pos]
            if dtype == torch.float32:
                worst = float(diff.abs().max())
                assert worst < bound32, f"{rid}:{pos}: off by {worst:.3e} of {size:.3e}"
                continue
            rows += 1
            rel = float(diff.pow(2).sum().sqrt() / ref[pos].pow(2).sum().sqrt())
            if rel >= row_bound and close[pos]:
                loose_alone += 1
                continue
            if rel >= row_bound:
                loose += 1
                assert rel < worst_row * max(float(alone.max()), row_bound), f"{rid}:{pos}: relative error {rel:.3e}, rounding alone up to {float(alone.max()):.3e}"
                continue
            num += float(diff.pow(2).sum())
            num_alone += float((coarse[pos] - ref[pos]).pow(2).sum())
            den += float(ref[pos].pow(2).sum())
    if dtype != torch.float32:
        assert loose <= 0.05 * rows + 1 + 1.5 * loose_alone, f"{loose} of {rows} rows are off by more than {row_bound}, {loose_alone} by rounding alone"
        assert (num / den) ** 0.5 < max(together, 2.0 * (num_alone / den) ** 0.5), f"relative error of all rows {(num / den) ** 0.5:.3e}"


def _requests(which: str) -> dict[str, list[int]]:
    vocab = CONFIGS[which]["vocab"]
    return {f"r{i}": random_tokens(n, vocab, 50 + i) for i, n in enumerate(LENGTHS[which])}


# ---- configuration and model --------------------------------------------------------------------------

def test_config_reads_every_layer_by_itself():
    c = config_from_dict(CONFIGS["A"])
    assert isinstance(c, GoguzenConfig)
    assert [l.mixer.kind for l in c.layers] == ["attention", "parallel", "parallel", "attention", "parallel"]
    assert [l.weights_of for l in c.layers] == [None, None, 1, 0, None] and [c.owner_of(i) for i in range(5)] == [0, 1, 1, 0, 4]
    a = c.layers[0].mixer
    assert (a.window, a.keep_first, a.vdim, a.rot.scaling.original) == (19, 5, 24, 40.0)
    b = c.layers[1].mixer
    assert (b.left.temp_every, b.left.temp_coef, b.right.conv, b.right.norm_groups) == (7.0, 0.4, 3, 2)
    m = c.layers[0].mlp
    assert (m.experts, m.top, m.expert.ff, m.expert.limit, m.shared.ff, m.shared.limit) == (6, 2, 40, 0.9, 56, 1.3)
    assert c.layers[4].mlp is None and (c.embedding_scale, c.logit_scale, c.logit_softcap) == (1.7, 0.8, 9.0)
    assert GoguzenConfig.from_dict(c.to_dict()) == c
    plainer = config_from_dict(CONFIGS["C"]).layers[3].mixer
    assert plainer.window is None and plainer.rot is None
    assert GoguzenConfig.from_dict(config_from_dict(CONFIGS["B"]).to_dict()).logit_softcap is None


@pytest.mark.parametrize(
    "change",
    [
        lambda c: c["layers"][0]["mixer"].pop("scale"),
        lambda c: c["layers"][0].update(type="convolution"),
        lambda c: c["layers"][4]["mixer"]["left"].update(kv_heads=3),  # four heads on three
        lambda c: c["layers"][4]["mixer"]["left"].update(vdim=8),  # values that are keys have their size
        lambda c: c["layers"][4]["mixer"]["left"]["q_temp"].update(every=0),
        lambda c: c["layers"][4]["mixer"].pop("right"),
        lambda c: c["layers"][4]["mixer"]["right"].update(groups=3),
        lambda c: c["layers"][4]["mixer"]["right"].update(norm_groups=7),
        lambda c: c["layers"][0]["mixer"]["rot"].update(dims=40),  # more than a head has
        lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5),
        lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(low=8.0),  # above high
        lambda c: c["layers"][0]["mixer"]["mask"].update(size=0),
        lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=-1),
        lambda c: c["layers"][0]["mlp"].update(kind="dense"),
        lambda c: c["layers"][0]["mlp"]["router"].update(top=9),
        lambda c: c["layers"][0]["mlp"]["expert"].update(limit=0.0),
        lambda c: c["layers"][3]["mixer"].update(scale=0.4),  # not equal to the layer whose tensors it uses
        lambda c: c["layers"][2].update(weights_of=2),
        lambda c: c["layers"][2].update(weights_of=7),
        lambda c: c.update(layers=[]),
        lambda c: c.update(logit_softcap=-1.0),
    ],
)
def test_config_refuses_what_does_not_fit(change):
    cfg = copy.deepcopy(CONFIGS["A"])
    change(cfg)
    with pytest.raises(ConfigError):
        config_from_dict(cfg)


def test_model_is_built_from_the_framework_parts():
    from mini_llm_runtime_amd.parts.attention import GQAAttention
    from mini_llm_runtime_amd.parts.block import PreNormBlock
    from mini_llm_runtime_amd.parts.feed_forward import ClampedGLU, RoutedExperts
    from mini_llm_runtime_amd.parts.pooled_attention import PooledWindowAttention
    from mini_llm_runtime_amd.parts.side_by_side import SideBySide
    from mini_llm_runtime_amd.parts.state_space import StateSpace

    model = build_model(config_from_dict(CONFIGS["A"]))
    assert all(isinstance(layer, PreNormBlock) for layer in model.layers)
    # five listed layers, three of which have tensors; every listed one is a site of its own
    assert [type(layer.mixer) for layer in model.layers] == [PooledWindowAttention, SideBySide, SideBySide]
    assert [entry.layer for entry in model.spec.order] == [0, 1, 1, 0, 2] and model.num_sites == 5
    assert [model.cache_site_of(i) for i in range(5)] == [0, 1, 2, 3, 4]
    pair = model.layers[1].mixer
    assert isinstance(pair.members["left"], GQAAttention) and isinstance(pair.members["right"], StateSpace)
    assert pair.members["left"].param_specs()["qkv_weight"].shape == (96, 64)  # queries and keys, no values
    ff = model.layers[0].feed_forward
    assert isinstance(ff, RoutedExperts) and isinstance(ff.shared, ClampedGLU) and model.layers[2].feed_forward is None
    assert not model.spec.tie_word_embeddings and model.replayable and model.splittable
    specs = model.site_cache_specs()
    assert specs[0] == specs[3] and (specs[0].window, specs[0].keep_first) == (19, 5)  # one pool, two sites
    assert {n: type(s).__name__ for n, s in specs[2].members.items()} == {"left": "PagedKVSpec", "right": "CompositeSpec"}
    assert {name for name in model.param_specs() if name.startswith("layers.1.mixer.") and "out_norm" in name} == {
        "layers.1.mixer.left_out_norm", "layers.1.mixer.right_out_norm"}


def test_joint_input_product_and_outputs_apart(tmp_path):
    """A parallel layer multiplies its input once (both members' rows under each other) and norms two outputs."""
    folder, cfg, weights = make_dir(tmp_path, "A")
    _, model, cache, runner = make_runner(folder, TorchOps(torch.float32, "cpu"), block_size=16, num_blocks=4, max_requests=1)
    pair = model.layers[1].mixer
    assert pair.in_weight.shape == (96 + (2 * 64 + 2 * 2 * 24 + 4), 64) and pair.members["left"].in_weight is None
    assert pair.members["right"].o_weight.shape == (64, 64) and pair.o_weight is None
    stored = sum(t.numel() * 4 for t in weights.values())
    # everything once (the smaller things the parts make of them are not counted as weights)
    assert abs(model.weight_bytes() - stored) < 0.02 * stored


# ---- mechanisms alone -----------------------------------------------------------------------------------

@pytest.mark.parametrize("scaling", [None, (4.0, 1.0, 4.0, 40), (8.0, 1.0, 1.0, 100), (2.0, 2.0, 32.0, 4096), (16.0, 0.5, 1.5, 9)])
def test_frequencies_in_bands(scaling):
    from mini_llm_runtime_amd.parts.position import RotaryEmbedding

    rot = _rot(10000.0, 32, scaling)
    part = RotaryEmbedding(48, rot["base"], rot["dims"], rot.get("scaling"))
    got = torch.from_numpy(part._inv_freq_host)
    torch.testing.assert_close(got, plain.rotary_frequencies(rot), rtol=1e-13, atol=0)
    assert part.amplitude == 1.0
    if scaling == (4.0, 1.0, 4.0, 40):  # all three bands are there
        f = 10000.0 ** (-torch.arange(0, 32, 2, dtype=torch.float64) / 32)
        kept, slowed = int((got == f).sum()), int(torch.isclose(got, f / 4.0, rtol=1e-13, atol=0.0).sum())
        assert kept > 0 and slowed > 0 and kept + slowed < 16
    with pytest.raises(ValueError):
        RotaryEmbedding(8, 10.0, 8, {"factor": 2.0, "low": 3.0, "high": 2.0, "original": 8})


def test_the_window_gives_pages_back_and_the_first_ones_stay():
    from mini_llm_runtime_amd.cache.manager import CacheManager

    spec = PagedKVSpec(1, 16, 10, keep_first=5)
    manager = CacheManager([spec], block_size=4, num_blocks=12, max_requests=2, dtype=torch.float32, device="cpu")
    group = manager.groups[0]
    assert group.kept_blocks == 2  # positions 0..4 lie in pages 0 and 1
    assert group.lifetime_blocks(1000, 1) == 2 + -(-(9 + 1) // 4) + 1 and group.lifetime_blocks(6, 1) == 2
    assert manager.try_create_reserved("a", 40, 7)
    held = []
    for n in (7, 7, 7, 7, 7, 5):
        manager.begin_step([("a", n)])
        manager.commit_step()
        manager.check_invariants()
        request = manager.get_request("a")
        live = [i for i, b in enumerate(request.tables[0]) if b >= 0]
        first = max(0, request.num_tokens - 9)  # the next query sees positions from here on
        assert live == sorted(set(range(0, 2)) & set(range(len(request.tables[0]))) | set(range(first // 4, len(request.tables[0]))))
        held.append(len(live))
    assert max(held) <= 6
    manager.release_request("a")
    assert group.allocator.free_count == group.num_blocks and group.allocator.reserved_count == 0
    with pytest.raises(ValueError):
        PagedKVSpec(1, 16, keep_first=3)  # goes with a window


def _tolerance(dtype):
    return dict(rtol=2e-5, atol=2e-5) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2)


def _step_context(lengths, starts, ops):
    cu = [0]
    for n in lengths:
        cu.append(cu[-1] + n)
    dev = ops.device
    entry = [r for r, n in enumerate(lengths) for _ in range(n)]
    position = [s + i for s, n in zip(starts, lengths) for i in range(n)]
    return SimpleNamespace(
        num_entries=len(lengths), cu_q=torch.tensor(cu, dtype=torch.int32, device=dev),
        q_starts=torch.tensor(starts, dtype=torch.int32, device=dev),
        token_entry=torch.tensor(entry, dtype=torch.int32, device=dev),
        positions=torch.tensor(position, dtype=torch.int32, device=dev),
        context_lens=torch.tensor([s + n for s, n in zip(starts, lengths)], dtype=torch.int32, device=dev),
        max_context_len=max(s + n for s, n in zip(starts, lengths)),
    )


MASKS = [(10, 3), (75, 7), (64, 64), (100, 33), (5, 90), (1, 1), (300, 17), (40, 200), (16, 16)]


@pytest.mark.parametrize("dtype", GPU_CASES)
@pytest.mark.parametrize("window,keep", MASKS)
@pytest.mark.parametrize("heads,kv,dim,lengths,starts,wide", [
    (4, 2, 64, [1, 1, 1, 1], [700, 0, 33, 96], False),  # decoded tokens: one partition and several
    (2, 1, 32, [130, 1, 2], [0, 300, 165], False),  # prompt tiles beside decoded tokens
    (2, 2, 48, [70, 9], [400, 60], False),
    (1, 1, 128, [300, 40], [333, 0], True),
    (8, 2, 24, [5, 1], [120, 203], False),  # no multiple of 16: the plain kernel
])
def test_window_beside_kept_first_tokens(dtype, window, keep, heads, kv, dim, lengths, starts, wide):
    """Every attention kernel, with what no query of the step sees not there at all (no page) or NaN; against the
    stand-in's formulas."""
    from mini_llm_runtime_amd.kernels.plans import attention_plan
    from mini_llm_runtime_amd.kernels.tuning import KernelTuning
    from mini_llm_runtime_amd.parts.context import PlanInput

    hip, double = _ops("hip", dtype), TorchOps(dtype, "cpu")
    if wide:
        hip.tuning = KernelTuning(wide_attention_groups=1)
    g = torch.Generator().manual_seed(heads * dim + window)
    block = 16
    tokens, contexts = sum(lengths), [s + n for s, n in zip(starts, lengths)]
    need = [-(-c // block) for c in contexts]
    pages = sum(need) + 1
    order = torch.randperm(pages, generator=g).tolist()
    table = torch.full((len(lengths), max(need)), -1, dtype=torch.int32)
    keys = torch.full((pages, kv, block, dim), float("nan"), dtype=dtype)
    values = torch.full((pages, kv, dim, block), float("nan"), dtype=dtype)
    for r, (s, c) in enumerate(zip(starts, contexts)):
        for page in range(need[r]):
            first, last = page * block, page * block + block - 1
            if first >= keep and last < s - window + 1:
                continue  # behind every query's window and not kept: given back
            table[r, page] = order.pop()
            n = min(block, c - first)  # the rest of the last page was never written
            keys[table[r, page], :, :n] = torch.randn(kv, n, dim, generator=g).to(dtype)
            values[table[r, page], :, :, :n] = torch.randn(kv, dim, n, generator=g).to(dtype)
    q = torch.randn(tokens, heads * dim, generator=g).to(dtype)
    sinks = torch.randn(heads, generator=g)
    kw = dict(num_heads=heads, num_kv_heads=kv, head_dim=dim, block_size=block, scale=0.4, window=window, keep_first=keep)
    want = double.paged_attention(q, keys, values, table, _step_context(lengths, starts, double), sinks=sinks, **kw)
    shape = attention_plan(PlanInput(np.asarray(lengths), np.asarray(starts), max(contexts)))
    dev = {k: torch.from_numpy(v).to(torch.int32).cuda() for k, v in shape.arrays.items()}
    bound = dict(rtol=2e-5, atol=2e-5) if dtype == torch.float32 else dict(rtol=2e-2, atol=1e-2)
    for partition in (64, 256):
        hip.decode_partition = partition
        got = hip.paged_attention(
            q.cuda(), keys.cuda(), values.cuda(), table.cuda(), _step_context(lengths, starts, hip), sinks=sinks.cuda(),
            plan=SimpleNamespace(**shape.sizes, **dev), **kw,
        )
        torch.testing.assert_close(got.float().cpu(), want.float(), **bound)


@pytest.mark.parametrize("dtype", GPU_CASES)
@pytest.mark.parametrize("heads,kv,dim,block,column", [(4, 2, 32, 8, 0), (1, 1, 20, 4, 7), (6, 3, 40, 16, 100), (2, 1, 128, 16, 3)])
def test_keys_that_are_values_and_queries_that_grow(dtype, heads, kv, dim, block, column):
    hip, double = _ops("hip", dtype), TorchOps(dtype, "cpu")
    g = torch.Generator().manual_seed(heads + dim)
    tokens = 37
    pages = -(-tokens // block) + 1
    D = -(-dim // 16) * 16
    projected = torch.randn(tokens, column + (heads + kv) * dim + 5, generator=g) * 2.0
    slots = torch.randperm(pages * block, generator=g)[:tokens].to(torch.int32)
    slots[3] = -1
    # on, before and behind multiples of the length in which queries grow, near and far
    positions = torch.tensor([0, 1, 5, 6, 7, 12, 13, 14, 20, 9999, 1000000] + list(range(100, 126)), dtype=torch.int32)
    weights = [(1 + 0.4 * torch.randn(dim, generator=g)).to(dtype) for _ in range(2)]
    results = []
    for ops in (double, hip):
        to = (lambda t: t.cuda()) if ops is hip else (lambda t: t)
        keys = to(torch.zeros(pages, kv, block, D, dtype=dtype))
        values = to(torch.zeros(pages, kv, D, block, dtype=dtype))
        q, gate, kept = ops.head_norm_rope_write(
            to(projected), heads=heads, kv_heads=kv, head_dim=dim, value_dim=dim, kernel_dim=D, eps=1e-5, rotation=None,
            slot_mapping=to(slots), key_pages=keys, value_pages=values, block_size=block, weights=tuple(to(w) for w in weights),
            values_are_keys=True, temperature=(to(positions), 7.0, 0.45), projected_column=column,
        )
        assert gate is None and kept is None
        results.append([t.float().cpu() for t in (q, keys, values)])
    for a, b in zip(*results):
        torch.testing.assert_close(b, a, **_tolerance(dtype))
    # the stand-in itself: the growth of one query by the formula, a stored value is the key's plain sum
    rows = projected[:, column : column + dim].double()
    want = plain.rms_norm(rows, weights[0].double(), 1e-5) * plain.query_temperature(positions, 7.0, 0.45)[:, None]
    torch.testing.assert_close(results[0][0][:, :dim].double(), want, **_tolerance(dtype))
    at = int(slots[10])
    torch.testing.assert_close(
        results[0][2][at // block, 0, :dim, at % block], projected[10, column + heads * dim : column + (heads + 1) * dim].to(dtype).float()
    )


@pytest.mark.parametrize("dtype", GPU_CASES)
@pytest.mark.parametrize("rows,hidden", [(1, 64), (5, 70), (70, 256), (3, 2048), (300, 1000), (2, 4096), (9, 4100)])
@pytest.mark.parametrize("slices", [(0, 0), (3, 0), (0, 2), (9, 4)])
def test_two_outputs_normed_before_they_are_added(dtype, rows, hidden, slices):
    from mini_llm_runtime_amd.kernels.pending import NormedDelta

    hip, double = _ops("hip", dtype), TorchOps(dtype, "cpu")
    g = torch.Generator().manual_seed(rows + hidden)
    x = torch.randn(rows, hidden, generator=g)
    ys = [
        torch.randn(s, rows, hidden, generator=g) if s else (torch.randn(rows, hidden, generator=g) * 3.0).to(dtype)
        for s in slices
    ]
    ws = [(1 + 0.3 * torch.randn(hidden, generator=g)).to(dtype) for _ in range(2)]
    nw = (1 + 0.3 * torch.randn(hidden, generator=g)).to(dtype)
    for scales, second in (((0.5, 0.5), True), ((0.3, -1.2), True), ((0.7, 1.0), False)):
        outs = []
        for ops in (double, hip):
            to = (lambda t: t.cuda()) if ops is hip else (lambda t: t.clone())
            own = to(x)
            owed = NormedDelta(to(ys[0]), to(ws[0]), 1e-5, (to(ys[1]), to(ws[1])) if second else None, *scales)
            h = ops.rmsnorm(own, to(nw), 1e-6, delta=owed)
            taken = ops.settle(ops.gather_rows(owed, torch.tensor([rows - 1], dtype=torch.int32, device=own.device)))
            outs.append((own.cpu(), h.float().cpu(), taken.float().cpu()))
        torch.testing.assert_close(outs[1][0], outs[0][0], rtol=1e-5, atol=1e-5)
        torch.testing.assert_close(outs[1][1], outs[0][1], **_tolerance(dtype))
        torch.testing.assert_close(outs[1][2], outs[0][2], rtol=1e-5, atol=1e-5)
        torch.testing.assert_close(outs[0][0][-1] - x[-1], outs[0][2][0], rtol=1e-4, atol=1e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("experts,top", [(1, 1), (13, 4), (7, 7), (64, 6), (200, 8)])
def test_softmax_over_the_chosen_logits(experts, top):
    hip, double = _ops("hip", torch.float32), TorchOps(torch.float32, "cpu")
    g = torch.Generator().manual_seed(experts)
    z = torch.randn(23, experts, generator=g) * 3.0
    z[1] += 300.0  # far from zero: only differences count
    z[2] = z[2] * 60.0  # weights of nothing and all
    z[3, :] = 1.25  # equal logits: the first ones, equal weights
    kw = dict(top=top, groups=1, keep_groups=1, scale=1.0, scores="chosen_softmax")
    ids, weights = hip.route_experts(z.cuda(), None, **kw)
    want_ids, want = double.route_experts(z, None, **kw)
    assert torch.equal(ids.cpu(), want_ids)
    torch.testing.assert_close(weights.cpu(), want, rtol=1e-5, atol=1e-7)
    dense = torch.zeros(23, experts, dtype=torch.float64).scatter(1, ids.cpu().long(), weights.cpu().double())
    keep = [i for i in range(23) if i != 3]
    torch.testing.assert_close(dense[keep], plain.route(z.double(), top)[keep], rtol=1e-5, atol=1e-7)


@pytest.mark.parametrize("dtype", GPU_CASES)
@pytest.mark.parametrize("tokens,hidden,inner,experts,top,side", [
    (3, 64, 24, 6, 2, 40),  # few rows an expert: straight from memory
    (5, 1024, 520, 4, 2, 136),  # an expert's matrix of a megabyte: whole lines through LDS
    (130, 64, 40, 4, 2, 0),  # tiles of 64 rows
    (700, 136, 64, 3, 2, 72),  # tiles of 128 rows
    (9, 36, 27, 3, 3, 11),  # an odd size, gated behind its product
    (4, 33, 18, 2, 1, 10),  # slices that do not start at a multiple of 16 bytes
    (1, 2048, 64, 8, 4, 4096),  # the product beside them in slices of k
])
def test_clamped_experts_and_a_product_beside_them(dtype, tokens, hidden, inner, experts, top, side):
    hip = _ops("hip", dtype)
    g = torch.Generator().manual_seed(tokens + inner)
    h = torch.randn(tokens, hidden, generator=g).to(dtype)
    gate, up = ((torch.randn(experts, inner, hidden, generator=g) * 2.0 / math.sqrt(hidden)).to(dtype) for _ in range(2))
    down = (torch.randn(experts, hidden, inner, generator=g) / math.sqrt(inner)).to(dtype)
    ids = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(tokens)]).to(torch.int32)
    weights = torch.rand(tokens, top, generator=g)
    woven = inner % 2 == 0
    if woven:
        first = torch.stack([gate.view(experts, -1, 2, hidden), up.view(experts, -1, 2, hidden)], 2)
    else:
        first = torch.stack([gate, up], 1)
    first = first.reshape(experts * 2 * inner, hidden).contiguous()
    beside = None
    if side:
        beside = (torch.randn(tokens, side, generator=g).to(dtype), (torch.randn(hidden, side, generator=g) / math.sqrt(side)).to(dtype))
    limit, alpha = 0.8, 1.702
    got = hip.expert_products(
        h.cuda(), first.cuda(), down.reshape(experts * hidden, inner).contiguous().cuda(), ids.cuda(), weights.cuda(),
        experts=experts, activation="clamped_glu", glu=(limit, alpha), woven=woven,
        **({"beside": tuple(t.cuda() for t in beside)} if side else {}),
    )
    assert got.shape[0] >= top + bool(side) and got.shape[1:] == (tokens, hidden)
    h64 = h.double()
    want = torch.zeros(tokens, hidden, dtype=torch.float64)
    for e in range(experts):
        a = torch.clamp(h64 @ gate[e].double().T, max=limit)
        u = torch.clamp(h64 @ up[e].double().T, -limit, limit)
        a = (a * torch.sigmoid(alpha * a) * (u + 1.0))
        for j in range(top):
            rows = (ids[:, j] == e).nonzero()[:, 0]
            want[rows] += weights[rows, j, None].double() * (a[rows] @ down[e].double().T)
    if side:
        want += beside[0].double() @ beside[1].double().T
    torch.testing.assert_close(got.sum(0).double().cpu(), want, **(dict(rtol=2e-5, atol=2e-5) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2)))


# ---- one layer of each kind ----------------------------------------------------------------------------------

ONE_LAYER = {
    "attention": (_attn(4, 2, 16, 24, 0.3, 12, 3, _rot(1000.0, 8, BANDS)), None),
    "attention-full": (_attn(2, 2, 8, 8, 0.4), None),
    "attention-no-kept": (_attn(2, 1, 16, 16, 0.4, 9, 0, _rot(1000.0, 16)), None),
    "parallel": (_both(_left(4, 2, 16, 0.3, 5, 0.5), _ssm(4, 12, 20, 2, 4, 2)), None),
    "parallel-steady": (_both(_left(2, 2, 12, 0.3), _ssm(2, 8, 12, 1, 2, 4)), None),
    "mixture": (_attn(1, 1, 8, 8, 0.3), _moe(5, 2, 40, 0.8, (24, 1.2))),
    "mixture-alone": (_attn(1, 1, 8, 8, 0.3), _moe(4, 3, 16, 0.6)),
    "mixture-odd": (_attn(1, 1, 8, 8, 0.3), _moe(3, 1, 33, 0.8, (17, 0.4))),
}


@pytest.mark.parametrize("backend,dtype", CASES)
@pytest.mark.parametrize("kind", list(ONE_LAYER))
def test_one_layer_of_each_kind(tmp_path, kind, backend, dtype):
    cfg = _model(50, 32, 1e-5, [ONE_LAYER[kind]])
    weights = make_weights(cfg, 21)
    folder = write_model(tmp_path, "one", cfg, weights)
    requests = {"a": random_tokens(75, 50, 3), "b": random_tokens(1, 50, 4)}
    _, _, cache, runner = make_runner(folder, _ops(backend, dtype), block_size=8, num_blocks=10, max_requests=2)
    cache.poison()
    for family in (schedules.whole, lambda r: schedules.bulk_then_tail(r, tail=9), schedules.portions):
        _compare(schedules.run_schedule(runner, cache, family(requests)), requests, weights, cfg, dtype)


# ---- keys far away, at page borders and at the edges of what is seen ----------------------------------------------

def _needle_model(dim: int, mixer):
    """One head whose keys are the normed stream and whose queries are the normed stream with its halves swapped;
    token 39's embedding is token 38's with its halves swapped.  Token 39's query then equals the key of token 38 and of
    nothing else, and ONE such key, however far, takes nearly all of the weight."""
    cfg = _model(40, dim, 1e-6, [(mixer, None)], scale=1.0, logit_scale=1.0, cap=30.0)
    weights = make_weights(cfg, 2)
    eye = torch.eye(dim).to(torch.bfloat16)
    ones = torch.ones(dim, dtype=torch.bfloat16)
    p = "l0.mix." if mixer[0] == "attention" else "l0.mix.left."
    weights["l0.norm1"] = ones
    weights[p + "q"], weights[p + "q.norm"] = eye.roll(dim // 2, dims=0).contiguous(), ones
    weights[p + "k"], weights[p + "k.norm"] = eye.clone(), ones.clone()
    weights["embed"][39] = weights["embed"][38].roll(dim // 2)
    return cfg, weights


def _needle_tokens(length, marked):
    toks = [1 + (i % 30) for i in range(length)]  # ids 1..30 in turn
    toks[marked] = 38
    toks[-1] = 39  # asks for the marked one
    return toks


def _needle_steps(toks):
    cut = max(1, len(toks) - 5)
    return (
        schedules.whole({"a": toks}),  # the asking token at the end of a prompt
        schedules.bulk_then_tail({"a": toks}, tail=3),  # decoded alone
        schedules.bulk_then_tail({"a": toks}, tail=40),  # behind many decoded tokens, pages given back in between
        schedules.portions({"a": toks}, sizes=(cut - 1, 2, 3, 2)),  # at the end of a short portion
    )


def _ask(tmp_path, cfg, weights, toks, backend, dtype, block):
    folder = write_model(tmp_path, "needle", cfg, weights)
    want = plain.forward(cfg, _f64(weights), toks)[0][-1]
    _, _, cache, runner = make_runner(folder, _ops(backend, dtype), block_size=block, num_blocks=-(-len(toks) // block), max_requests=1)
    cache.poison()
    for steps in _needle_steps(toks):
        got = schedules.run_schedule(runner, cache, steps)
        row = got[("a", len(toks) - 1)].double()
        err = float((row - want).abs().max())
        assert err < (1e-4 if dtype == torch.float32 else 5e-2) * float(want.abs().max()), err


@pytest.mark.parametrize("backend,dtype", CASES)
@pytest.mark.parametrize("length,marked", [(70, 0), (200, 15), (700, 16), (131, 63), (97, 95)])
def test_one_far_key_that_takes_the_weight(tmp_path, backend, dtype, length, marked):
    if backend == "double" and length > 300:
        pytest.skip("the CPU stand-in is slow at this size")
    cfg, weights = _needle_model(32, _both(_left(1, 1, 32, 1.0, 50, 0.3), _ssm(1, 8, 4, 1, 2, 1)))
    toks = _needle_tokens(length, marked)
    other = list(toks)
    other[marked] = 37
    w64 = _f64(weights)
    with_key, without = plain.forward(cfg, w64, toks)[0][-1], plain.forward(cfg, w64, other)[0][-1]
    assert float((with_key - without).abs().max()) > 0.2 * float(with_key.abs().max()), "the oracle does not see the key"
    _ask(tmp_path, cfg, weights, toks, backend, dtype, 16)


@pytest.mark.parametrize("backend,dtype", CASES)
@pytest.mark.parametrize("block", [4, 16])
@pytest.mark.parametrize("length,window,keep", [(70, 20, 5), (131, 33, 16), (97, 1, 17), (90, 16, 1), (150, 64, 40), (60, 48, 30)])
def test_keys_just_inside_and_just_outside(tmp_path, backend, dtype, length, window, keep, block):
    """The marked key at the first and last place that is seen and at their neighbours that are not; where it is not
    seen, an oracle whose edge is off by one sees it."""
    asks = length - 1
    rot = _rot(1e9, 4)  # positions enter, but too slowly to hide the key
    cfg, weights = _needle_model(32, _attn(1, 1, 32, 32, 1.0, window, keep, rot))
    w64 = _f64(weights)
    for marked, seen, off in (
        (asks - window + 1, True, {"size": window - 1, "keep_first": keep}),
        (asks - window, False, {"size": window + 1, "keep_first": keep}),
        (keep - 1, True, {"size": window, "keep_first": keep - 1}),
        (keep, False, {"size": window, "keep_first": keep + 1}),
    ):
        inside = asks - marked < window or marked < keep
        if marked == asks or inside != seen:
            continue  # both edges meet, or the key asks for itself
        toks = _needle_tokens(length, marked)
        wrong = copy.deepcopy(cfg)
        wrong["layers"][0]["mixer"]["mask"] = off
        right_row, wrong_row = plain.forward(cfg, w64, toks)[0][-1], plain.forward(wrong, w64, toks)[0][-1]
        wrong_sees = asks - marked < off["size"] or marked < off["keep_first"]
        if off["size"] and wrong_sees != seen:  # (where window and kept tokens overlap, one edge alone does not show)
            assert float((right_row - wrong_row).abs().max()) > 0.2 * float(right_row.abs().max()), (marked, "the edge does not show")
        _ask(tmp_path, cfg, weights, toks, backend, dtype, block)


@pytest.mark.parametrize("backend,dtype", CASES)
@pytest.mark.parametrize("kind", ["attention", "left"])
def test_a_sink_that_takes_most_of_the_weight(tmp_path, kind, backend, dtype):
    """A sink per head, one of them far above every score, one far below: left out, scaled or counted per partition it
    would show in every row."""
    mixer = _attn(2, 1, 16, 16, 0.3, 50, 4) if kind == "attention" else _both(_left(2, 1, 16, 0.3), _ssm(1, 8, 4, 1, 2, 1))
    cfg = _model(64, 32, 1e-6, [(mixer, None)], scale=0.3)  # the mixer's output is what the logits show
    weights = make_weights(cfg, 5)
    name = "l0.mix.sink" if kind == "attention" else "l0.mix.left.sink"
    weights[name] = torch.tensor([8.0, -8.0], dtype=torch.bfloat16)
    without = dict(weights, **{name: torch.tensor([-60.0, -60.0], dtype=torch.bfloat16)})
    toks = random_tokens(230, 64, 1)
    a, b = plain.forward(cfg, _f64(weights), toks)[0], plain.forward(cfg, _f64(without), toks)[0]
    assert float((a - b).abs().max()) > 0.2 * float(a.abs().max())
    folder = write_model(tmp_path, "sink", cfg, weights)
    _, _, cache, runner = make_runner(folder, _ops(backend, dtype), block_size=8, num_blocks=29, max_requests=1)
    cache.poison()
    for family in (schedules.whole, lambda r: schedules.bulk_then_tail(r, tail=30)):
        _compare(schedules.run_schedule(runner, cache, family({"a": toks})), {"a": toks}, weights, cfg, dtype)


@pytest.mark.parametrize("backend,dtype", CASES)
def test_a_state_that_never_forgets_through_one_slot(tmp_path, backend, dtype):
    """Decays held at one: the first tokens stay in the state (and, at the first places, in the convolution's carried
    inputs), so a state lost between two steps, or a slot cleared too late or not at all, shows at later positions.
    The layer runs twice with the same tensors: every run keeps its own."""
    mixer = _both(_left(1, 1, 8, 0.3), _ssm(2, 16, 24, 1, 4, 1))
    cfg = _model(64, 32, 1e-6, [(mixer, None), (mixer, None, 0)])
    weights = make_weights(cfg, 11)
    weights["l0.mix.right.A_log"] = torch.full((2,), -30.0, dtype=torch.bfloat16)  # decay exp(-1e-13 ..)
    folder = write_model(tmp_path, "keeper", cfg, weights)
    a = random_tokens(90, 64, 1)
    b = [(a[0] + 1) % 64] + a[1:]  # differs in the first token only
    w64 = _f64(weights)
    ref_a, ref_b = plain.forward(cfg, w64, a)[0], plain.forward(cfg, w64, b)[0]
    assert float((ref_a[3] - ref_b[3]).abs().max()) > 0.02 * float(ref_a[3].abs().max())
    assert float((ref_a[20] - ref_b[20]).abs().max()) > 1e-3 * float(ref_a[20].abs().max())
    _, _, cache, runner = make_runner(folder, _ops(backend, dtype), block_size=8, num_blocks=12, max_requests=1)
    for family in (schedules.whole, lambda r: schedules.bulk_then_tail(r, tail=40), schedules.portions):
        for name, toks in (("a", a), ("b", b), ("a", a)):  # one slot, used again and again
            got = schedules.run_schedule(runner, cache, family({name: toks}))
            _compare(got, {name: toks}, weights, cfg, dtype)


# ---- whole models under every schedule -------------------------------------------------------------------

FAMILIES = {
    "whole": schedules.whole,
    "bulk_then_tail": lambda r: schedules.bulk_then_tail(r, tail=48),
    "portions": schedules.portions,
    "mixed": schedules.mixed,
    "mixed_two_slots": lambda r: schedules.mixed(r, max_live=2, seed=5, decode_tail=20),
    "mixed_long_portions": lambda r: schedules.mixed(r, max_live=3, seed=8, max_portion=130),
}


@pytest.mark.parametrize("backend,dtype", CASES)
@pytest.mark.parametrize("family", list(FAMILIES))
@pytest.mark.parametrize("which", list(CONFIGS))
def test_schedule_matches_plain(tmp_path, which, family, backend, dtype):
    if backend == "double" and (which == "D" or (which in ("A", "C") and family not in ("mixed", "portions"))):
        pytest.skip("the CPU stand-in is slow at this size")
    folder, cfg, weights = make_dir(tmp_path, which)
    requests = _requests(which)
    steps = FAMILIES[family](requests)
    bs = BLOCK[which]
    _, model, cache, runner = make_runner(
        folder, _ops(backend, dtype), block_size=bs, num_blocks=max(1, schedules.pages_needed(steps, bs)),
        max_requests=schedules.most_live(steps),
    )
    cache.poison()
    for bank in cache.state_banks.values():  # stale states in every slot: a request must start from zeros
        bank.tensor.fill_(float("nan"))
    got = schedules.run_schedule(runner, cache, steps)
    _compare(got, requests, weights, cfg, dtype)
    cache.check_invariants()
    assert all(g.allocator.free_count == g.num_blocks for g in cache.groups), "pages were not given back"


@pytest.mark.parametrize("backend,dtype", CASES)
def test_the_batch_and_the_cut_do_not_matter(tmp_path, backend, dtype):
    """The same request alone and whole, and in portions beside others on other pages and in another slot."""
    folder, cfg, weights = make_dir(tmp_path, "A")
    requests = _requests("A")
    results = []
    for steps in (schedules.whole(requests), schedules.mixed(requests)):
        _, _, cache, runner = make_runner(folder, _ops(backend, dtype), block_size=16, num_blocks=24, max_requests=4)
        results.append(schedules.run_schedule(runner, cache, steps))
    one, other = results
    size = float(torch.stack([v.double() for v in one.values()]).pow(2).mean().sqrt())
    off = [float((one[k].double() - other[k].double()).abs().max()) / size for k in one]
    if dtype == torch.float32:
        assert max(off) < 1e-3
    else:  # but for a few rows where rounding chooses between two experts
        assert sorted(off)[int(0.95 * len(off))] < 0.1 and sum(o >= 0.2 for o in off) <= 0.05 * len(off) + 1


@pytest.mark.parametrize("dtype", GPU_CASES)
def test_long_decoding(tmp_path, dtype):
    """Two hundred tokens decoded one by one behind a prompt (replayed steps, partitions of the keys that grow, pages
    behind the window given back and used again while the first ones stay, states swapped at every commit), two
    requests side by side."""
    folder, cfg, weights = make_dir(tmp_path, "D")
    requests = {"a": random_tokens(330, cfg["vocab"], 21), "b": random_tokens(263, cfg["vocab"], 22)}
    steps = []
    for pos in range(330):  # a's prompt of 130 and b's of 63 in one step each, then a token of each per step
        entries = []
        for rid, toks in requests.items():
            head = len(toks) - 200
            if pos == head - 1:
                entries.append({"id": rid, "tokens": toks[:head], "want": list(range(head))})
            elif head <= pos < len(toks):
                entries.append({"id": rid, "tokens": [toks[pos]], "want": [0]})
        if entries:
            steps.append({"step": len(steps), "entries": entries, "end": []})
    steps[-1]["end"] = ["a"]
    for step in reversed(steps):
        if any(e["id"] == "b" for e in step["entries"]):
            step["end"] = step["end"] + ["b"]
            break
    _, _, cache, runner = make_runner(
        folder, _ops("hip", dtype), block_size=16, num_blocks=schedules.pages_needed(steps, 16), max_requests=2
    )
    cache.poison()
    _compare(schedules.run_schedule(runner, cache, steps), requests, weights, cfg, dtype)


@pytest.mark.parametrize("backend,dtype", CASES)
@pytest.mark.parametrize("which", ["A", "C"])
def test_layer_outputs_match_plain(tmp_path, which, backend, dtype):
    folder, cfg, weights = make_dir(tmp_path, which)
    toks = random_tokens(31, cfg["vocab"], 8)
    _, _, cache, runner = make_runner(folder, _ops(backend, dtype), block_size=16, num_blocks=4, max_requests=1)
    cache.create_request("a")
    out = runner.step([StepEntry.of("a", toks, [0, 17, 30])], capture_sites=True)
    _, layers = plain.forward(cfg, _f64(weights), toks)
    assert out.site_outputs.shape == (len(cfg["layers"]), 3, cfg["width"])
    want = layers[:, [0, 17, 30]]
    got = out.site_outputs.double().cpu()
    if dtype == torch.float32:
        torch.testing.assert_close(got, want, rtol=1e-3, atol=1e-3)
        return
    # bfloat16: a row within 6 %, or within 3 times of what rounding alone does to it
    coarse = plain.forward(cfg, _f64(weights), toks, round_to=torch.bfloat16)[1][:, [0, 17, 30]]
    size = want.pow(2).sum(-1).sqrt()
    rel, alone = (got - want).pow(2).sum(-1).sqrt() / size, (coarse - want).pow(2).sum(-1).sqrt() / size
    assert bool((rel < torch.clamp(3.0 * alone, min=6e-2)).all()), (rel, alone)


@pytest.mark.parametrize("dtype", GPU_CASES)
def test_replayed_steps_equal_plain_steps(tmp_path, dtype):
    """Steps with state slots, carried inputs, routed experts and pages that are given back are recorded and replayed;
    the replays give what the unrecorded steps give, bit for bit."""
    folder, cfg, _ = make_dir(tmp_path, "A")
    requests = {"a": random_tokens(90, cfg["vocab"], 1), "b": random_tokens(75, cfg["vocab"], 2)}
    steps = schedules.bulk_then_tail(requests, tail=40)
    results = []
    for use_graphs in (False, True):
        _, _, cache, runner = make_runner(folder, _ops("hip", dtype), block_size=16, num_blocks=16, max_requests=2)
        runner.use_graphs = use_graphs
        results.append(schedules.run_schedule(runner, cache, steps))
    plain_steps, replayed = results
    assert plain_steps.keys() == replayed.keys()
    for key in plain_steps:
        assert torch.equal(plain_steps[key], replayed[key]), key


# ---- generation through the engine ------------------------------------------------------------------------

@pytest.mark.parametrize("backend,dtype", CASES)
@pytest.mark.parametrize("which", ["A", "B"])
def test_greedy_generation_through_the_engine(tmp_path, which, backend, dtype):
    folder, cfg, weights = make_dir(tmp_path, which)
    ops = _ops(backend, dtype)
    engine = ContinuousBatchEngine.from_model_dir(
        folder, dtype=ops.dtype, ops=ops, block_size=BLOCK[which], num_blocks=40, max_running_requests=3,
        max_batch_tokens=24,
    )
    prompts = [random_tokens(n, cfg["vocab"], 9 + n) for n in (5, 30, 1, 17)]
    outs = engine.generate(prompts, max_new_tokens=24)  # long enough to pass page borders while decoding
    w64 = _f64(weights)
    for prompt, tokens in zip(prompts, outs):
        assert len(tokens) == 24
        seq = list(prompt)
        for i, tok in enumerate(tokens):
            logits = plain.forward(cfg, w64, seq)[0][-1]
            best = int(torch.argmax(logits))
            if tok != best:
                # only rounding may choose between two nearly equal logits, and only in bfloat16
                assert dtype == torch.bfloat16, f"token {i}: {tok} != {best}"
                alone = float((plain.forward(cfg, w64, seq, round_to=dtype)[0][-1] - logits).abs().max())
                assert float(logits[best] - logits[tok]) < max(6e-2 * float(logits.abs().max()), 3.0 * alone)
                break
            seq.append(tok)


# ---- the command line and the replay program --------------------------------------------------------------

def test_preset_and_random_model_writer(tmp_path):
    from helpers import read_weights
    from mini_llm_runtime_amd import cli
    from mini_llm_runtime_amd.config.presets import preset_names

    assert "goguzen-tiny" in preset_names()
    assert cli.main(["random-model", "--config", "goguzen-tiny", "--seed", "2", "--out", str(tmp_path / "m")]) == 0
    cfg, w = read_weights(tmp_path / "m")
    assert cfg["architecture"] == "Goguzen" and w["embed"].shape == (320, 96) and w["head"].shape == (320, 96)
    assert w["l0.mix.v"].shape == (32, 96) and w["l0.mix.q.norm"].shape == (144,) and w["l0.mix.sink"].shape == (6,)
    assert w["l1.mix.left.k.norm"].shape == (32,) and w["l1.mix.right.conv"].shape == (192, 4) and "l1.mix.left.v" not in w
    assert w["l1.mix.left.out"].shape == (96,) and w["l1.mlp.e6.down"].shape == (96, 48) and "l2.norm1" not in w
    assert w["l0.mlp.router.b"].shape == (7,) and w["l0.mlp.shared.gate"].shape == (64, 96)
    logits, layers = plain.forward(cfg, _f64(w), [1, 2, 3])  # the plain implementation reads the same folder
    assert logits.shape == (3, 320) and layers.shape == (4, 3, 96) and torch.isfinite(logits).all()


@pytest.mark.gpu
def test_generate_command_and_trace_replay(tmp_path, gpu_device):
    import subprocess
    import sys

    folder, cfg, weights = make_dir(tmp_path, "A")
    w64 = _f64(weights)
    prompt = random_tokens(21, cfg["vocab"], 4)
    proc = subprocess.run(
        [sys.executable, "-m", "mini_llm_runtime_amd.cli", "generate", "--model", str(folder), "--dtype", "float32",
         "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "5"],
        cwd=ROOT, capture_output=True, text=True, timeout=300,
    )
    assert proc.returncode == 0, proc.stderr[-2000:]
    out = json.loads(proc.stdout.strip().splitlines()[-1])
    seq = list(prompt)
    for tok in out["generated_token_ids"]:
        assert tok == int(torch.argmax(plain.forward(cfg, w64, seq)[0][-1]))
        seq.append(tok)
    # the replay program: requests in portions beside each other, slots and pages used again
    toks = {"a": random_tokens(40, cfg["vocab"], 5), "b": random_tokens(27, cfg["vocab"], 6), "c": random_tokens(33, cfg["vocab"], 7)}
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": toks["a"][:25], "want": [0, 24]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": toks["a"][25:27], "want": [1]}, {"id": "b", "tokens": toks["b"], "want": [26]}], "end": ["b"]},
        {"step": 2, "entries": [{"id": "a", "tokens": toks["a"][27:], "want": [12]}, {"id": "c", "tokens": toks["c"][:32], "want": []}], "end": ["a"]},
        {"step": 3, "entries": [{"id": "c", "tokens": toks["c"][32:], "want": [0]}], "end": ["c"]},
    ]
    for dtype, bound in (("float32", 3e-4), ("bfloat16", 6e-2)):
        proc = subprocess.run(
            [str(ROOT / "bin" / "trace_run"), "--model", str(folder), "--dtype", dtype, "--out", str(tmp_path / dtype),
             "--max-tokens", "128", "--max-live", "2"],
            input="".join(json.dumps(s) + "\n" for s in steps), cwd=ROOT, capture_output=True, text=True, timeout=300,
        )
        assert proc.returncode == 0, proc.stderr[-2000:]
        assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
        wanted = {0: [("a", 0), ("a", 24)], 1: [("a", 26), ("b", 26)], 2: [("a", 39)], 3: [("c", 32)]}
        for step, rows in wanted.items():
            got = torch.from_numpy(np.fromfile(tmp_path / dtype / f"{step}.f32", dtype="<f4").reshape(len(rows), cfg["vocab"]))
            for row, (rid, pos) in zip(got, rows):
                ref = plain.forward(cfg, w64, toks[rid][: pos + 1])[0][-1]
                rel = float((row.double() - ref).pow(2).sum().sqrt() / ref.pow(2).sum().sqrt())
                allowed = bound
                if dtype == "bfloat16" and rel >= bound:  # held against what rounding alone does to this row
                    coarse = plain.forward(cfg, w64, toks[rid][: pos + 1], round_to=torch.bfloat16)[0][-1]
                    allowed = max(bound, 3.0 * float((coarse - ref).pow(2).sum().sqrt() / ref.pow(2).sum().sqrt()))
                assert rel < allowed, (dtype, step, rid, pos, rel)
