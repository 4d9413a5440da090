"""The Rofetar decoder in the engine against the plain implementation (`plain_rofetar.py`).

Each mechanism alone (short convolutions with activation, unit norms and gates; the scan of a decaying state, plain
and by the delta rule, token by token and in chunks, with its state rows; gate and norm in parts of a row; per-head
weighted norms with rotation and cache write; capped scores with one more in the denominator on every attention
kernel; the GELU gating; one-layer models of every mixer), keys placed so that one far score stands out, states that
never forget through one reused slot, then whole models under every way of cutting and batching over poisoned pages
and stale slots, the stream after every layer, replays against unrecorded steps, and greedy generation through the
engine, the command line and the replay program.  The tests make their own small configurations and weights; sizes
differ from layer to layer, also where a model could make them equal, and some are 1.

`double` cases run everything above the kernels on the CPU stand-in; `hip` cases run the HIP kernels
(`-m gpu`) in float32 and bfloat16.
"""

from __future__ import annotations

import copy
import json
import math
from pathlib import Path
from types import SimpleNamespace

import pytest
import torch

import mini_llm_runtime_amd.models  # noqa: F401
import plain_rofetar as plain
import schedules
from helpers import StepEntry, make_runner, random_tokens
from kernel_doubles import TorchOps
from mini_llm_runtime_amd.config import ConfigError
from mini_llm_runtime_amd.config.rofetar import RofetarConfig
from mini_llm_runtime_amd.engine import ContinuousBatchEngine
from mini_llm_runtime_amd.models import build_model, config_from_dict
from mini_llm_runtime_amd.weights import save_state_dict

ROOT = Path(__file__).resolve().parents[1]


# ---- configurations -----------------------------------------------------------------------------------

def _rot(base, dims, scaling=None):
    out = {"base": base, "dims": dims}
    if scaling is not None:
        out["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return out


def _attn(heads, kv_heads, dim, vdim, scale, softcap=None, rot=None, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if softcap is not None:
        m["softcap"] = softcap
    if rot is not None:
        m["rot"] = rot
    if kv_from is not None:
        m["kv_from"] = kv_from
    return "attention", m


def _ssm(heads, vdim, state, groups, conv, norm_groups):
    return "mamba2", {
        "heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups,
    }


def _delta(heads, kv_heads, dim, vdim, conv):
    return "delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _model(vocab, width, eps, layers):
    return {
        "architecture": "Rofetar", "vocab": vocab, "width": width, "norm": {"eps": eps},
        "layers": [{"type": kind, "mixer": mixer, "mlp": mlp} for (kind, mixer), mlp in layers],
    }


YARN = (4.0, 64, 16.0, 1.0)
ROT_A = _rot(10000.0, 8, YARN)
CONFIGS = {
    # every mixer, layers that read another's keys with queries and constants of their own, values narrower than keys
    "A": _model(97, 64, 1e-5, [
        (_attn(4, 2, 16, 12, 0.3, 15.0, ROT_A), _dense(96)),
        (_delta(4, 2, 16, 24, 4), _dense(40)),
        (_ssm(4, 16, 24, 2, 3, 2), None),
        (_attn(4, 2, 16, 12, 0.2, 6.0, ROT_A, kv_from=0), None),
        (_delta(2, 2, 12, 8, 2), None),
        (_attn(4, 2, 16, 12, 0.25, None, ROT_A, kv_from=0), _dense(72)),
    ]),
    # one head everywhere, widths no kernel likes, an odd feed-forward, a convolution of one tap and one of six
    "B": _model(61, 36, 1e-6, [
        (_delta(1, 1, 20, 20, 1), _dense(27)),
        (_ssm(1, 20, 10, 1, 6, 1), _dense(16)),
        (_attn(1, 1, 20, 20, 0.22, 4.0), None),
        (_ssm(3, 10, 7, 3, 1, 5), None),
    ]),
    # as many key/value heads as heads, values wider than keys, every dim turns, norm parts that cut through heads
    "C": _model(128, 48, 1e-5, [
        (_ssm(6, 16, 32, 2, 4, 3), _dense(64)),
        (_attn(3, 3, 48, 64, 0.15, 30.0, _rot(20000.0, 48)), None),
        (_delta(6, 3, 16, 16, 4), None),
        (_attn(8, 2, 32, 32, 0.2, 10.0, _rot(500000.0, 16, (8.0, 32, 32.0, 2.0))), _dense(48)),
        (_attn(8, 2, 32, 32, 0.3, 20.0, _rot(500000.0, 16, (8.0, 32, 32.0, 2.0)), kv_from=3), _dense(56)),
    ]),
    # long requests: decode partitions, many key tiles, states carried over many chunks
    "D": _model(80, 64, 1e-5, [
        (_delta(4, 2, 32, 32, 4), _dense(64)),
        (_attn(4, 2, 32, 32, 0.3, 12.0, _rot(10000.0, 32)), None),
        (_ssm(4, 32, 40, 2, 4, 2), None),
        (_attn(4, 2, 32, 32, 0.4, 12.0, _rot(10000.0, 32), kv_from=1), _dense(64)),
        (_delta(2, 1, 48, 64, 3), None),
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
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        w[p + "norm1"] = normal(width, std=0.2, mean=1.0)
        if layer["type"] == "attention":
            w[p + "mix.q"] = matrix(m["heads"] * m["dim"], width)
            w[p + "mix.q.norm"] = normal(m["dim"], std=0.2, mean=1.0)
            if "kv_from" not in m:
                w[p + "mix.k"] = matrix(m["kv_heads"] * m["dim"], width)
                w[p + "mix.v"] = matrix(m["kv_heads"] * m["vdim"], width)
                w[p + "mix.k.norm"] = normal(m["dim"], std=0.2, mean=1.0)
        elif layer["type"] == "mamba2":
            inner, bc = m["heads"] * m["vdim"], 2 * m["groups"] * m["state"]
            w[p + "mix.in"] = matrix(2 * inner + bc + m["heads"], width, 1.5)
            w[p + "mix.conv"] = normal(inner + bc, m["conv"], std=0.6)
            w[p + "mix.conv.b"] = normal(inner + bc, std=0.2)
            w[p + "mix.dt_bias"] = normal(m["heads"], std=0.7, mean=-2.0)
            w[p + "mix.A_log"] = normal(m["heads"], std=0.7)
            w[p + "mix.D"] = normal(m["heads"], std=0.5, mean=0.7)
            w[p + "mix.norm"] = normal(inner, std=0.2, mean=1.0)
        else:
            qk, v = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for n, rows in (("q", qk), ("k", qk), ("v", v)):
                w[p + f"mix.{n}"] = matrix(rows, width, 1.5)
                w[p + f"mix.{n}.conv"] = normal(rows, m["conv"], std=0.6)
            w[p + "mix.b"] = matrix(m["heads"], width)
            w[p + "mix.a"] = matrix(m["heads"], width)
            w[p + "mix.A_log"] = normal(m["heads"], std=0.7)
            w[p + "mix.dt_bias"] = normal(m["heads"], std=0.7, mean=-2.0)
            w[p + "mix.g"] = matrix(v, width, 1.5)
            w[p + "mix.norm"] = normal(m["vdim"], std=0.2, mean=1.0)
        w[p + "mix.o"] = matrix(width, m["heads"] * m["vdim"])
        f = layer["mlp"]
        if f is not None:
            w[p + "norm2"] = normal(width, std=0.2, mean=1.0)
            for n, rows, cols, gain in (("gate", f["ff"], width, 1.5), ("up", f["ff"], width, 1.5), ("down", width, f["ff"], 1.0)):
                w[p + f"mlp.{n}"] = matrix(rows, cols, gain)
                w[p + f"mlp.{n}.b"] = normal(rows, std=0.3)
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
    return write_model(tmp_path, f"rofetar{which}", cfg, weights), cfg, weights


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


def _compare(got, requests, weights, cfg, dtype, f32_bound=3e-4, row_bound=6e-2, together=3e-2, worst_row=4.0):
    """float32: every value within 3e-4 of the logits' size, or within 4 times of what rounding the inputs of the
    products to float32 does to the worst row (a sublayer's output is divided by its own size on its way into the
    stream, so where a head's read-out nearly vanishes any rounding is blown up).  bfloat16: all rows together
    within 3 % (relative L2, the mean over the vocabulary taken off) or twice what rounding alone does; every row
    within 6 %, but for a few (one in twenty, and as many as rounding alone puts beyond 6 %) that may be off by up
    to `worst_row` times what rounding alone does to the worst row of their request.  A wrong key, page, slot or state
    changes most rows, by half and more."""
    assert got, "no logits came back"
    w64 = _f64(weights)
    num = den = num_alone = 0.0
    loose = rows = loose_alone = 0
    for rid, toks in requests.items():
        ref, _ = plain.forward(cfg, w64, toks)
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
            if rel >= row_bound:
                loose += 1
                assert rel < worst_row * max(float(alone.max()), row_bound / 2), f"{rid}:{pos}: relative error {rel:.3e}, rounding alone up to {float(alone.max()):.3e}"
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
    assert isinstance(c, RofetarConfig)
    assert [l.mixer.kind for l in c.layers] == ["attention", "delta", "mamba2", "attention", "delta", "attention"]
    assert c.layers[0].mixer.rot.scaling.factor == 4.0 and c.layers[0].mixer.kv_from is None
    assert c.layers[3].mixer.kv_from == 0 and c.layers[3].mixer.softcap == 6.0 and c.layers[5].mixer.softcap is None
    assert c.layers[2].mixer.norm_groups == 2 and c.layers[2].mlp is None and c.layers[1].mlp.ff == 40
    assert RofetarConfig.from_dict(c.to_dict()) == c
    assert RofetarConfig.from_dict(config_from_dict(CONFIGS["B"]).to_dict()).layers[2].mixer.rot is None


@pytest.mark.parametrize(
    "change",
    [
        lambda c: c["layers"][0]["mixer"].pop("scale"),
        lambda c: c["layers"][0].update(type="convolution"),
        lambda c: c["layers"][0]["mixer"].update(kv_heads=3),  # four heads on three
        lambda c: c["layers"][0]["mixer"]["rot"].update(dims=40),  # more than a head has
        lambda c: c["layers"][0]["mixer"].update(softcap=-1.0),
        lambda c: c["layers"][3]["mixer"].update(kv_from=1),  # a layer without keys
        lambda c: c["layers"][3]["mixer"].update(kv_from=5),  # a later one
        lambda c: c["layers"][5]["mixer"].update(kv_from=3),  # one that has none of its own
        lambda c: c["layers"][3]["mixer"].update(kv_heads=1),  # other heads than the keys it reads
        lambda c: c["layers"][3]["mixer"].update(rot=_rot(10000.0, 8)),  # another rotation than the keys'
        lambda c: c["layers"][1]["mixer"].update(conv=0),
        lambda c: c["layers"][2]["mixer"].update(groups=3),
        lambda c: c["layers"][2]["mixer"].update(norm_groups=7),
        lambda c: c["layers"][1]["mlp"].update(kind="sparse"),
        lambda c: c.update(layers=[]),
    ],
)
def test_config_refuses_what_does_not_fit(change):
    cfg = copy.deepcopy(CONFIGS["A"])
    change(cfg)
    with pytest.raises(ConfigError):
        config_from_dict(cfg)


def test_model_is_built_from_the_framework_parts():
    from mini_llm_runtime_amd.parts.attention import GQAAttention
    from mini_llm_runtime_amd.parts.block import PostNormBlock
    from mini_llm_runtime_amd.parts.feed_forward import GeGLU
    from mini_llm_runtime_amd.parts.gated_delta import GatedDelta
    from mini_llm_runtime_amd.parts.state_space import StateSpace

    model = build_model(config_from_dict(CONFIGS["A"]))
    assert all(isinstance(layer, PostNormBlock) for layer in model.layers)
    assert [type(layer.mixer) for layer in model.layers] == [GQAAttention, GatedDelta, StateSpace, GQAAttention, GatedDelta, GQAAttention]
    assert [model.cache_site_of(i) for i in range(6)] == [0, 1, 2, 0, 4, 0]
    assert "k_norm_weight" not in model.layers[3].mixer.param_specs()
    assert model.layers[3].mixer.param_specs()["qkv_weight"].shape == (64, 64)  # queries only
    assert isinstance(model.layers[1].feed_forward, GeGLU) and model.layers[2].feed_forward is None
    assert not model.spec.tie_word_embeddings and model.replayable and model.splittable
    # states and the convolutions' inputs live in the manager's slots, keys and values in pages, shared ones nowhere
    kinds = [type(s).__name__ for s in model.site_cache_specs()]
    assert kinds == ["PagedKVSpec", "CompositeSpec", "CompositeSpec", "NoneType", "CompositeSpec", "NoneType"]
    one_tap = build_model(config_from_dict(CONFIGS["B"])).site_cache_specs()[0]
    assert type(one_tap).__name__ == "SlotStateSpec"  # nothing carried beside the state


# ---- mechanisms alone, on the GPU ------------------------------------------------------------------------

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


@pytest.mark.gpu
@pytest.mark.parametrize("taps,units,unit_dim,plain_channels,heads,sigmoid", [
    (4, 4, 16, 40, 3, True), (1, 2, 20, 7, 1, True), (2, 0, 0, 300, 5, False), (3, 6, 128, 520, 70, True), (6, 1, 256, 3, 2, False),
])
def test_convolution_unit_norms_and_gates(taps, units, unit_dim, plain_channels, heads, sigmoid):
    """Entries of 1, 5, 2 and 40 tokens: one fresh on a row of NaN, one shorter than the convolution is long."""
    hip, double = _ops("hip", torch.float32), TorchOps(torch.float32, "cpu")
    g = torch.Generator().manual_seed(taps * 100 + heads)
    lengths, starts = [1, 5, 2, 40], [3, 0, 1, 9]
    tokens, channels = sum(lengths), units * unit_dim + plain_channels
    column = 5
    width = column + channels + 2 * heads + 1
    projected = torch.randn(tokens, width, generator=g)
    conv = torch.randn(taps, channels, generator=g) * 0.5
    bias = torch.randn(channels, generator=g) * 0.3 if taps != 3 else None
    state = torch.randn(9, max(taps - 1, 1), channels, generator=g)
    state[5] = float("nan")
    read, write = torch.tensor([2, 5, 6, 0], dtype=torch.int32), torch.tensor([3, 4, 7, 1], dtype=torch.int32)
    rate, dt_bias = -torch.rand(heads, generator=g) - 0.1, torch.randn(heads, generator=g)
    results = []
    for ops in (double, hip):
        to = (lambda t: t.cuda()) if ops is hip else (lambda t: t.clone())
        held = to(state)
        carried = SimpleNamespace(tensor=held, read_rows=to(read), write_rows=to(write)) if taps > 1 else None
        out, gates = ops.conv_gates(
            to(projected), to(conv), None if bias is None else to(bias), carried, _step_context(lengths, starts, ops),
            column=column, heads=heads, rate=to(rate), dt_bias=to(dt_bias), step_column=column + channels,
            write_column=column + channels + heads + 1 if sigmoid else None, unit_heads=units, unit_dim=unit_dim,
            scaled_heads=units // 2, unit_scale=0.37,
        )
        results.append((out.cpu(), gates.cpu(), held.cpu()))
    for want, got in zip(*results):
        torch.testing.assert_close(got, want, rtol=2e-5, atol=2e-6, equal_nan=True)


SCANS = [(2, 1, 16, 32), (3, 3, 20, 12), (4, 2, 64, 48), (1, 1, 128, 70), (2, 2, 200, 20), (1, 1, 1, 1), (6, 2, 48, 64), (2, 1, 33, 16)]


@pytest.mark.gpu
@pytest.mark.parametrize("chunked", [False, True], ids=["walk", "chunks"])
@pytest.mark.parametrize("delta", [False, True], ids=["plain", "delta"])
@pytest.mark.parametrize("heads,key_heads,dim,vdim", SCANS)
def test_scan_and_its_state_rows(heads, key_heads, dim, vdim, delta, chunked):
    """Entries of 1, 5, 150, 64 and 65 tokens, one that starts its request on a row full of NaN, the others on carried
    states; rows that no entry writes stay as they were.  Against the stand-in's loop over tokens in float32."""
    hip, double = _ops("hip", torch.float32), TorchOps(torch.float32, "cpu")
    g = torch.Generator().manual_seed(heads * 1000 + dim)
    lengths, starts = [1, 5, 150, 64, 65], [3, 0, 9, 0, 2]
    tokens = sum(lengths)
    qk, v = key_heads * dim, heads * vdim
    offsets = (v + 2, v + 2 + qk, 0)
    mixed = torch.randn(tokens, v + 2 + 2 * qk + 3, generator=g)
    for at in offsets[:2]:
        rows = mixed[:, at : at + qk].view(tokens, key_heads, dim)
        rows /= rows.norm(dim=-1, keepdim=True)
    # decays from none to nearly all within a chunk, writes of the delta rule within 0..1
    gates = torch.stack([-torch.rand(tokens, heads, generator=g) ** 4 * 6.0, torch.rand(tokens, heads, generator=g)], -1)
    state = torch.randn(12, heads, dim, vdim, generator=g) * 0.5
    state[5] = float("nan")
    read = torch.tensor([2, 5, 6, 0, 8], dtype=torch.int32)
    write = torch.tensor([3, 4, 7, 1, 9], dtype=torch.int32)
    skip = None if delta else torch.randn(heads, generator=g)
    kw = dict(heads=heads, key_heads=key_heads, head_dim=dim, value_dim=vdim, offsets=offsets, delta=delta)
    want_state = state.clone()
    want = double.decay_scan(mixed, gates, want_state, read, write, _step_context(lengths, starts, double), skip=skip, **kw)
    got_state = state.cuda()
    got = hip.decay_scan(
        mixed.cuda(), gates.cuda(), got_state, read.cuda(), write.cuda(), _step_context(lengths, starts, hip),
        skip=None if skip is None else skip.cuda(), chunked=chunked, **kw,
    )
    torch.testing.assert_close(got.cpu(), want, rtol=2e-5, atol=2e-5)
    torch.testing.assert_close(got_state.cpu(), want_state, rtol=2e-5, atol=2e-5, equal_nan=True)
    for row in (0, 2, 5, 6, 8, 10):
        assert torch.equal(got_state[row].cpu().nan_to_num(7.0), state[row].nan_to_num(7.0))


@pytest.mark.gpu
@pytest.mark.parametrize("delta", [False, True], ids=["plain", "delta"])
@pytest.mark.parametrize("taps", [1, 2, 4])
@pytest.mark.parametrize("heads,key_heads,dim,vdim", [(2, 1, 16, 32), (6, 2, 64, 80), (3, 3, 100, 12), (4, 2, 144, 70), (1, 1, 1, 1)])
def test_single_token_step_in_one_kernel(heads, key_heads, dim, vdim, taps, delta):
    """Convolution, gates and scan of single tokens in one kernel: as the separate kernels, and as the stand-in; one
    entry starts its request on rows of NaN."""
    hip, double = _ops("hip", torch.float32), TorchOps(torch.float32, "cpu")
    g = torch.Generator().manual_seed(heads * 100 + dim + taps)
    starts, tokens = [4, 0, 1], 3
    qk, v = key_heads * dim, heads * vdim
    channels, column = 2 * qk + v, 6
    offsets = (0, qk, 2 * qk) if delta else (v + qk, v, 0)
    projected = torch.randn(tokens, column + channels + 2 * heads + 2, generator=g)
    conv, bias = torch.randn(taps, channels, generator=g) * 0.5, None if delta else torch.randn(channels, generator=g) * 0.3
    rate, dt_bias = -torch.rand(heads, generator=g) - 0.1, torch.randn(heads, generator=g)
    skip = None if delta else torch.randn(heads, generator=g)
    held = torch.randn(8, max(taps - 1, 1), channels, generator=g)
    state = torch.randn(8, heads, dim, vdim, generator=g) * 0.5
    held[5], state[5] = float("nan"), float("nan")
    read, write = torch.tensor([2, 5, 6], dtype=torch.int32), torch.tensor([3, 4, 7], dtype=torch.int32)
    results = []
    for ops, fused in ((double, None), (hip, False), (hip, True)):
        to = (lambda t: None if t is None else t.cuda()) if ops is hip else (lambda t: None if t is None else t.clone())
        views = [SimpleNamespace(tensor=to(t), read_rows=to(read), write_rows=to(write)) for t in (held, state)]
        out = ops.conv_decay_scan(
            to(projected), to(conv), to(bias), views[0] if taps > 1 else None, views[1], _step_context([1] * tokens, starts, ops),
            column=column, heads=heads, key_heads=key_heads, head_dim=dim, value_dim=vdim, offsets=offsets, rate=to(rate),
            dt_bias=to(dt_bias), step_column=column + channels + 1,
            write_column=column + channels + heads + 2 if delta else None, delta=delta, skip=to(skip), fused=fused,
        )
        results.append((out.cpu(), views[0].tensor.cpu(), views[1].tensor.cpu()))
    for want, apart, one in zip(*results):
        torch.testing.assert_close(one, want, rtol=2e-5, atol=1e-5, equal_nan=True)
        torch.testing.assert_close(one, apart, rtol=2e-5, atol=1e-5, equal_nan=True)


@pytest.mark.gpu
def test_delta_scan_with_one_key_over_and_over():
    """The same key every token, writes of full strength, no decay: every write replaces the one before (the
    triangular system of a chunk is as far from the identity as it gets)."""
    hip = _ops("hip", torch.float32)
    tokens, dim, vdim = 200, 64, 32
    k = torch.nn.functional.normalize(torch.ones(dim) + 0.1 * torch.arange(dim), dim=0)
    g = torch.Generator().manual_seed(1)
    v = torch.randn(tokens, vdim, generator=g)
    mixed = torch.cat([k.expand(tokens, dim), k.expand(tokens, dim), v], 1).contiguous()
    gates = torch.stack([torch.zeros(tokens, 1), torch.ones(tokens, 1)], -1)
    rows = torch.zeros(1, dtype=torch.int32), torch.ones(1, dtype=torch.int32)
    for chunked in (False, True):
        state = torch.zeros(2, 1, dim, vdim).cuda()
        got = hip.decay_scan(
            mixed.cuda(), gates.cuda(), state, rows[0].cuda(), rows[1].cuda(), _step_context([tokens], [0], hip), heads=1,
            key_heads=1, head_dim=dim, value_dim=vdim, offsets=(0, dim, 2 * dim), delta=True, chunked=chunked,
        )
        torch.testing.assert_close(got.cpu(), v, rtol=1e-4, atol=1e-4)  # S^T k is the newest value


@pytest.mark.parametrize("dtype", GPU_CASES)
@pytest.mark.parametrize("tokens,inner,groups", [(1, 64, 1), (19, 60, 5), (7, 2560, 1), (5, 4096, 2), (3, 3, 3)])
def test_gate_and_norm_in_parts(dtype, tokens, inner, groups):
    hip, double = _ops("hip", dtype), TorchOps(dtype, "cpu")
    g = torch.Generator().manual_seed(inner)
    y, projected = torch.randn(tokens, inner, generator=g), torch.randn(tokens, inner + 9, generator=g)
    weight = 1 + 0.3 * torch.randn(inner, generator=g)
    want = double.gate_group_norm(y, projected, gate_column=4, groups=groups, eps=1e-5, norm_weight=weight)
    got = hip.gate_group_norm(y.cuda(), projected.cuda(), gate_column=4, groups=groups, eps=1e-5, norm_weight=weight.cuda())
    torch.testing.assert_close(got.float().cpu(), want.float(), **_tolerance(dtype))


@pytest.mark.parametrize("dtype", GPU_CASES)
@pytest.mark.parametrize("heads,kv,dim,vdim,rdims,block", [(4, 2, 32, 16, 16, 8), (1, 1, 20, 20, 0, 4), (6, 3, 16, 40, 16, 16), (2, 2, 128, 32, 64, 16), (3, 0, 24, 24, 8, 8)])
def test_weighted_head_norms_before_the_rotation(dtype, heads, kv, dim, vdim, rdims, block):
    hip, double = _ops("hip", dtype), TorchOps(dtype, "cpu")
    g = torch.Generator().manual_seed(heads + dim)
    tokens = 37
    pages = -(-tokens // block) + 1
    D = -(-max(dim, vdim) // 16) * 16
    projected = torch.randn(tokens, (heads + kv) * dim + kv * vdim, generator=g) * 2.0
    rotation = None
    if rdims:  # an amplitude other than one: norm and rotation do not commute
        angle = torch.rand(tokens, rdims // 2, generator=g) * 6.0
        rotation = (torch.cos(angle) * 1.4, torch.sin(angle) * 1.4, rdims)
    slots = torch.randperm(pages * block, generator=g)[:tokens].to(torch.int32)
    slots[3] = -1
    weights = [(1 + 0.4 * torch.randn(dim, generator=g)).to(dtype) for _ in range(2)]
    results = []
    for ops in (double, hip):
        to = (lambda t: t.cuda()) if ops is hip else (lambda t: t)
        keys = to(torch.zeros(pages, max(kv, 1), block, D, dtype=dtype))
        values = to(torch.zeros(pages, max(kv, 1), D, block, dtype=dtype))
        q, gate, kept = ops.head_norm_rope_write(
            to(projected), heads=heads, kv_heads=kv, head_dim=dim, value_dim=vdim, kernel_dim=D, eps=1e-5,
            rotation=None if rotation is None else (to(rotation[0]), to(rotation[1]), rdims), slot_mapping=to(slots),
            key_pages=keys, value_pages=values, block_size=block, weights=tuple(to(w) for w in weights),
        )
        assert gate is None and kept is None
        results.append([t.float().cpu() for t in (q, keys, values)])
    for a, b in zip(*results):
        torch.testing.assert_close(b, a, **_tolerance(dtype))


@pytest.mark.parametrize("dtype", GPU_CASES)
@pytest.mark.parametrize("cap", [2.0, 20.0])
@pytest.mark.parametrize("heads,kv,dim,lengths,starts", [
    (4, 2, 64, [1, 1, 1], [700, 0, 33]),  # decoded tokens: one partition and several
    (2, 1, 32, [130, 1, 2], [0, 300, 65]),  # prompt tiles beside decoded tokens
    (3, 3, 128, [70], [400]),
    (8, 2, 24, [5, 1], [20, 3]),  # no multiple of 16: the plain kernel
])
def test_capped_scores_and_one_more_in_the_denominator(dtype, cap, heads, kv, dim, lengths, starts):
    """Large scores, so that the cap bends them; against the stand-in's formulas."""
    from mini_llm_runtime_amd.kernels.plans import attention_plan
    from mini_llm_runtime_amd.parts.context import PlanInput
    import numpy as np

    hip, double = _ops("hip", dtype), TorchOps(dtype, "cpu")
    g = torch.Generator().manual_seed(heads * dim + len(lengths))
    block = 16
    tokens, contexts = sum(lengths), [s + n for s, n in zip(starts, lengths)]
    need = [-(-c // block) for c in contexts]
    pages = sum(need) + 1
    order = torch.randperm(pages, generator=g).tolist()
    table = torch.full((len(lengths), max(need)), -1, dtype=torch.int32)
    for r, n in enumerate(need):
        table[r, :n] = torch.tensor([order.pop() for _ in range(n)], dtype=torch.int32)
    keys = torch.randn(pages, kv, block, dim, generator=g).to(dtype)
    values = torch.randn(pages, kv, dim, block, generator=g).to(dtype)
    q = torch.randn(tokens, heads * dim, generator=g).to(dtype)
    sinks = torch.zeros(heads)
    kw = dict(num_heads=heads, num_kv_heads=kv, head_dim=dim, block_size=block, scale=0.9, window=None, softcap=cap)
    want = double.paged_attention(q, keys, values, table, _step_context(lengths, starts, double), sinks=sinks, **kw)
    shape = attention_plan(PlanInput(np.asarray(lengths), np.asarray(starts), max(contexts)))
    dev = {k: torch.from_numpy(v).to(torch.int32).cuda() for k, v in shape.arrays.items()}
    plan = SimpleNamespace(**shape.sizes, **dev)
    got = hip.paged_attention(
        q.cuda(), keys.cuda(), values.cuda(), table.cuda(), _step_context(lengths, starts, hip), sinks=sinks.cuda(), plan=plan, **kw
    )
    torch.testing.assert_close(got.float().cpu(), want.float(), **(dict(rtol=2e-5, atol=2e-5) if dtype == torch.float32 else dict(rtol=2e-2, atol=1e-2)))


@pytest.mark.parametrize("dtype", GPU_CASES)
@pytest.mark.parametrize("m,k,inner", [(1, 64, 24), (5, 72, 200), (40, 256, 384), (300, 128, 1000), (2100, 64, 640), (7, 36, 18)])
def test_gelu_gating_in_the_products_epilogue(dtype, m, k, inner):
    hip, double = _ops("hip", dtype), TorchOps(dtype, "cpu")
    g = torch.Generator().manual_seed(m + inner)
    x = torch.randn(m, k, generator=g).to(dtype)
    weight = (torch.randn(2 * inner, k, generator=g) * 2.0 / math.sqrt(k)).to(dtype)
    bias = torch.randn(2 * inner, generator=g).to(dtype)
    want = double.linear(x, weight, bias, geglu=True)
    got = hip.linear(x.cuda(), weight.cuda(), bias.cuda(), geglu=True)
    torch.testing.assert_close(got.float().cpu(), want.float(), **_tolerance(dtype))
    if dtype == torch.bfloat16 and k % 8 == 0 and m > 64:  # every tile, the one with an instance of its own included
        for kernel in (11, 22, 23, 44, 45, 46, 47, 48):
            got = hip.linear(x.cuda(), weight.cuda(), bias.cuda(), geglu=True, mfma_kernel=kernel)
            torch.testing.assert_close(got.float().cpu(), want.float(), **_tolerance(dtype))
    sums = torch.randn(m, 2 * 13, generator=g) * 2.0  # an odd size, gated behind its product
    torch.testing.assert_close(hip.glu_gelu(sums.cuda()).float().cpu(), double.glu_gelu(sums).float(), **_tolerance(dtype))
    torch.testing.assert_close(hip.rounded(sums.cuda()).cpu(), sums.to(dtype), rtol=0, atol=0)


# ---- one layer of each kind ----------------------------------------------------------------------------------

ONE_LAYER = {
    "attention": (_attn(4, 2, 16, 24, 0.3, 8.0, _rot(1000.0, 8, YARN)), None),
    "attention-plain": (_attn(2, 2, 8, 8, 0.4), None),
    "state-space": (_ssm(4, 12, 20, 2, 4, 2), None),
    "delta": (_delta(4, 2, 12, 20, 4), None),
    "feed-forward": (_delta(1, 1, 8, 8, 2), _dense(40)),
    "feed-forward-odd": (_ssm(1, 8, 8, 1, 2, 1), _dense(33)),
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


# ---- keys far away and at page borders ------------------------------------------------------------------------

def _needle_model(dim: int, reads: bool):
    """Attention of one head whose keys are the stream itself and whose queries are the stream with its halves
    swapped; token 39's embedding is token 38's with its halves swapped.  Token 39's query then equals the key of token 38
    and of nothing else, and ONE such key, however far, takes nearly all of the weight.  With `reads` a second layer asks
    the first one's keys again with queries of its own."""
    layers = [(_attn(1, 1, dim, dim, 1.0, 20.0), None)]
    if reads:
        layers.append((_attn(1, 1, dim, dim, 1.0, 20.0, kv_from=0), None))
    cfg = _model(40, dim, 1e-6, layers)
    weights = make_weights(cfg, 2)
    eye = torch.eye(dim).to(torch.bfloat16)
    for i in range(len(layers)):
        weights[f"l{i}.mix.q"] = eye.roll(dim // 2, dims=0).contiguous()
        weights[f"l{i}.mix.q.norm"] = torch.ones(dim, dtype=torch.bfloat16)
    weights["l0.mix.k"], weights["l0.mix.k.norm"] = eye.clone(), torch.ones(dim, dtype=torch.bfloat16)
    weights["embed"][39] = weights["embed"][38].roll(dim // 2)
    if reads:  # the first layer hands on little, so that the second one's query still is the token's embedding
        weights["l0.norm1"] = torch.full((dim,), 0.05, dtype=torch.bfloat16)
    return cfg, weights


@pytest.mark.parametrize("backend,dtype", CASES)
@pytest.mark.parametrize("reads", [False, True], ids=["own", "shared"])
@pytest.mark.parametrize("length,marked", [(70, 0), (200, 15), (700, 16), (131, 63), (97, 95)])
def test_one_far_key_that_takes_the_weight(tmp_path, backend, dtype, length, marked, reads):
    if backend == "double" and length > 300:
        pytest.skip("the CPU stand-in is slow at this size")
    cfg, weights = _needle_model(32, reads)
    folder = write_model(tmp_path, "needle", cfg, weights)
    toks = [1 + (i % 30) for i in range(length)]  # ids 1..30 in turn
    toks[marked] = 38
    toks[-1] = 39  # asks for the marked one
    other = list(toks)
    other[marked] = 37
    w64 = _f64(weights)
    with_key, without = plain.forward(cfg, w64, toks)[0][-1], plain.forward(cfg, w64, other)[0][-1]
    assert float((with_key - without).abs().max()) > 0.2 * float(with_key.abs().max()), "the oracle does not see the key"
    _, _, cache, runner = make_runner(folder, _ops(backend, dtype), block_size=16, num_blocks=-(-length // 16), max_requests=1)
    cache.poison()
    cut = max(1, length - 5)
    for steps in (
        schedules.whole({"a": toks}),  # the asking token at the end of a prompt
        schedules.bulk_then_tail({"a": toks}, tail=3),  # decoded alone
        schedules.portions({"a": toks}, sizes=(cut - 1, 2, 3, 2)),  # at the end of a short portion
    ):
        got = schedules.run_schedule(runner, cache, steps)
        row = got[("a", length - 1)].double()
        err = float((row - with_key).abs().max())
        assert err < (1e-4 if dtype == torch.float32 else 5e-2) * float(with_key.abs().max()), err


@pytest.mark.parametrize("backend,dtype", CASES)
@pytest.mark.parametrize("kind", ["delta", "mamba2"])
def test_a_state_that_never_forgets_through_one_slot(tmp_path, kind, backend, dtype):
    """Decays held at one: the first tokens stay in the state (and, at the first places, in the convolution's carried
    inputs), so a state lost between two steps, or a slot cleared too late or not at all, shows at later positions."""
    mixer = _delta(2, 1, 24, 16, 4) if kind == "delta" else _ssm(2, 16, 24, 1, 4, 1)
    cfg = _model(64, 32, 1e-6, [(mixer, None)])
    weights = make_weights(cfg, 11)
    weights["l0.mix.A_log"] = torch.full((2,), -30.0, dtype=torch.bfloat16)  # decay exp(-1e-13 ..)
    if kind == "delta":
        weights["l0.mix.b"] = weights["l0.mix.b"] * 0.2
    folder = write_model(tmp_path, "keeper", cfg, weights)
    a = random_tokens(90, 64, 1)
    b = [(a[0] + 1) % 64] + a[1:]  # differs in the first token only
    w64 = _f64(weights)
    ref_a, ref_b = plain.forward(cfg, w64, a)[0], plain.forward(cfg, w64, b)[0]
    assert float((ref_a[3] - ref_b[3]).abs().max()) > 0.02 * float(ref_a[3].abs().max())
    assert float((ref_a[20] - ref_b[20]).abs().max()) > 1e-3 * float(ref_a[20].abs().max())
    _, _, cache, runner = make_runner(folder, _ops(backend, dtype), block_size=8, num_blocks=1, max_requests=1)
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


@pytest.mark.parametrize("dtype", GPU_CASES)
def test_long_decoding(tmp_path, dtype):
    """Two hundred tokens decoded one by one behind a prompt (replayed steps, partitions of the keys that grow,
    page after page taken, states swapped at every commit), two requests side by side."""
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
    """Steps with state slots, carried inputs and shared pages are recorded and replayed; the replays give what the
    unrecorded steps give, bit for bit."""
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

    assert "rofetar-tiny" in preset_names()
    assert cli.main(["random-model", "--config", "rofetar-tiny", "--seed", "2", "--out", str(tmp_path / "m")]) == 0
    cfg, w = read_weights(tmp_path / "m")
    assert cfg["architecture"] == "Rofetar" and w["embed"].shape == (320, 96) and w["head"].shape == (320, 96)
    assert w["l0.mix.q.conv"].shape == (48, 4) and w["l1.mix.k.norm"].shape == (24,) and "l3.mix.k" not in w
    assert w["l2.mix.conv"].shape == (192, 4) and w["l2.mix.D"].shape == (6,) and "l2.norm2" not in w
    logits, layers = plain.forward(cfg, _f64(w), [1, 2, 3])  # the plain implementation reads the same folder
    assert logits.shape == (3, 320) and layers.shape == (4, 3, 96) and torch.isfinite(logits).all()


@pytest.mark.gpu
def test_generate_command_and_trace_replay(tmp_path, gpu_device):
    import subprocess
    import sys

    import numpy as np

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
