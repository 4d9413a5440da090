"""Drawn Rofetar configurations: every size, constant, layer order and option drawn anew, random weights, a drawn
schedule and page size, the engine against the plain implementation.  A model of this design that nobody has
looked at must run without a change of code; this is the nearest a test gets.

Bounds as in `test_rofetar._compare`, wider for single rows.  A sublayer's output is divided by its own size, in a
state-space layer in parts of a few numbers, so where a part nearly vanishes its direction is what rounding made of
it: in one of these models (seed 28) the rows that bfloat16 moves by 5 to 13 % in the kernels move by 6 to 7 % in the
stand-in's bfloat16 too, by 2 to 3 % with the plain implementation's inputs rounded, and are the worst ones, at 1e-5,
in float32.

140 more configurations from the same generator were run once on the GPU in both dtypes.  float32 passed all of them,
bfloat16 missed a single row in two: in one a state-space head's write and skip cancel to a hundredth, in the other a
delta head's read-out does, and the bfloat16 stream turns that head's sign over.  From the sums that the input product
really left, the kernels' read-outs are those of float64 to 5e-6."""

from __future__ import annotations

import json
import random
from pathlib import Path

import pytest
import torch

import mini_llm_runtime_amd.models  # noqa: F401
import schedules
from helpers import make_runner, random_tokens
from mini_llm_runtime_amd.weights import save_state_dict
from test_rofetar import FAMILIES, _attn, _compare, _delta, _dense, _model, _ops, _rot, _ssm, make_weights


def _draw_rot(rng: random.Random, most: int):
    if rng.random() < 0.15:
        return None
    dims = rng.choice([d for d in (2, 4, 8, 16, 32, 64, most) if d <= most and d % 2 == 0])
    scaling = None
    if rng.random() < 0.7:
        scaling = (rng.choice([2.0, 4.0, 8.0, 32.0]), rng.choice([16, 64, 256, 4096]), rng.choice([4.0, 8.0, 32.0]), rng.choice([0.5, 1.0, 2.0]))
    return _rot(rng.choice([100.0, 10000.0, 500000.0]), dims, scaling)


def draw_config(seed: int) -> dict:
    rng = random.Random(seed)
    width = rng.choice([48, 64, 70, 72, 96, 100, 128, 160, 192, 256])
    layers, owners = [], []
    for i in range(rng.randint(1, 6)):
        mlp = None if rng.random() < 0.4 else _dense(rng.choice([24, 40, 45, 64, 136, 320]))
        kind = rng.choice(["attention", "delta", "mamba2"])
        scale, softcap = round(rng.uniform(0.08, 0.5), 3), rng.choice([None, 5.0, 15.0, 30.0])
        if kind == "attention" and owners and rng.random() < 0.5:
            source = rng.choice(owners)
            m = layers[source][0][1]
            mixer = _attn(m["heads"], m["kv_heads"], m["dim"], m["vdim"], scale, softcap, m.get("rot"), kv_from=source)
        elif kind == "attention":
            kv = rng.choice([1, 2, 3, 4])
            dim = rng.choice([8, 16, 20, 32, 48, 64, 128])
            mixer = _attn(
                kv * rng.choice([1, 2, 3, 4]), kv, dim, rng.choice([dim, 8, 12, 16, 32, 40, 64, 96]), scale, softcap,
                _draw_rot(rng, dim),
            )
            owners.append(i)
        elif kind == "delta":
            kv = rng.choice([1, 2, 3])
            dim = rng.choice([4, 8, 16, 20, 32, 48, 64, 100, 128, 144])
            mixer = _delta(kv * rng.choice([1, 2, 3]), kv, dim, rng.choice([dim, 8, 12, 16, 32, 40, 64, 96]), rng.choice([1, 2, 3, 4, 5]))
        else:
            groups = rng.choice([1, 2, 3])
            heads, vdim = groups * rng.choice([1, 2, 4]), rng.choice([8, 12, 16, 32, 40, 64])
            parts = rng.choice([n for n in (1, 2, 3, 4, 6, 8) if (heads * vdim) % n == 0])
            mixer = _ssm(heads, vdim, rng.choice([4, 8, 16, 24, 48, 64, 96, 128, 160]), groups, rng.choice([1, 2, 3, 4, 7]), parts)
        layers.append((mixer, mlp))
    return _model(rng.randint(50, 600), width, rng.choice([1e-5, 1e-6]), layers)


def _run(tmp_path, seed: int, backend: str, dtype: torch.dtype) -> None:
    cfg = draw_config(seed)
    rng = random.Random(1000 + seed)
    folder = Path(tmp_path) / f"drawn{seed}"
    folder.mkdir()
    (folder / "config.json").write_text(json.dumps(cfg))
    weights = make_weights(cfg, seed)
    save_state_dict(folder / "model.safetensors", weights)
    longest = 200 if backend == "hip" else 40
    requests = {f"r{i}": random_tokens(rng.randint(1, longest), cfg["vocab"], seed * 10 + i) for i in range(rng.randint(2, 4))}
    family = rng.choice(sorted(FAMILIES))
    steps = FAMILIES[family](requests)
    bs = rng.choice([4, 8, 16, 32])
    _, _, cache, runner = make_runner(
        folder, _ops(backend, dtype), block_size=bs, num_blocks=max(1, schedules.pages_needed(steps, bs)),
        max_requests=schedules.most_live(steps),
    )
    cache.poison()
    for bank in cache.state_banks.values():
        bank.tensor.fill_(float("nan"))
    got = schedules.run_schedule(runner, cache, steps)
    try:
        _compare(got, requests, weights, cfg, dtype, f32_bound=1e-3, together=4e-2, worst_row=8.0)
    except AssertionError as e:
        raise AssertionError(f"{e}\nconfiguration {seed}: {json.dumps(cfg)}; {family}, pages of {bs}") from None
    cache.check_invariants()


@pytest.mark.parametrize("seed", range(6))
def test_drawn_configuration_on_the_stand_in(tmp_path, seed):
    _run(tmp_path, seed, "double", torch.float32)


@pytest.mark.gpu
@pytest.mark.parametrize("seed", range(32))
def test_drawn_configuration(tmp_path, seed):
    _run(tmp_path, seed, "hip", torch.float32 if seed % 2 else torch.bfloat16)
