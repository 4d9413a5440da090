"""Drawn Goguzen configurations: every size, constant, layer order and option drawn anew, random weights, a drawn
schedule and page size, the engine against the plain implementation.  A model of this design that nobody has
looked at must run without a change of code; this is the nearest a test gets.

Bounds as in `test_goguzen._compare`, wider for single rows: a mixer's output is divided by its own size before it is
added, the state space's in parts of a few numbers, so where one nearly vanishes its direction is what rounding made of
it."""

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
from test_goguzen import FAMILIES, _attn, _both, _compare, _left, _model, _moe, _ops, _rot, _ssm, make_weights


def _draw_rot(rng: random.Random, most: int):
    if rng.random() < 0.15:
        return None
    dims = rng.choice([d for d in (0, 2, 4, 8, 16, 32, 64, most) if d <= most and d % 2 == 0])
    scaling = None
    if rng.random() < 0.7:
        low = rng.choice([0.5, 1.0, 2.0])
        scaling = (rng.choice([2.0, 4.0, 8.0, 32.0]), low, low * rng.choice([1.0, 2.0, 4.0]), rng.choice([16, 64, 256, 4096]))
    return _rot(rng.choice([100.0, 10000.0, 500000.0]), dims, scaling)


def draw_config(seed: int) -> dict:
    rng = random.Random(seed)
    width = rng.choice([48, 64, 70, 72, 96, 100, 128, 160, 192, 256])
    layers = []
    for i in range(rng.randint(1, 5)):
        if layers and rng.random() < 0.3:
            source = rng.randrange(len(layers))
            layers.append((*layers[source][:2], source))
            continue
        mlp = None
        if rng.random() < 0.7:
            experts = rng.choice([1, 2, 3, 5, 8, 12])
            shared = None if rng.random() < 0.3 else (rng.choice([8, 21, 48, 96]), rng.choice([0.5, 1.0, 1.5, 7.0]))
            mlp = _moe(experts, rng.randint(1, min(experts, 4)), rng.choice([8, 15, 24, 40, 64, 136]), rng.choice([0.5, 1.0, 2.0, 7.0]), shared)
        scale, kv = round(rng.uniform(0.08, 0.5), 3), rng.choice([1, 2, 3, 4])
        heads, dim = kv * rng.choice([1, 2, 3, 4]), rng.choice([8, 16, 20, 32, 48, 64, 128])
        if rng.random() < 0.5:
            size = None if rng.random() < 0.15 else rng.choice([1, 5, 16, 24, 33, 64, 90])
            keep = rng.choice([0, 1, 3, 6, 16, 20, 70])
            vdim = rng.choice([dim, 8, 12, 16, 32, 40, 64, 96])
            mixer = _attn(heads, kv, dim, vdim, scale, size, keep if size else 0, _draw_rot(rng, dim))
        else:
            every = None if rng.random() < 0.2 else rng.choice([1, 3, 16, 50, 128])
            groups = rng.choice([1, 2, 3])
            state_heads, vdim = groups * rng.choice([1, 2, 4]), rng.choice([8, 12, 16, 32, 40, 64])
            parts = rng.choice([n for n in (1, 2, 3, 4, 6, 8) if (state_heads * vdim) % n == 0])
            state = _ssm(state_heads, vdim, rng.choice([4, 8, 16, 24, 48, 64, 96, 128, 160]), groups, rng.choice([1, 2, 3, 4, 7]), parts)
            mixer = _both(_left(heads, kv, dim, scale, every, rng.choice([0.1, 0.3, -0.1])), state)
        layers.append((mixer, mlp))
    return _model(
        rng.randint(50, 600), width, rng.choice([1e-5, 1e-6]), layers, scale=rng.choice([0.5, 1.0, 3.0]),
        logit_scale=rng.choice([0.5, 1.0, 1.3]), cap=rng.choice([None, 5.0, 20.0]),
    )


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
