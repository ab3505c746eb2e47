"""Seeded random Mefurax configurations: any order of the two mixers, with or without a feed-forward, dense or routed, with and
without a shared expert; any number of heads and groups; key and value heads that are multiples of nothing, up to sizes of real
models' heads; windows and chunks from one position to longer than the sequence, or none; rotations of a part or all of a head;
convolutions of one to seven taps; capped scores or not; values mixed or not; widths and vocabularies that are no multiple of
four.  Every configuration goes through a mixed trace (pages and state slots used again): on the CPU with the kernels' twins, on
the GPU through ``bin/trace_run`` in both types."""
import io
import os
import random
import subprocess
import sys
import tempfile

import numpy as np
import pytest
import torch

import plain_mefurax as plain
import traces
from helpers import random_tokens, relative_error
from llmserver_amd.config import config_from_dict
from llmserver_amd.engine.replay import make_runner, replay
from llmserver_amd.weights import RandomInit, write_random_model
from tiny_mefurax import chunked, config, dense, moe, sloped
from torch_ops import TorchOps

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
SEEDS = list(range(12))
FLOAT32_ERROR = 3e-5
_MADE = {}


def random_config(seed):
    rng = random.Random(9000 + seed)
    big = seed % 2 == 1                      # every other seed has heads of the sizes real models use
    values = rng.choice([32, 64, 128]) if big else rng.choice([6, 12, 20, 24, 36])       # a token's values, as many in every layer that mixes
    layers = []
    for _ in range(rng.randint(1, 4)):
        kv_heads = rng.choice([d for d in range(1, 7) if values % d == 0])
        heads, vdim = kv_heads * rng.randint(1, 3), values // kv_heads
        dim = rng.choice([32, 64, 96, 128]) if big else rng.randint(2, 40)
        reach = rng.choice([None, 1, 2, 7, 16, 33, 64, 100, 200])
        mixes = rng.random() < 0.7
        if not mixes:
            vdim = rng.choice([16, 64, 80]) if big else rng.randint(1, 30)
        if rng.random() < 0.5:
            mixer = sloped(heads, kv_heads, dim, vdim, rng.uniform(0.05, 0.4), rng.randint(1, 7), reach, mixes)
        else:
            mixer = chunked(heads, kv_heads, dim, vdim, rng.uniform(0.5, 1.5) * dim ** -0.5, (2 * rng.randint(1, dim // 2), 10.0 ** rng.uniform(1.5, 6.0)),
                            rng.choice([None, rng.uniform(1.0, 50.0)]), reach, mixes)
            if mixer["mixer"]["softcap"] is None:
                del mixer["mixer"]["softcap"]
        kind = rng.random()
        mlp = None
        if kind < 0.3:
            mlp = dense(rng.choice([64, 96]) if big else rng.randint(3, 60))
        elif kind < 0.9:
            experts = rng.randint(1, 10)
            mlp = moe(rng.choice([32, 64]) if big else rng.randint(3, 60), experts, rng.randint(1, min(4, experts)), rng.choice([None, 32, 17, 80]))
        layers.append((mixer, mlp))
    width = rng.choice([64, 128, 256]) if big else rng.choice([24, 40, 50, 64, 72, 100, 134])
    raw = config(rng.randint(30, 400), width, 10.0 ** rng.uniform(-6, -3), rng.uniform(0.5, 4.0), layers)
    return raw, RandomInit(seed=seed, std=rng.uniform(0.08, 0.2), norm_noise=0.25, bias_std=0.3), rng.choice([4, 8, 16, 32])


def made(seed):
    """(config.json, folder, page size, requests, steps, exact logits per request, tensors) of a seed, made once."""
    if seed not in _MADE:
        raw, init, page = random_config(seed)
        folder = tempfile.mkdtemp(prefix=f"llmserver_amd_test_mr{seed}_")
        write_random_model(config_from_dict(dict(raw)), folder, init)
        lengths = (1, 37, 90, 5, 64, 2, 130, 18)
        requests = {f"q{i}": random_tokens(raw["vocab"], n, 50 * seed + i) for i, n in enumerate(lengths)}
        steps = traces.mixed(requests, seed=seed, budget_tokens=256)
        for rid in ("q2", "q6"):                             # (and whole, so that portions of prompts meet the kernels made for them)
            steps.append({"step": len(steps), "entries": [{"id": rid + "w", "tokens": requests[rid], "want": list(range(len(requests[rid])))}],
                          "end": [rid + "w"]})
            requests[rid + "w"] = requests[rid]
        raw_read, tensors = plain.read_folder(folder)
        for layer in raw_read["layers"]:                     # (the oracle wants a cap: one that bends nothing where there is none)
            if layer["type"] == "attention_2":
                layer["mixer"].setdefault("softcap", 1e9)
        exact = {rid: plain.forward(raw_read, tensors, tokens).numpy() for rid, tokens in requests.items()}
        _MADE[seed] = (raw_read, folder, page, requests, steps, exact, tensors)
    return _MADE[seed]


_BOUNDS = {}


def float32_bound(seed, rid, position):
    """What a position's logits may differ by in float32, in units of their largest magnitude: three times what the plain
    implementation itself loses when it computes in float32 (the 99th percentile over the seed's positions), and never
    less than FLOAT32_ERROR; a badly conditioned position is allowed ten times the plain implementation's own loss there:
    still far below what a wrong key, window or state does."""
    if seed not in _BOUNDS:
        raw, folder, _, requests, _, exact, _ = made(seed)
        single = plain.read_folder(folder, dtype=torch.float32)[1]
        raw = {**raw, "layers": [{**layer, "mixer": {**layer["mixer"], **({"softcap": 1e4} if layer["mixer"].get("softcap") == 1e9 else {})}} for layer in raw["layers"]]}
        lost = {(r, p): relative_error(row, want) for r, tokens in requests.items()
                for p, (row, want) in enumerate(zip(plain.forward(raw, single, tokens).numpy(), exact[r]))}
        _BOUNDS[seed] = (max(FLOAT32_ERROR, 3.0 * float(np.quantile(list(lost.values()), 0.99))), lost)
    everywhere, lost = _BOUNDS[seed]
    return max(everywhere, 10.0 * lost[(rid, position)])


def test_the_seeds_cover_every_mixer_and_option():
    raws = [random_config(seed)[0] for seed in SEEDS]
    layers = [layer for raw in raws for layer in raw["layers"]]
    mixers = [layer["mixer"] for layer in layers]
    assert {layer["type"] for layer in layers} == {"attention", "attention_2"}
    kinds = [layer["mlp"] and layer["mlp"]["kind"] for layer in layers]
    assert {None, "dense", "moe"} == set(kinds)
    assert any("shared" in layer["mlp"] for layer in layers if layer["mlp"]) and any("shared" not in (layer["mlp"] or {}) for layer in layers)
    for name in ("mask", "softcap"):
        assert any(name in m for m in mixers) and any(name not in m for m in mixers)
    assert any(m.get("conv", 0) > 4 for m in mixers) and any(m.get("conv") == 1 for m in mixers)
    assert any(m["v_mix"] for m in mixers) and any(not m["v_mix"] for m in mixers)
    first = [next((layer["type"] for layer in raw["layers"] if layer["mixer"]["v_mix"]), None) for raw in raws]
    assert {"attention", "attention_2"} <= set(first)


@pytest.mark.parametrize("seed", SEEDS)
def test_random_configurations_with_the_twins(seed, tmp_path):
    raw, folder, page, requests, steps, exact, _ = made(seed)
    runner = make_runner(folder, "float32", traces.peak_tokens(steps), page, device="cpu", ops=TorchOps())
    replay(runner, traces.to_lines(steps).splitlines(), str(tmp_path), io.StringIO())
    runner.cache.check_invariants()
    results = traces.collect(steps, str(tmp_path), raw["vocab"])
    assert len(results) == sum(len(t) for t in requests.values())
    for (rid, position), logits in results.items():
        assert relative_error(logits, exact[rid][position]) <= float32_bound(seed, rid, position), f"seed {seed} {rid} {position}: {raw}"


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", SEEDS)
def test_random_configurations_on_the_gpu(seed, dtype, tmp_path):
    raw, folder, page, requests, steps, exact, tensors = made(seed)
    print(f"random configuration {seed} {dtype}: {raw}", flush=True)
    out = tmp_path / "out"
    command = [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out),
               "--max-tokens", str(traces.peak_tokens(steps)), "--page-size", str(page)]
    done = subprocess.run(command, input=traces.to_lines(steps), capture_output=True, text=True, timeout=600)
    assert done.returncode == 0, done.stderr[-3000:]
    results = traces.collect(steps, str(out), raw["vocab"])
    assert len(results) == sum(len(t) for t in requests.values())
    errors = []
    for (rid, position), logits in results.items():
        if dtype == "float32":
            assert relative_error(logits, exact[rid][position]) <= float32_bound(seed, rid, position), f"seed {seed} {rid} {position}: {raw}"
        else:
            errors.append(relative_error(logits, exact[rid][position]))
    if errors:
        # what the plain implementation loses on the same sequences when it rounds where 16-bit kernels round
        rounding = plain.rounding_to(torch.bfloat16)
        lost = [relative_error(row, want) for rid, tokens in requests.items()
                for row, want in zip(plain.forward(raw, tensors, tokens, r=rounding).numpy(), exact[rid])]
        assert np.isfinite(errors).all()
        print(f"  median {np.median(errors):.2e} / {np.median(lost):.2e}, 90th {np.quantile(errors, 0.9):.2e} / {np.quantile(lost, 0.9):.2e}", flush=True)
        assert np.median(errors) <= 1.3 * np.median(lost), (seed, np.median(errors), np.median(lost))
        assert np.quantile(errors, 0.9) <= 3.0 * np.quantile(lost, 0.9), (seed, np.quantile(errors, 0.9), np.quantile(lost, 0.9))
