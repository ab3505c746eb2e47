"""Setodra through the engine's own step function, cache manager, scheduler and entry point on the CPU (torch twins
of the kernels) against the plain implementation: configuration and weights, each mechanism, every way of cutting
and batching, pages and state slots used again, far keys and far states, passes over layers, and greedy generation."""
import io
import json
import math
import os
import tempfile

import numpy as np
import pytest
import torch

import plain_setodra as plain
import traces
from helpers import random_tokens
from llmserver_amd.config import ConfigError, UnsupportedModelError, config_from_dict
from llmserver_amd.engine.batch import StepEntry
from llmserver_amd.engine.replay import make_runner, replay
from llmserver_amd.parts import PagedKVSpec, RotaryPosition, StateSpec, YarnScaling
from llmserver_amd.weights import build_model
from tiny_setodra import CASES, SA, SB, SC, SD, SE, model_folder, plain_logits, plain_model, rotation
from torch_ops import ChunkedDecayOps, TorchOps


def runner_for(case, max_tokens, page=None, live=4, ops=None):
    return make_runner(model_folder(case), "float32", max_tokens, page or CASES[case][2], device="cpu", ops=ops or TorchOps(), max_live=live)


def run(case, steps, tmp_path, page=None, ops=None):
    runner = runner_for(case, traces.peak_tokens(steps), page, ops=ops)
    replay(runner, traces.to_lines(steps).splitlines(), str(tmp_path), io.StringIO())
    runner.cache.check_invariants()
    assert not runner.cache.requests and runner.cache.state_slots_free() == 4
    assert all(free == group.pool.num_pages for free, group in zip(runner.cache.available_pages(), runner.cache.groups))
    return traces.collect(steps, str(tmp_path), CASES[case][0]["vocab"])


def check(case, results, requests, atol=1.5e-4):          # (float32 twins against float64)
    for (rid, position), logits in results.items():
        expected = plain_logits(case, tuple(requests[rid]))[position].numpy()
        np.testing.assert_allclose(logits, expected, atol=atol, rtol=3e-4, err_msg=f"{case} {rid} position {position}")
    assert len(results) == sum(len(tokens) for tokens in requests.values())


def requests_of(case, lengths, seed0=300):
    return {f"q{i}": random_tokens(CASES[case][0]["vocab"], n, seed0 + i) for i, n in enumerate(lengths)}


def copy_of(raw):
    return json.loads(json.dumps(raw))


# -- configuration and weights ---------------------------------------------------------------------------------------
def test_the_configuration_reads_back_and_refuses_what_is_not_built():
    for raw in (SA, SB, SC, SD, SE):
        config = config_from_dict(dict(raw))
        again = config_from_dict(config.to_dict())
        assert again.layers == config.layers and again.loop == config.loop and again.to_dict() == config.to_dict()
    config = config_from_dict(dict(SA))
    assert config.layers[2].mlp is None and config.layers[0].mixer.norm_groups == 3 and config.layers[1].mixer.rot.scaling.factor == 4.0
    assert config.layers[0].mlp.identity == 3 and config.layers[0].mlp.shared_ff == 28 and config.layers[3].mlp.shared_ff == 0
    assert config.layer_runs() == ((0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None))
    plain_one = config_from_dict(dict(SB))
    assert plain_one.loop is None and plain_one.embedding_scale == 1.0 and plain_one.layers[0].mixer.rot.dims == 0
    assert plain_one.layers[0].mlp.identity == 0 and plain_one.layers[1].mixer.rot.scaling is None
    assert config_from_dict(dict(SD)).layer_runs() == ((0, 0),)

    def broken(change, error, match):
        other = copy_of(SA)
        change(other)
        with pytest.raises(error, match=match):
            config_from_dict(other)

    broken(lambda c: c["layers"][1].update(type="something else"), UnsupportedModelError, "something else")
    broken(lambda c: c["layers"][1]["mlp"].update(kind="other"), UnsupportedModelError, "other")
    broken(lambda c: c["layers"][0]["mixer"].pop("state"), ConfigError, "state")
    broken(lambda c: c["layers"][0]["mixer"].update(groups=3), ConfigError, "groups")
    broken(lambda c: c["layers"][0]["mixer"].update(norm_groups=5), ConfigError, "parts")
    broken(lambda c: c["layers"][1]["mixer"].pop("rot"), ConfigError, "rot")
    broken(lambda c: c["layers"][2]["mixer"]["rot"].update(dims=5), ConfigError, "even")
    broken(lambda c: c["layers"][2]["mixer"].update(decay=[0.5]), ConfigError, "decays")
    broken(lambda c: c["layers"][1]["mixer"].update(kv_rank=250), UnsupportedModelError, "rows of up to 256")
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=9), ConfigError, "uses 9")
    broken(lambda c: c["loop"].update(stop=9), ConfigError, "loop")


def test_the_model_declares_the_checkpoints_tensors_and_its_caches():
    model = build_model(config_from_dict(dict(SA)))
    specs = model.param_specs()
    assert {"embed", "head", "final.norm", "loop.step", "l0.norm1", "l0.norm2", "l0.mix.in", "l0.mix.conv", "l0.mix.conv.b", "l0.mix.dt_bias",
            "l0.mix.A_log", "l0.mix.D", "l0.mix.norm", "l0.mix.o", "l0.mlp.router", "l0.mlp.correction", "l0.mlp.e4.down", "l0.mlp.shared.gate",
            "l0.mlp.shared.sg", "l1.mix.dkv.norm", "l2.mix.g", "l2.mix.v"} <= set(specs)
    assert not {"l0.mlp.e5.gate", "l2.norm2", "l3.mlp.shared.sg", "l1.mix.g", "l1.mix.sink", "l0.hc1.in", "l4.norm1"} & set(specs)
    assert specs["l0.mix.in"].shape == (2 * 24 + 2 * 20 + 4, 48) and specs["l0.mix.conv"].shape == (64, 4) and specs["l3.mix.conv"].shape == (40, 1)
    assert specs["l0.mlp.router"].shape == (8, 48) and specs["l0.mlp.correction"].shape == (8,) and specs["l0.mlp.shared.sg"].shape == (1, 48)
    assert specs["l1.mix.q"].shape == (60, 48) and specs["l1.mix.dkv"].shape == (22, 48) and specs["loop.step"].shape == (3, 48)
    assert specs["l2.mix.q"].shape == (20, 48) and specs["l2.mix.g"].shape == (14, 48)
    caches = model.cache_specs()
    assert len(caches) == 8                                  # a cache or state for every run of a layer, looped ones three times
    assert caches[0] == StateSpec((4 * 10 * 6 + 3 * 64,), "float32") and caches[7] == StateSpec((3 * 5 * 10,), "float32")
    for run_of in (1, 3, 5):
        assert isinstance(caches[run_of], PagedKVSpec) and caches[run_of].window is None and caches[run_of].n_kv_heads == 1
    for run_of in (2, 4, 6):
        assert caches[run_of] == StateSpec((2 * 10 * 7,), "float32")
    assert "loop.step" not in build_model(config_from_dict(dict(SB))).param_specs()


def test_stretched_frequencies_by_hand():
    """Eight pairs over an original length of 64: pairs that turn more than ``fast`` times over it keep their frequency, pairs
    that turn fewer than ``slow`` times are divided by the factor, the pairs between are mixed linearly in their number."""
    position = RotaryPosition(16, 1000.0, scaling=YarnScaling(4.0, 64.0, 4.0, 0.5))
    got = position.inverse_frequencies().double().numpy()
    plain_ones = [1000.0 ** (-i / 8) for i in range(8)]
    first = math.floor(16 * math.log(64 / (2 * math.pi * 4.0)) / (2 * math.log(1000.0)))
    last = math.ceil(16 * math.log(64 / (2 * math.pi * 0.5)) / (2 * math.log(1000.0)))
    assert (first, last) == (1, 4)
    want = [plain_ones[0], plain_ones[1], plain_ones[2] * (2 / 3 + 1 / 12), plain_ones[3] * (1 / 3 + 2 / 12)] + [f / 4 for f in plain_ones[4:]]
    np.testing.assert_allclose(got, want, rtol=1e-6)
    assert abs(position.scaling.amplitude - (0.1 * math.log(4.0) + 1.0)) < 1e-12
    dims, oracle, amplitude = plain.rotation({"rot": rotation(16, 1000.0, (4.0, 64.0, 4.0, 0.5))})
    np.testing.assert_allclose(got, oracle, rtol=1e-6)
    assert dims == 16 and abs(amplitude - position.scaling.amplitude) < 1e-12
    # an edge in front of the first pair, and a ramp without width
    for scaling in ((2.0, 10.0, 50.0, 1.0), (2.0, 64.0, 2.0, 2.0)):
        np.testing.assert_allclose(RotaryPosition(16, 1000.0, scaling=YarnScaling(*scaling)).inverse_frequencies().double().numpy(),
                                   plain.rotation({"rot": rotation(16, 1000.0, scaling)})[1], rtol=1e-6)


# -- schedules ---------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("case", sorted(CASES))
@pytest.mark.parametrize("schedule", ["whole", "tail", "portions", "mixed"])
def test_every_schedule_matches_the_plain_implementation(case, schedule, tmp_path):
    lengths = (5, 17, 33, 70, 41, 1, 64, 60, 20, 2) if schedule == "mixed" else (70, 33, 1, 2)
    requests = requests_of(case, lengths)
    if schedule == "whole":
        steps = traces.whole(requests)
    elif schedule == "tail":
        steps = traces.tail_decoded(requests, 32)
    elif schedule == "portions":
        steps = traces.changing_portions(requests, sizes=(2, 7, 1, 3, 33, 2, 2, 16, 5))
    else:
        steps = traces.mixed(requests, seed=11, budget_tokens=256)
        assert max(len(s["entries"]) for s in steps) >= 3 and sum(lengths) > traces.peak_tokens(steps)
    check(case, run(case, steps, tmp_path), requests)


@pytest.mark.parametrize("case", ["SA", "SC"])
def test_the_products_made_inside_the_kernels_give_the_same(case, tmp_path):
    """The same through the parts' other way: the shared expert's products beside the routed experts', the latent's beside
    attention (what the kernels are asked for in steps of few tokens)."""
    ops = TorchOps()
    ops.inside = ops.inside_shared = True
    requests = requests_of(case, (20, 3))
    check(case, run(case, traces.changing_portions(requests, sizes=(2, 7, 1, 3, 2)), tmp_path, ops=ops), requests)


def test_the_stream_behind_every_layer_run_is_the_plain_implementations():
    """The stream behind each run of a layer, a looped layer once a pass, in front of what opens the next pass."""
    raw, tensors = plain_model("SA")
    tokens = random_tokens(97, 23, 2)
    kept = []
    plain.forward(raw, tensors, tokens, keep=kept)
    runner = runner_for("SA", 64)
    runner.cache.open("r")
    seen = []
    runner.model.after_call = lambda index, stream, pending: seen.append(stream[0].clone())
    runner.step([StepEntry("r", tokens, [])])
    assert len(seen) == len(kept) == 8
    for index, (got, expected) in enumerate(zip(seen, kept)):
        np.testing.assert_allclose(got.numpy(), expected.numpy(), atol=1e-4, rtol=1e-4, err_msg=f"run {index}")


def test_prefill_equals_token_by_token_decoding_from_the_first_token(tmp_path):
    """Every token alone, from position 0: states, convolutions and cache rows start from nothing."""
    for case in ("SA", "SB", "SC"):
        requests = requests_of(case, (40,))
        check(case, run(case, traces.tail_decoded(requests, 64), tmp_path / case), requests)


@pytest.mark.parametrize("case", ["SA", "SC"])
@pytest.mark.parametrize("chunk", [5, 16, 64])
def test_long_portions_through_the_chunked_form_of_the_recurrences(case, chunk, tmp_path):
    """Steps that bring many tokens run their recurrences in chunks (products over a chunk's tokens, the state walked from
    chunk to chunk), steps of single tokens as the scan; both leave the same state and logits, whatever the chunks' size
    and wherever a portion ends: in the middle of a chunk, at its last token, one token into the next."""
    requests = requests_of(case, (3 * chunk + 1 if chunk < 64 else 130, 2 * chunk, chunk - 1, 70))
    steps = traces.changing_portions(requests, sizes=(chunk + 3, 2, 2 * chunk, 1, chunk))
    ops = ChunkedDecayOps(chunk=chunk, chunked_from=chunk // 2)
    check(case, run(case, steps, tmp_path, ops=ops), requests)
    assert ops.chunked_steps > 0


@pytest.mark.parametrize("page", [4, 8, 64])
def test_page_sizes_and_page_borders(page, tmp_path):
    requests = requests_of("SA", (2 * page + 1, page, page - 1, page + 1))
    steps = traces.changing_portions(requests, sizes=(page - 1, 2, page, 1, page + 1))
    check("SA", run("SA", steps, tmp_path, page=page), requests)


def test_state_slots_and_pages_are_used_again_in_any_order():
    """Eight requests through four slots: a slot's next holder must start from zeros (matrices and convolution inputs), not
    from its predecessor's state; batches of unequal portions in changing order."""
    runner = runner_for("SA", 4 * 64, live=4)
    tokens = {i: random_tokens(97, 18 + 5 * i, 900 + i) for i in range(8)}
    got = {}
    for first in (0, 4):
        live = list(range(first, first + 4))
        for rid in live:
            runner.cache.open(rid)
        assert sorted(runner.cache.record(rid).state_slot for rid in live) == [0, 1, 2, 3]
        done = {rid: 0 for rid in live}
        turn = 0
        while any(done[rid] < len(tokens[rid]) for rid in live):
            entries = []
            for rid in live[::-1] if turn % 2 else live:
                size = (1, 3, 2, 7)[(rid + turn) % 4]
                if done[rid] < len(tokens[rid]):
                    piece = tokens[rid][done[rid]:done[rid] + size]
                    entries.append(StepEntry(rid, piece, list(range(len(piece)))))
            logits = runner.step(entries)
            row = 0
            for entry in entries:
                for _ in entry.tokens:
                    got[(entry.request_id, done[entry.request_id])] = logits[row].numpy()
                    done[entry.request_id] += 1
                    row += 1
            turn += 1
        for rid in live[::-1]:
            runner.cache.close(rid)
    for (rid, position), logits in got.items():
        expected = plain_logits("SA", tuple(tokens[rid]))[position].numpy()
        np.testing.assert_allclose(logits, expected, atol=1e-4, rtol=3e-4, err_msg=f"{rid} {position}")


# -- mechanisms that random weights could hide ---------------------------------------------------------------------
def sharpened(case, change, change_config=None):
    """The case's tensors with ``change(tensors)`` applied, written to a folder of its own; (folder, config, tensors)."""
    from safetensors.torch import save_file
    raw, tensors = plain_model(case)
    tensors = {name: tensor.clone() for name, tensor in tensors.items()}
    change(tensors)
    raw = copy_of(raw)
    if change_config is not None:
        change_config(raw)
    folder = tempfile.mkdtemp(prefix="llmserver_amd_test_sharp_")
    save_file({name: tensor.to(torch.bfloat16).contiguous() for name, tensor in tensors.items()}, os.path.join(folder, "model.safetensors"))
    with open(os.path.join(folder, "config.json"), "w") as handle:
        json.dump(raw, handle)
    return (folder, *plain.read_folder(folder))


def logits_of(folder, tokens, cuts, page=8):
    runner = make_runner(folder, "float32", 64 * (-(-len(tokens) // 64)), page, device="cpu", ops=TorchOps())
    runner.cache.open("r")
    rows, start = [], 0
    for size in cuts:
        piece = tokens[start:start + size]
        if not piece:
            break
        rows.append(runner.step([StepEntry("r", piece, list(range(len(piece))))]).clone())
        start += len(piece)
    assert start == len(tokens)
    return torch.cat(rows).numpy()


# (what the GPU tests run again on the kernels: case, change of the tensors, change of the configuration, tokens)
def far_state(tensors):
    """Step sizes and decays pushed to where the state keeps everything: exp(A_log) small, steps of about one."""
    for name in list(tensors):
        if name.endswith("A_log"):
            tensors[name][:] = -9.0
        if name.endswith("dt_bias"):
            tensors[name][:] = -2.0
    tensors["l2.mix.q"] *= 0.0                     # (attention sees every key alike: nothing else tells the first tokens apart from later ones)


def far_state_config(raw):
    raw["layers"][1]["mixer"]["decay"] = [0.9999, 1.0]


def far_key(tensors):
    for layer in (1, 3):
        tensors[f"l{layer}.mix.q"] *= 5.0
        tensors[f"l{layer}.mix.uk"] *= 5.0


def oldest_tap(tensors):
    for name in list(tensors):
        if name.endswith("mix.conv"):
            tensors[name][:, 1:] *= 0.05
            tensors[name][:, 0] *= 6.0


SHARP = {"far state": ("SC", far_state, far_state_config, 200), "far key": ("SB", far_key, None, 230), "oldest tap": ("SA", oldest_tap, None, 60),
         "oldest of six taps": ("SB", oldest_tap, None, 60)}


def test_tokens_hundreds_back_decide_through_the_states():
    """Decays pushed to one keep everything for ever: what the states took in hundreds of tokens ago decides the logits,
    in a prompt and for decoded tokens; a state that is lost, or cut off where a portion starts, shows."""
    case, change, change_config, length = SHARP["far state"]
    folder, raw, tensors = sharpened(case, change, change_config)
    tokens = random_tokens(200, length, 5)
    expected = plain.forward(raw, tensors, tokens).numpy()
    other = plain.forward(raw, tensors, random_tokens(200, 20, 6) + tokens[20:]).numpy()
    assert np.abs(other[-1] - expected[-1]).max() > 1e-2
    for cuts in ([200], [180] + [1] * 20, [3, 100, 2, 50, 45]):
        np.testing.assert_allclose(logits_of(folder, tokens, cuts, page=16), expected, atol=2e-4, rtol=5e-4, err_msg=str(cuts))


def test_a_key_hundreds_back_among_hundreds_decides_in_latent_attention():
    """Queries and keys scaled up: a few keys carry all the weight, and which ones depends on the whole context; the first
    tokens replaced change the logits at the end."""
    case, change, _, length = SHARP["far key"]
    folder, raw, tensors = sharpened(case, change)
    tokens = random_tokens(130, length, 15)
    expected = plain.forward(raw, tensors, tokens).numpy()
    assert np.abs(plain.forward(raw, tensors, random_tokens(130, 30, 1) + tokens[30:]).numpy()[200:] - expected[200:]).max() > 1e-2
    for cuts in ([230], [200] + [1] * 30, [129, 2, 64, 35]):
        for page in (8, 64):
            np.testing.assert_allclose(logits_of(folder, tokens, cuts, page), expected, atol=3e-4, rtol=1e-3, err_msg=f"{cuts} {page}")


@pytest.mark.parametrize("name", ["oldest tap", "oldest of six taps"])
def test_the_convolutions_oldest_tap_reaches_over_earlier_steps(name):
    """Nearly all of a convolution's weight on its oldest tap: portions shorter than its reach, single tokens, and both."""
    case, change, _, length = SHARP[name]
    folder, raw, tensors = sharpened(case, change)
    tokens = random_tokens(raw["vocab"], length, 9)
    expected = plain.forward(raw, tensors, tokens).numpy()
    moved = {n: (torch.roll(t, 1, dims=1) if n.endswith("mix.conv") else t) for n, t in tensors.items()}
    assert np.abs(plain.forward(raw, moved, tokens).numpy() - expected).max() > 1e-2
    for cuts in ([60], [1] * 60, [2] * 30, [2, 1, 3, 4, 5, 1, 1, 6, 2, 35], [59, 1]):
        np.testing.assert_allclose(logits_of(folder, tokens, cuts), expected, atol=1.5e-4, rtol=3e-4, err_msg=str(cuts))


def planted(module_changes, case="SA", count=50, change_config=None, threshold=3e-3):
    """The oracle with a mistake planted gives other logits than the oracle; the engine gives the oracle's."""
    raw, tensors = plain_model(case)
    tokens = random_tokens(raw["vocab"], count, 3)
    expected = plain_logits(case, tuple(tokens)).numpy()
    kept = {name: getattr(plain, name) for name in module_changes}
    try:
        for name, make in module_changes.items():
            setattr(plain, name, make(kept[name]))
        wrong_raw = copy_of(raw)
        if change_config is not None:
            change_config(wrong_raw)
        assert np.abs(plain.forward(wrong_raw, tensors, tokens).numpy() - expected).max() > threshold
    finally:
        for name, function in kept.items():
            setattr(plain, name, function)
    for cuts in ([count], [count - 20] + [1] * 20):
        np.testing.assert_allclose(logits_of(model_folder(case), tokens, cuts), expected, atol=1.5e-4, rtol=3e-4)


def test_the_rotation_is_stretched_and_its_amplitude_applied():
    planted({}, change_config=lambda raw: raw["layers"][1]["mixer"]["rot"].pop("scaling"))
    planted({"rotation": lambda kept: lambda sizes: (lambda t: None if t is None else (t[0], t[1], 1.0))(kept(sizes))})
    planted({}, case="SB", change_config=lambda raw: raw["layers"][3]["mixer"]["rot"]["scaling"].update(original=1000))


def test_the_choice_is_corrected_and_the_weights_are_not():
    def weights_with_correction(kept):
        def route(h, t, p, router):
            scores = torch.softmax(h @ t[p + "router"].T, dim=-1) + t[p + "correction"]
            chosen = torch.topk(scores, router["top"], dim=-1).indices
            picked = scores.gather(1, chosen)
            return chosen, picked / (picked.sum(dim=-1, keepdim=True) + 1e-20) * router["scale"]
        return route

    def choice_without_correction(kept):
        return lambda h, t, p, router: kept(h, {**t, p + "correction": t[p + "correction"] * 0}, p, router)

    planted({"route": weights_with_correction})
    planted({"route": choice_without_correction})


def test_identity_experts_return_their_input_and_the_shared_expert_is_gated():
    def nothing_from_identity(kept):
        def route(h, t, p, router):
            chosen, weights = kept(h, t, p, router)
            return chosen, weights * (chosen < router["experts"])
        return route

    raw, tensors = plain_model("SA")
    h = torch.randn(40, 48, dtype=torch.float64)
    chosen, _ = plain.route(h, tensors, "l0.mlp.", raw["layers"][0]["mlp"]["router"])
    assert (chosen >= 5).any() and (chosen < 5).any()                # both kinds are chosen
    planted({"route": nothing_from_identity})
    planted({"experts": lambda kept: lambda h, t, p, mlp, r=plain.same: kept(h, {**t, p + "shared.sg": t[p + "router"][:1] * 0}, p, mlp, r)})


def test_a_pass_begins_with_its_vector_and_every_later_one_with_the_embedding_again():
    """Another vector for one pass, passes that keep no cache of their own, or an embedding that is not added again give
    other logits (the last by an embedding scale that reaches the passes only)."""
    raw, tensors = plain_model("SA")
    tokens = random_tokens(97, 50, 3)
    expected = plain_logits("SA", tuple(tokens)).numpy()
    for number in range(3):
        other = dict(tensors)
        other["loop.step"] = tensors["loop.step"].clone()
        other["loop.step"][number] *= -1.0
        assert np.abs(plain.forward(raw, other, tokens).numpy() - expected).max() > 1e-2
    planted({"passes": lambda kept: lambda config: [(layer, 0 if number else number) for layer, number in kept(config)]})
    planted({"passes": lambda kept: lambda config: [(layer, None) for layer, _ in kept(config)]})
    for cuts in ([1] * 50, [2, 33, 7, 8]):
        np.testing.assert_allclose(logits_of(model_folder("SA"), tokens, cuts), expected, atol=1.5e-4, rtol=3e-4)


# -- the oracle itself -------------------------------------------------------------------------------------------------
def test_the_oracles_mechanisms_by_hand():
    f64 = lambda values: torch.tensor(values, dtype=torch.float64)
    assert torch.allclose(plain.norm(f64([[3.0, 4.0]]), f64([1.0, 2.0]), 0.0), f64([[3.0, 8.0]]) / 12.5 ** 0.5)
    # four dimensions of five turn: halves pair (0, 2) and (1, 3); the second pair turns by p / base^(1/2)
    x = f64([[[1.0, 2.0, 3.0, 4.0, 7.0]]])
    a, b = 3.0, 3.0 / 100.0 ** 0.5
    turned = plain.rotate(x, torch.tensor([3]), plain.rotation({"rot": {"dims": 4, "base": 100.0}}))
    assert torch.allclose(turned, f64([[[np.cos(a) - 3 * np.sin(a), 2 * np.cos(b) - 4 * np.sin(b), 3 * np.cos(a) + np.sin(a),
                                         4 * np.cos(b) + 2 * np.sin(b), 7.0]]]))
    # a convolution of two taps: the last column meets the token itself; zeros before the start
    assert torch.allclose(plain.short_convolution(f64([[1.0], [2.0], [5.0]]), f64([[10.0, 1.0]]), f64([0.5])), f64([[1.5], [12.5], [25.5]]))
    # a state-space head of one channel by hand: in = [z, x, B, C, dt], one tap, no skip; softplus(0) = ln 2
    one = f64([[1.0]])
    t = {"p.in": f64([[1.0], [2.0], [3.0], [4.0], [0.0]]), "p.conv": f64([[1.0]] * 3), "p.conv.b": f64([0.0] * 3), "p.dt_bias": f64([0.0]),
         "p.A_log": f64([0.0]), "p.D": f64([0.5]), "p.norm": f64([3.0]), "p.o": one}
    kept = plain.unit_root_mean_square
    try:
        plain.unit_root_mean_square = lambda x, eps: x
        out = plain.mamba2(torch.ones(2, 1, dtype=torch.float64), t, "p.", {"heads": 1, "vdim": 1, "state": 1, "groups": 1, "norm_groups": 1}, 0.0)
    finally:
        plain.unit_root_mean_square = kept
    s = lambda z: z / (1 + np.exp(-z))
    x, B, C, dt = s(2.0), s(3.0), s(4.0), np.log(2.0)
    first = dt * B * x
    second = np.exp(-dt) * first + dt * B * x
    assert torch.allclose(out, 3.0 * s(1.0) * f64([[first * C + 0.5 * x], [second * C + 0.5 * x]]))
    # retention of one channel: S = 1, 1.5, 1.75 under a decay of one half; each head's read-out over its own size
    t = {"p.q": one, "p.k": one, "p.v": one, "p.g": one, "p.o": one}
    try:
        plain.unit_root_mean_square = lambda x, eps: x
        out = plain.retention(torch.ones(3, 1, dtype=torch.float64), t, "p.", {"heads": 1, "dim": 1, "vdim": 1, "decay": [0.5]}, 0.0)
    finally:
        plain.unit_root_mean_square = kept
    assert torch.allclose(out, s(1.0) * f64([[1.0], [1.5], [1.75]]))
    # the router: softmax of (0, ln 3) is (1/4, 3/4); the correction turns the choice, the weight is the score over the sum
    t = {"p.router": f64([[0.0], [np.log(3.0)]]), "p.correction": f64([0.6, 0.0])}
    chosen, weights = plain.route(one, t, "p.", {"top": 1, "scale": 2.0, "experts": 1})
    assert chosen.tolist() == [[0]] and torch.allclose(weights, f64([[2.0]]))
    chosen, weights = plain.route(one, t, "p.", {"top": 2, "scale": 2.0, "experts": 1})
    assert torch.allclose(weights.gather(1, chosen.argsort()), f64([[0.5, 1.5]]))
    assert plain.passes({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]


# -- generation through the entry point, the scheduler and the engine ------------------------------------------------------
def test_greedy_generation_through_the_entry_point_equals_the_oracles():
    """More requests than places, prompts cut into portions by the token budget, a pool so small that requests wait
    for pages: the engine's own scheduler, cache manager, step function and sampler produce the oracle's tokens."""
    from llmserver_amd.entrypoints import generate
    for case, vocab in (("SA", 97), ("SB", 130)):
        raw, tensors = plain_model(case)
        prompts = [random_tokens(vocab, n, 700 + n) for n in (19, 3, 41, 8, 1, 27)]
        expected = [plain.greedy_generate(raw, tensors, prompt, 6) for prompt in prompts]
        got = generate(model_folder(case), prompts, max_new_tokens=6, dtype="float32", device="cpu", block_size=8, num_blocks=26,
                       max_batch_size=3, max_num_batched_tokens=24, prefill_chunk_size=16, ops=TorchOps())
        assert got == expected
