"""Mefurax through the engine's own step function, cache manager, scheduler and entry point on the CPU (torch twins of the
kernels) against the plain implementation: configuration and weights, each mechanism, every way of cutting and batching, pages
and state slots used again, keys at the edges of windows and chunks, and greedy generation."""
import io
import json
import os
import random
import tempfile

import numpy as np
import pytest
import torch

import plain_mefurax as plain
import traces
from helpers import random_tokens
from llmserver_amd.cache import CacheManager
from llmserver_amd.config import ConfigError, UnsupportedModelError, config_from_dict
from llmserver_amd.engine.batch import StepEntry
from llmserver_amd.engine.cost import StepRow, cache_bytes
from llmserver_amd.engine.replay import make_runner, replay
from llmserver_amd.parts import PagedAndStateSpec, PagedKVSpec, StateSpec
from llmserver_amd.parts.attention import build_attention_plan, distance_slopes, group_tiling
from llmserver_amd.weights import build_model
from tiny_mefurax import CASES, MA, MB, MC, MD, ME, model_folder, plain_logits, plain_model
from torch_ops import TorchOps


def runner_for(case, max_tokens, page=None, live=4, ops=None):
    return make_runner(model_folder(case), "float32", max_tokens, page or CASES[case][2], device="cpu", ops=ops or TorchOps(), max_live=live)


def run(case, steps, tmp_path, page=None, ops=None):
    runner = runner_for(case, traces.peak_tokens(steps), page, ops=ops)
    replay(runner, traces.to_lines(steps).splitlines(), str(tmp_path), io.StringIO())
    runner.cache.check_invariants()
    assert not runner.cache.requests and runner.cache.state_slots_free() in (4, None)
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
    for raw in (MA, MB, MC, MD, ME):
        config = config_from_dict(dict(raw))
        again = config_from_dict(config.to_dict())
        assert again.layers == config.layers and again.to_dict() == config.to_dict() and again.alpha == raw["postln_alpha"]
    config = config_from_dict(dict(MA))
    assert config.layers[2].mlp is None and config.layers[0].mixer.chunk == 12 and config.layers[1].mixer.window == 9
    assert config.layers[0].mlp.shared == 28 and config.layers[3].mlp.shared is None and config.layers[1].mixer.taps == 3
    other = config_from_dict(dict(MB))
    assert other.layers[0].mixer.window is None and other.layers[1].mixer.chunk is None and not other.layers[1].mixer.v_mix
    bare = copy_of(MB)
    for key in ("softcap", "v_mix", "kv_heads"):
        bare["layers"][1]["mixer"].pop(key)
    bare = config_from_dict(bare).layers[1].mixer
    assert bare.softcap is None and bare.v_mix is False and bare.kv_heads == bare.heads

    def broken(change, error, match):
        raw = copy_of(MA)
        change(raw)
        with pytest.raises(error, match=match):
            config_from_dict(raw)

    broken(lambda c: c["layers"][1].update(type="something else"), UnsupportedModelError, "something else")
    broken(lambda c: c["layers"][1]["mlp"].update(kind="other"), UnsupportedModelError, "other")
    broken(lambda c: c.pop("postln_alpha"), ConfigError, "postln_alpha")
    broken(lambda c: c["layers"][1]["mixer"].pop("conv"), ConfigError, "conv")
    broken(lambda c: c["layers"][1]["mixer"].update(conv=0), ConfigError, "taps")
    broken(lambda c: c["layers"][1]["mixer"].update(kv_heads=3), ConfigError, "no multiple")
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5), ConfigError, "even")
    broken(lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), ConfigError, "positive")
    broken(lambda c: c["layers"][0]["mixer"].update(v_mix=1), ConfigError, "true or false")
    broken(lambda c: c["layers"][1]["mixer"].update(vdim=4), ConfigError, "values a token")
    broken(lambda c: c["layers"][1]["mixer"].update(scale=0.0), ConfigError, "scale")
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=9), ConfigError, "use 9")
    broken(lambda c: c["layers"][0]["mlp"]["shared"].pop("ff"), ConfigError, "ff")
    broken(lambda c: c["layers"][1]["mixer"].update(dim=300), UnsupportedModelError, "up to 256")
    broken(lambda c: c["layers"][1]["mixer"].update(dim=256, heads=60), UnsupportedModelError, "14336")


def test_the_model_declares_the_checkpoints_tensors_and_its_caches():
    model = build_model(config_from_dict(dict(MA)))
    specs = model.param_specs()
    assert {"embed", "head", "final.norm", "l0.norm1", "l0.norm2", "l0.mix.q", "l0.mix.g", "l0.mix.vmix", "l0.mix.o", "l0.mlp.router", "l0.mlp.e4.up",
            "l0.mlp.e4.down", "l0.mlp.shared.up", "l0.mlp.shared.down", "l1.mix.q.b", "l1.mix.v.conv", "l1.mix.q.norm", "l1.mix.vmix", "l1.mlp.gate",
            "l2.norm1"} <= set(specs)
    assert not {"l0.mix.q.b", "l0.mix.q.norm", "l0.mix.q.conv", "l0.mlp.e0.gate", "l0.mlp.shared.gate", "l0.mlp.shared.sg", "l1.mix.g", "l1.mix.o.b",
                "l2.norm2", "l3.mlp.shared.up", "l0.mlp.e5.up", "l4.norm1"} & set(specs)
    assert specs["l0.mix.g"].shape == (3, 48) and specs["l1.mix.q.norm"].shape == (24,) and specs["l1.mix.k.norm"].shape == (12,)
    assert specs["l1.mix.k.conv"].shape == (12, 3) and specs["l1.mix.v.b"].shape == (6,) and specs["l1.mix.vmix"].shape == ()
    assert specs["l0.mix.vmix"].optional and not specs["l1.mix.vmix"].optional
    assert "l1.mix.vmix" not in build_model(config_from_dict(dict(MB))).param_specs()
    caches = model.cache_specs()
    assert caches[0] == PagedKVSpec(1, 16, None, 12) and caches[2] == PagedKVSpec(2, 16, None, 21)
    assert caches[1] == PagedAndStateSpec(PagedKVSpec(2, 16, 9), StateSpec((-(-2 * 42 // 4) * 4,), "float32"))
    assert caches[3].state.shape == (-(-(6 * 5 + 3 * 5 + 6) // 4) * 4,)
    # a convolution of one tap keeps nothing
    assert build_model(config_from_dict(dict(MB))).cache_specs()[2] == PagedKVSpec(1, 32, 30)


# -- chunks in the cache manager, the plan and the costs -----------------------------------------------------------------
def test_pages_of_a_chunk_are_given_back_when_the_next_one_begins():
    cache = CacheManager({0: PagedKVSpec(1, 16, chunk=10), 1: PagedKVSpec(1, 16)}, 4, 16, allocate_storage=False)
    cache.open("a")
    held = []
    for count in range(1, 26):
        cache.ensure("a", count)
        cache.advance("a", count)
        held.append([page >= 0 for page in cache.record("a").tables[0]])
        cache.check_invariants()
    # the next token stands at position `count`: everything from its chunk's first position on is still there
    for count, listed in zip(range(1, 26), held):
        first = count // 10 * 10
        assert listed == [4 * (block + 1) > first for block in range(len(listed))], (count, listed)
    assert all(page >= 0 for page in cache.record("a").tables[1]) and not cache.prefix_caching_possible
    cache.close("a")
    assert cache.available_pages() == [16, 16]
    both = PagedKVSpec(1, 16, window=7, chunk=10)
    assert [both.first_key(p) for p in (0, 5, 9, 10, 13, 19, 20)] == [0, 0, 3, 10, 10, 13, 20] and both.bounded
    assert not PagedKVSpec(1, 16).bounded and PagedKVSpec(1, 16).first_key(100) == 0


@pytest.mark.parametrize("seed", range(30))
def test_every_token_meets_the_keys_of_its_chunk_exactly_once(seed):
    rng = random.Random(seed)
    group, n_kv, chunk = rng.choice([1, 2, 5, 16, 20]), rng.choice([1, 2, 8]), rng.choice([1, 7, 32, 64, 500, 3000])
    window = rng.choice([None, None, 40])
    spec = PagedKVSpec(1, 16, window, chunk)
    single = seed % 3 == 0
    rows = rng.randint(1, 8)
    row_len = [1 if single else rng.choice([1, 1, 2, 33, 200, 900]) for _ in range(rows)]
    row_ctx = [n + rng.choice([0, 0, 5, 64, 1000, 5000]) for n in row_len]
    options = dict(workgroup_tiles=rng.choice([0, 4, 8]), tile_key_ranges=rng.choice([1, 128]), tile_halves=rng.choice([1, 2]))
    if single:
        options = dict(fixed_splits=rng.choice([1, 3, 8]), single_token_shortcut=rng.random() < 0.7)
    plan = build_attention_plan(row_len, row_ctx, group, n_kv, window, chunk=chunk, **options)
    _, per_tile, _ = group_tiling(group)
    met = {}
    for entries, span in ((plan.items, per_tile), (plan.tiles, plan.tiles_per_workgroup * per_tile)):
        for row, q0, k_begin, k_end in entries.tolist():
            for token in range(q0, min(q0 + span, row_len[row])):
                met.setdefault((row, token), []).append((k_begin, k_end))
    for row in range(rows):
        for token in range(row_len[row]):
            position = row_ctx[row] - row_len[row] + token
            keys = [key for lo, hi in met[(row, token)] for key in range(max(lo, spec.first_key(position)), min(hi, position + 1))]
            assert sorted(keys) == list(range(spec.first_key(position), position + 1)), (row, token)
            # nothing before the first token's chunk of the workgroup's tiles is touched: those pages may be gone
            assert min(lo for lo, hi in met[(row, token)] if lo < hi) >= spec.first_key(row_ctx[row] - row_len[row])


def test_the_costs_count_a_chunks_keys_only():
    model = build_model(config_from_dict(dict(ME)))          # a window of 6, chunks of 5 and of 1
    rows = [StepRow(1, 14), StepRow(1, 3)]
    row_bytes = lambda heads, size, keys: 2 * heads * size * 4 * keys
    state = 4 * (-(-4 * (2 * 6 * 2 + 2 * 7) // 4) * 4)
    assert cache_bytes(model, rows, torch.float32) == row_bytes(2, 16, 6 + 3) + row_bytes(3, 16, 4 + 3) + row_bytes(1, 32, 1 + 1) + 2 * state
    mixer = model.blocks[1].mixer
    assert mixer.mixing_flops(3, 12) == 2.0 * 3 * (4 + 9) * (5 + 1 + 2)           # positions 9, 10 and 11: five keys, one, two


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


def test_the_shared_experts_products_made_inside_the_kernels_give_the_same(tmp_path):
    ops = TorchOps()
    ops.inside_shared = True
    for case in ("MA", "MC"):
        requests = requests_of(case, (20, 3))
        check(case, run(case, traces.changing_portions(requests, sizes=(2, 7, 1, 3, 2)), tmp_path / case, ops=ops), requests)


def test_the_stream_behind_every_layer_is_the_plain_implementations():
    raw, tensors = plain_model("MA")
    tokens = random_tokens(97, 23, 2)
    kept = []
    plain.forward(raw, tensors, tokens, keep=kept)
    runner = runner_for("MA", 64)
    runner.cache.open("r")
    seen = []
    runner.model.after_call = lambda index, stream, pending: seen.append(stream.clone())
    runner.step([StepEntry("r", tokens, [])])
    assert len(seen) == len(kept) == 4
    for index, (got, expected) in enumerate(zip(seen, kept)):
        np.testing.assert_allclose(got.numpy(), expected.numpy(), atol=5e-5, rtol=1e-4, err_msg=f"layer {index}")


def test_prefill_equals_token_by_token_decoding_from_the_first_token(tmp_path):
    for case in ("MA", "MB", "MC", "ME"):
        requests = requests_of(case, (60,))
        check(case, run(case, traces.tail_decoded(requests, 64), tmp_path / case), requests)


def test_long_decoding(tmp_path):
    """A prompt of one token and 300 decoded ones: windows and chunks go by many times, their pages are given back and used again."""
    requests = requests_of("MC", (301,))
    steps = traces.tail_decoded(requests, 300)
    check("MC", run("MC", steps, tmp_path), requests)


@pytest.mark.parametrize("page", [4, 8, 64])
def test_page_sizes_and_page_borders(page, tmp_path):
    requests = requests_of("MA", (2 * page + 1, page, page - 1, page + 1))
    steps = traces.changing_portions(requests, sizes=(page - 1, 2, page, 1, page + 1))
    check("MA", run("MA", steps, tmp_path, page=page), requests)


@pytest.mark.parametrize("case,sizes", [("MA", (9, 12, 17, 21)), ("MC", (40, 48, 32, 100)), ("ME", (5, 6))])
def test_portions_that_end_at_and_around_the_edges_of_windows_and_chunks(case, sizes, tmp_path):
    longest = 3 * max(sizes) + 5
    requests = requests_of(case, (longest,) * (3 * len(sizes)))
    steps = []
    for (rid, tokens), (size, off) in zip(requests.items(), [(size, off) for size in sizes for off in (-1, 0, 1)]):
        cuts = sorted({0, longest, *(min(longest, max(0, k * size + off)) for k in range(1, 4))})
        for start, end in zip(cuts, cuts[1:]):
            steps.append({"step": len(steps), "entries": [{"id": rid, "tokens": tokens[start:end], "want": list(range(end - start))}],
                          "end": [rid] if end == longest else []})
    check(case, run(case, steps, tmp_path), requests)


def test_state_slots_and_pages_are_used_again_in_any_order():
    """Eight requests through four slots and pages for four: a slot's next holder must start from zeros before its first token,
    not from its predecessor's last inputs; batches of unequal portions in changing order."""
    runner = runner_for("MA", 4 * 64, live=4)
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
        expected = plain_logits("MA", tuple(tokens[rid]))[position].numpy()
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
def sharp_keys(tensors):
    """Queries that decide: norms' weights of the sloped layers scaled up, so that one key of the window stands out."""
    for name in list(tensors):
        if name.endswith("q.norm"):
            tensors[name] *= 6.0


def long_reach(raw):
    """Windows of 150 keys (the flattest head loses 2^-8 a position) and chunks of 160, whose scores are sharp, too."""
    for layer in raw["layers"]:
        sizes = layer["mixer"]
        if layer["type"] == "attention":
            sizes["mask"] = {"size": 150}
        else:
            sizes["mask"] = {"size": 160}
            sizes["scale"], sizes["softcap"] = 3.0, 60.0


def oldest_tap(tensors):
    for name in list(tensors):
        if name.endswith(".conv"):
            tensors[name][:, 1:] *= 0.05
            tensors[name][:, 0] *= 6.0


SHARP = {"far key": ("MC", sharp_keys, long_reach, 330), "oldest tap": ("MA", oldest_tap, None, 60), "oldest of six taps": ("MB", oldest_tap, None, 60)}


def test_keys_more_than_a_hundred_tokens_back_decide():
    """Sharp queries under windows and chunks longer than a hundred tokens: other tokens 110 to 139 places back change the logits."""
    case, change, change_config, length = SHARP["far key"]
    folder, raw, tensors = sharpened(case, change, change_config)
    tokens = random_tokens(200, length, 5)
    expected = plain.forward(raw, tensors, tokens).numpy()
    last = length - 1                                  # position 329: its chunk begins at 320, its window at 180
    changed = tokens[:190] + random_tokens(200, 30, 77) + tokens[220:]
    assert np.abs(plain.forward(raw, tensors, changed).numpy()[last] - expected[last]).max() > 1e-2
    for cuts in ([330], [300] + [1] * 30, [3, 147, 2, 8, 50, 100, 20]):
        np.testing.assert_allclose(logits_of(folder, tokens, cuts, page=16), expected, atol=2e-4, rtol=5e-4, err_msg=str(cuts))


@pytest.mark.parametrize("name", ["oldest tap", "oldest of six taps"])
def test_the_convolutions_oldest_tap_reaches_over_earlier_steps(name):
    """Nearly all of a convolution's weight on its oldest tap: portions shorter than its reach, single tokens, and both."""
    case, change, _, length = SHARP[name]
    folder, raw, tensors = sharpened(case, change)
    tokens = random_tokens(raw["vocab"], length, 9)
    expected = plain.forward(raw, tensors, tokens).numpy()
    moved = {n: (torch.roll(t, 1, dims=1) if n.endswith(".conv") else t) for n, t in tensors.items()}
    assert np.abs(plain.forward(raw, moved, tokens).numpy() - expected).max() > 1e-2
    for cuts in ([60], [1] * 60, [2] * 30, [2, 1, 3, 4, 5, 1, 1, 6, 2, 35], [59, 1]):
        np.testing.assert_allclose(logits_of(folder, tokens, cuts), expected, atol=1.5e-4, rtol=3e-4, err_msg=str(cuts))


def planted(module_changes, case="MA", count=50, change_config=None, threshold=3e-3):
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


def test_windows_and_chunks_end_where_they_should():
    for layer in (0, 1, 2, 3):
        for off in (-1, 1):
            planted({}, change_config=lambda raw, layer=layer, off=off: raw["layers"][layer]["mixer"]["mask"].update(
                size=raw["layers"][layer]["mixer"]["mask"]["size"] + off))
    # a chunk is no window, and is counted from the sequence's first position
    planted({"in_chunk": lambda kept: plain.in_window})
    shifted = lambda kept: lambda n, size: (lambda place: (place[:, None] >= place[None, :]) & ((place[:, None] + 1) // size == (place[None, :] + 1) // size))(torch.arange(n))
    planted({"in_chunk": shifted})
    planted({"in_window": lambda kept: lambda n, size: kept(n, None)})


def test_scores_fall_with_the_distance_by_heads():
    assert distance_slopes(8) == [0.5, 0.25, 0.125, 0.0625, 2.0 ** -5, 2.0 ** -6, 2.0 ** -7, 2.0 ** -8]
    assert distance_slopes(3) == pytest.approx([2.0 ** (-8 / 3), 2.0 ** (-16 / 3), 2.0 ** -8])
    planted({"slopes": lambda kept: lambda heads: [0.0] * heads})
    planted({"slopes": lambda kept: lambda heads: kept(heads)[::-1]})
    planted({"slopes": lambda kept: lambda heads: [2.0 ** (-8.0 * h / heads) for h in range(heads)]})


def test_values_are_mixed_with_the_first_layers():
    """Mixed with the layer before instead, the wrong way round, not at all, or with the first values already convolved away."""
    def with_the_layer_before(kept):
        def mixed(v, t, p, sizes, firsts, r=plain.same):
            out = kept(v, t, p, sizes, firsts, r)
            if sizes.get("v_mix"):
                firsts[:] = [out]
            return out
        return mixed

    def other_way_round(kept):
        def mixed(v, t, p, sizes, firsts, r=plain.same):
            return kept(v, {**t, p + "vmix": 1.0 - t[p + "vmix"]} if sizes.get("v_mix") else t, p, sizes, firsts, r)
        return mixed

    for case in ("MA", "MB"):
        planted({"mixed_values": other_way_round}, case=case)
    planted({"mixed_values": with_the_layer_before})
    planted({}, change_config=lambda raw: raw["layers"][1]["mixer"].update(v_mix=False))
    planted({"mixed_values": lambda kept: lambda v, t, p, sizes, firsts, r=plain.same: v})
    # the first layer's own number is not used
    raw, tensors = plain_model("MA")
    tokens = random_tokens(97, 20, 3)
    np.testing.assert_array_equal(plain.forward(raw, {**tensors, "l0.mix.vmix": tensors["l0.mix.vmix"] + 5.0}, tokens).numpy(), plain.forward(raw, tensors, tokens).numpy())
    folder, _, _ = sharpened("MA", lambda t: t.pop("l0.mix.vmix"))             # and a folder may leave it out
    np.testing.assert_allclose(logits_of(folder, tokens, [20]), plain.forward(raw, tensors, tokens).numpy(), atol=1.5e-4, rtol=3e-4)


def test_projections_are_convolved_before_they_are_normed_as_a_whole():
    def normed_first(kept):
        def attention(h, t, p, sizes, eps, firsts, r=plain.same):
            count = {name: t[p + name + ".conv"] for name in "qkv"}
            inner = plain.convolved
            try:
                plain.convolved = lambda u, taps: inner(plain.unit_root_mean_square(u, eps), taps) if any(taps is count[name] for name in "qk") else inner(u, taps)
                return kept(h, t, p, sizes, eps, firsts, r)
            finally:
                plain.convolved = inner
        return attention

    planted({"attention": normed_first})
    planted({"convolved": lambda kept: lambda u, taps: kept(u, taps.flip(1))})
    planted({"projected": lambda kept: lambda h, t, name, r=plain.same: r(h @ t[name].T)})
    # the norm runs over the heads together
    planted({"norm": lambda kept: lambda x, w, eps: torch.cat([plain.unit_root_mean_square(part, eps) for part in x.split(x.shape[1] // 2, dim=1)], dim=1) * w})
    planted({"norm": lambda kept: lambda x, w, eps: kept(x, 1.0 + w, eps)})


def test_chunked_heads_are_turned_in_neighbouring_pairs_normed_capped_and_gated():
    def halves(kept):
        def rotate(x, positions, dims, base):
            order = [i // 2 + (i % 2) * dims // 2 for i in range(dims)] + list(range(dims, x.shape[-1]))
            turned = kept(x[..., order], positions, dims, base)
            return turned[..., [order.index(i) for i in range(x.shape[-1])]]
        return rotate

    planted({"rotate_pairs": halves})
    planted({"rotate_pairs": lambda kept: lambda x, positions, dims, base: x})
    planted({}, change_config=lambda raw: [raw["layers"][i]["mixer"].update(softcap=1e6) for i in (0, 2)])
    planted({"unit_root_mean_square": lambda kept: lambda x, eps: x if x.dim() == 3 else kept(x, eps)})
    planted({"projected": lambda kept: lambda h, t, name, r=plain.same: kept(h, t, name, r) * (0.0 if name.endswith(".g") else 1.0)})


def test_the_norm_stands_behind_the_scaled_sum_and_its_weight_around_zero():
    planted({"norm_around_zero": lambda kept: lambda x, w, eps: kept(x, w - 1.0, eps)})
    planted({}, change_config=lambda raw: raw.update(postln_alpha=1.0))


def test_experts_square_the_rectifier_and_the_chosen_logits_alone_weigh():
    planted({"relu_squared": lambda kept: lambda z: torch.clamp(z, min=0.0)})
    planted({"gelu_tanh": lambda kept: lambda z: z * torch.sigmoid(z)})
    planted({"experts": lambda kept: lambda h, read, t, p, mlp, r=plain.same: kept(h, read, t, p, {**mlp, "shared": None}, r)})

    def over_all(kept):
        def route(h, t, p, router):
            logits = h @ t[p + "router"].T
            chosen = torch.topk(logits, router["top"], dim=-1).indices
            return chosen, torch.softmax(logits, dim=-1).gather(1, chosen)
        return route
    planted({"route": over_all})


# -- the oracle itself -------------------------------------------------------------------------------------------------
def test_the_oracles_mechanisms_by_hand():
    f64 = lambda values: torch.tensor(values, dtype=torch.float64)
    assert torch.allclose(plain.norm(f64([[3.0, 4.0]]), f64([1.0, 2.0]), 0.0), f64([[3.0, 8.0]]) / 12.5 ** 0.5)
    assert torch.allclose(plain.norm_around_zero(f64([[3.0, 4.0]]), f64([0.0, 1.0]), 0.0), f64([[3.0, 8.0]]) / 12.5 ** 0.5)
    # four dimensions of five turn: (0, 1) by p, (2, 3) by p / base^(1/2)
    a, b = 3.0, 3.0 / 100.0 ** 0.5
    turned = plain.rotate_pairs(f64([[[1.0, 2.0, 3.0, 4.0, 7.0]]]), torch.tensor([3]), 4, 100.0)
    assert torch.allclose(turned, f64([[[np.cos(a) - 2 * np.sin(a), 2 * np.cos(a) + np.sin(a), 3 * np.cos(b) - 4 * np.sin(b), 4 * np.cos(b) + 3 * np.sin(b), 7.0]]]))
    # a convolution of two taps: the last column meets the token itself; zeros before the start
    assert torch.allclose(plain.convolved(f64([[1.0], [2.0], [5.0]]), f64([[10.0, 1.0]])), f64([[1.0], [12.0], [25.0]]))
    assert plain.in_window(4, 2).tolist() == [[True, False, False, False], [True, True, False, False], [False, True, True, False], [False, False, True, True]]
    assert plain.in_chunk(4, 3).tolist() == [[True, False, False, False], [True, True, False, False], [True, True, True, False], [False, False, False, True]]
    # one head: equal keys, scores fall by the slope: weights 1 and e^-2 over two visible keys
    out = plain.attend(f64([[[1.0]]] * 2), f64([[[0.0]]] * 2), f64([[[10.0]], [[20.0]]]), {"heads": 1, "kv_heads": 1, "scale": 1.0},
                       lambda s: s - 2.0 * f64([[0.0, 0.0], [1.0, 0.0]]), plain.in_window(2, None))
    assert torch.allclose(out.flatten(), f64([10.0, (20.0 + 10.0 * np.exp(-2.0)) / (1.0 + np.exp(-2.0))]))
    # two query heads share a key/value head
    out = plain.attend(f64([[[1.0], [2.0], [1.0], [2.0]]]), f64([[[0.0], [0.0]]]), f64([[[3.0], [4.0]]]), {"heads": 4, "kv_heads": 2, "scale": 1.0}, lambda s: s,
                       plain.in_chunk(1, 1))
    assert out.flatten().tolist() == [3.0, 3.0, 4.0, 4.0]
    # values: the first layer's stay, later ones are mixed
    firsts = []
    assert plain.mixed_values(f64([1.0]), {"a.vmix": f64(9.0)}, "a.", {"v_mix": True}, firsts) == f64([1.0])
    assert torch.allclose(plain.mixed_values(f64([5.0]), {"b.vmix": f64(0.25)}, "b.", {"v_mix": True}, firsts), f64([4.0]))
    assert plain.mixed_values(f64([7.0]), {}, "c.", {}, firsts) == f64([7.0])
    # the router: logits 0, ln 3 and -5, two chosen: weights 1/4 and 3/4
    chosen, weights = plain.route(f64([[1.0]]), {"p.router": f64([[0.0], [np.log(3.0)], [-5.0]])}, "p.", {"top": 2})
    assert chosen.tolist() == [[1, 0]] and torch.allclose(weights, f64([[0.75, 0.25]]))
    assert plain.relu_squared(f64([-2.0, 3.0])).tolist() == [0.0, 9.0]
    assert torch.allclose(plain.gelu_tanh(f64([1.0])), f64([0.841192]), atol=1e-6)


# -- generation through the entry point, the scheduler and the engine ------------------------------------------------------
def test_greedy_generation_through_the_entry_point_equals_the_oracles():
    """More requests than places, prompts cut into portions by the token budget, a pool so small that requests wait
    for pages: the engine's own scheduler, cache manager, step function and sampler produce the oracle's tokens."""
    from llmserver_amd.entrypoints import generate
    for case, vocab in (("MA", 97), ("MB", 130)):
        raw, tensors = plain_model(case)
        prompts = [random_tokens(vocab, n, 700 + n) for n in (19, 3, 41, 8, 1, 27)]
        expected = [plain.greedy_generate(raw, tensors, prompt, 6) for prompt in prompts]
        got = generate(model_folder(case), prompts, max_new_tokens=6, dtype="float32", device="cpu", block_size=8, num_blocks=26,
                       max_batch_size=3, max_num_batched_tokens=24, prefill_chunk_size=16, ops=TorchOps())
        assert got == expected
