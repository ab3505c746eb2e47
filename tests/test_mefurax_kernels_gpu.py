"""The kernels that Mefurax brought: queries, keys and values composed from the product (short convolutions with state, norms
over heads and over whole projections, rotations, mixed values, the cache write), attention under chunks, scores that fall
with the distance and gates a head, the norm behind a scaled sum, and routed experts without gates beside a shared one; each
against its plain torch twin, in float32 and in bfloat16, on sizes that are no multiples of anything as well as on those the
faster forms take."""
import math

import numpy as np
import pytest
import torch

from llmserver_amd.parts.attention import build_attention_plan, distance_slopes
from test_latent_experts_kernels_gpu import batch, close
from torch_ops import TorchOps

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(scope="module")
def ops():
    from llmserver_amd.kernels import default_ops
    return default_ops()


class Ctx:
    def empty(self, shape, dtype=None):
        return torch.empty(shape, device="cuda", dtype=dtype)


def both(ops, outs, call):
    made = [outs(), outs()]
    for which, out in zip((ops, TorchOps()), made):
        call(which, out)
    return made


# (query heads, key/value heads, dim, value dim, extra columns behind the channels)
SHAPES = [(4, 2, 64, 64, 8), (2, 1, 128, 96, 0), (3, 3, 24, 40, 3), (4, 4, 16, 32, 4), (5, 1, 7, 10, 0), (6, 3, 40, 8, 8), (8, 8, 8, 16, 0), (2, 2, 256, 24, 0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n_q,n_kv,dim,vdim,extra", SHAPES)
@pytest.mark.parametrize("taps", [None, 1, 2, 3, 4, 6])
def test_queries_keys_and_values_over_steps_and_slots(ops, dtype, n_q, n_kv, dim, vdim, extra, taps):
    """Rows of unequal portions (shorter than the taps reach, too), steps of one token a row that move the state on
    themselves, a portion long enough for values in tiles, a request that starts again in a used slot; norms of either span
    with and without weights, rotations of either pairing, values mixed with another layer's and kept for others."""
    print(f"qkv_compose {dtype} {n_q}/{n_kv} {dim}/{vdim} taps {taps}", flush=True)
    torch.manual_seed(dim + (taps or 0))
    page, row = 8, -(-max(dim, vdim) // 16) * 16
    channels = n_q * dim + n_kv * (dim + vdim)
    slots = torch.tensor([2, 0, 3], dtype=torch.int32, device="cuda")
    weights = None if taps is None else 0.5 * torch.randn(taps, channels, device="cuda")
    kept = max((taps or 1) - 1, 0)
    states = [torch.randn(4, -(-kept * channels // 4) * 4 + 4, device="cuda") for _ in range(2)]
    states[1].copy_(states[0])
    pages = 150
    table = torch.randperm(pages, device="cuda").to(torch.int32)[:120].view(3, 40)
    pools = [(torch.randn(pages, n_kv, page, row, device="cuda").to(dtype), torch.randn(pages, n_kv, row, page, device="cuda").to(dtype))]
    pools.append(tuple(tensor.clone() for tensor in pools[0]))
    firsts = [0, 0, 0]
    pairs = [0, dim // 4, dim // 2]
    for step, lengths in enumerate(([5, 1, 37], [1, 1, 1], [1, 2, 2], [1, 1, 1], [18, 0, 2], [150, 3, 120], [1, 1, 1])):
        if step == 3:
            firsts[1] = 0                          # the second request ends; another one starts in its slot
        token_row, positions, row_start, row_len, row_ctx = batch(lengths, firsts, "cuda")
        n = sum(lengths)
        qkv = torch.randn(n, channels + extra, device="cuda").to(dtype)
        span = (None, "head", "projection")[step % 3]
        q_weight = k_weight = None
        if span is not None and step % 2:
            q_weight, k_weight = (1 + 0.3 * torch.randn(dim if span == "head" else heads * dim, device="cuda") for heads in (n_q, n_kv))
        turned = pairs[step % 3]
        cos_sin = ops.rotary_table(positions, 50.0 ** (-torch.arange(turned, device="cuda").float() / max(turned, 1))) if turned else None
        other = torch.randn(n, n_kv * vdim + extra, device="cuda").to(dtype)[:, :n_kv * vdim] if step % 2 else None
        single = max(lengths) == 1 == min(lengths)
        outs = []
        for which, state, (keys, values) in zip((ops, TorchOps()), states, pools):
            out_q = torch.full((n, n_q * row), float("nan"), device="cuda", dtype=dtype)
            own = torch.full((n, n_kv * vdim), float("nan"), device="cuda", dtype=dtype) if step != 1 else None
            which.qkv_compose(qkv, weights, state if kept else None, slots, token_row, positions, row_start, q_weight, k_weight, span, 1e-5, cos_sin,
                              "halves" if step in (1, 5) else "neighbours", keys, values, table, page, n_q, n_kv, dim, vdim, out_q, mix=0.3 if step % 2 else 0.0,
                              first=other, own_values=own, keep=single and kept > 0)
            if kept and not single:
                which.delta_conv_keep(qkv, channels, taps, state, 0, slots, row_start, row_len, row_ctx)
            outs.append((out_q, own))
        close(outs[0][0], outs[1][0], dtype, f"queries, step {step}")
        if outs[0][1] is not None:
            close(outs[0][1], outs[1][1], dtype, f"values kept, step {step}")
        close(pools[0][0], pools[1][0], dtype, f"keys, step {step}")
        close(pools[0][1], pools[1][1], dtype, f"values, step {step}")
        close(states[0], states[1], torch.float32, f"state, step {step}")
        firsts = [f + n for f, n in zip(firsts, lengths)]


@pytest.mark.parametrize("dtype", DTYPES)
def test_composed_rows_do_not_depend_on_how_tokens_are_cut(ops, dtype):
    """The same bits for a token whether it comes in a long portion (four tokens a workgroup, values in tiles), in portions or
    alone, in the form that keeps pieces in registers."""
    n_q, n_kv, dim, vdim, page, n, taps = 4, 2, 64, 64, 16, 300, 3
    channels = n_q * dim + n_kv * (dim + vdim)
    qkv = torch.randn(n, channels, device="cuda").to(dtype)
    weights = torch.randn(taps, channels, device="cuda")
    q_weight, k_weight = torch.rand(n_q * dim, device="cuda"), torch.rand(n_kv * dim, device="cuda")
    slots = torch.zeros(1, dtype=torch.int32, device="cuda")
    table = torch.randperm(19, device="cuda").to(torch.int32).view(1, 19)
    results = []
    for cuts in ([n], [1] * 40 + [257, 3], [7, 270, 2, 1, 1, 19]):
        state = torch.full((1, 2 * channels), float("nan"), device="cuda")          # (nothing is read that has not been written)
        keys, values = torch.zeros(19, n_kv, page, dim, device="cuda", dtype=dtype), torch.zeros(19, n_kv, vdim, page, device="cuda", dtype=dtype)
        queries, at = [], 0
        for count in cuts:
            token_row, positions, row_start, row_len, row_ctx = batch([count], [at], "cuda")
            out_q = torch.empty(count, n_q * dim, device="cuda", dtype=dtype)
            part = qkv[at:at + count].contiguous()
            ops.qkv_compose(part, weights, state, slots, token_row, positions, row_start, q_weight, k_weight, "projection", 1e-6, None, "neighbours",
                            keys, values, table, page, n_q, n_kv, dim, vdim, out_q, keep=count == 1)
            if count > 1:
                ops.delta_conv_keep(part, channels, taps, state, 0, slots, row_start, row_len, row_ctx)
            queries.append(out_q)
            at += count
        results.append((torch.cat(queries), keys, values))
    for other in results[1:]:
        for a, b in zip(results[0], other):
            assert torch.equal(a, b)


def chunked_case(ops, dtype, n_q, n_kv, d, page, lens, ctxs, window=None, chunk=None, sloped=False, gated=False, softcap=None, seed=0, **plan_options):
    """Random q/k/v through both implementations; pages in scrambled order from a pool that held other data, pages that no query
    sees any longer are gone from the tables; the oldest key the first query sees dominates its softmax."""
    torch.manual_seed(seed)
    rows, tokens = len(lens), sum(lens)
    n_pages = sum(-(-c // page) for c in ctxs) + 3
    keys = (5 * torch.randn(n_pages, n_kv, page, d, device="cuda")).to(dtype)
    values = (5 * torch.randn(n_pages, n_kv, d, page, device="cuda")).to(dtype)
    perm, used = torch.randperm(n_pages), 0
    table = torch.full((rows, max(-(-c // page) for c in ctxs)), -1, dtype=torch.int32)
    q = torch.randn(tokens, n_q * d, device="cuda").to(dtype)
    row_start = np.cumsum([0] + list(lens[:-1])).astype(np.int32)
    for r, c in enumerate(ctxs):
        blocks, position = -(-c // page), c - lens[r]
        far = max(0 if window is None else position - window + 1, 0 if chunk is None else position // chunk * chunk, 0)
        table[r, :blocks] = perm[used:used + blocks].int()
        used += blocks
        k, v = torch.randn(c, n_kv, d, device="cuda"), torch.randn(c, n_kv, d, device="cuda")
        head = q[row_start[r], :d].float()
        k[far, 0] = 6.0 * head / head.norm() * math.sqrt(d)
        v[far, 0] = 10.0
        place = torch.arange(c)
        at = table[r].long()[place // page].cuda()
        keys[at, :, (place % page).cuda(), :] = k.to(dtype)
        values[at, :, :, (place % page).cuda()] = v.to(dtype)
        table[r, :far // page] = -1
    tiles = ops.attention_workgroup_tiles(dtype, d, page) if plan_options.pop("tiles", True) else 0
    plan = build_attention_plan(lens, ctxs, n_q // n_kv, n_kv, window, workgroup_tiles=tiles, chunk=chunk, tuning=ops.attention_tuning_for(dtype, d),
                                tile_halves=ops.attention_tile_halves(dtype, d) if tiles else 1,
                                tile_key_ranges=ops.attention_tile_key_ranges(dtype, d) if tiles else 1, **plan_options)
    staged = {name: torch.from_numpy(getattr(plan, name)).cuda() for name in ("items", "item_slot", "merges", "tiles")}
    staged.update(n_tiles=len(plan.tiles), n_items=len(plan.items), n_merges=len(plan.merges), n_slots=plan.n_slots,
                  tiles_per_workgroup=plan.tiles_per_workgroup, tile_halves=plan.tile_halves, merge_in_workgroup=int(plan.merge_in_workgroup),
                  most_splits=int(plan.merges[:, 3].max()) if len(plan.merges) else 0)
    if plan.tile_slots is not None:
        staged["tile_slots"] = torch.from_numpy(plan.tile_slots).cuda()
    t = lambda a: torch.tensor(np.asarray(a), dtype=torch.int32, device="cuda")
    slopes = torch.tensor(distance_slopes(n_q), device="cuda") if sloped else None
    gates = torch.randn(tokens, n_q + 3, device="cuda").to(dtype)[:, 2:2 + n_q] if gated else None
    table = table.cuda()
    outs = both(ops, lambda: torch.zeros(tokens, n_q * d, device="cuda", dtype=dtype),
                lambda which, out: which.paged_attention(q, out, keys, values, table if which is ops else table.clamp(min=0), t(row_start), t(lens), t(ctxs),
                                                         staged, d ** -0.5, window, page, n_q, n_kv, d, Ctx(), softcap=softcap, chunk=chunk, slopes=slopes,
                                                         gates=gates))
    torch.cuda.synchronize()
    assert torch.isfinite(outs[0].float()).all()
    close(outs[0], outs[1], dtype, "attention")
    return plan


FORMS = [dict(chunk=64, gated=True, softcap=30.0), dict(window=50, sloped=True), dict(chunk=33, sloped=True, gated=True), dict(chunk=200, window=70, gated=True),
         dict(sloped=True)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n_q,n_kv,d,page", [(4, 2, 16, 16), (6, 2, 48, 12), (16, 8, 128, 16), (5, 1, 80, 8), (3, 3, 64, 4), (20, 1, 64, 16), (2, 1, 256, 16)])
@pytest.mark.parametrize("form", range(len(FORMS)))
def test_attention_under_chunks_slopes_and_gates(ops, dtype, n_q, n_kv, d, page, form):
    """Portions beside single tokens; prompts in workgroups of tiles with their keys whole, in halves and in ranges of their own;
    single tokens with keys whole, split, and merged in the workgroup."""
    print(f"attention {dtype} {n_q}/{n_kv} d{d} page {page} {FORMS[form]}", flush=True)
    options = FORMS[form]
    chunked_case(ops, dtype, n_q, n_kv, d, page, [5, 1, 20, 1], [17, 300, 193, 64], **options)
    plan = chunked_case(ops, dtype, n_q, n_kv, d, page, [300, 130], [300, 700], **options)
    if page % 8 == 0:
        assert len(plan.tiles) or dtype == torch.float32
    chunked_case(ops, dtype, n_q, n_kv, d, page, [260], [1500], target_waves=4, tiles=False, **options)
    for splits in (1, 3):
        chunked_case(ops, dtype, n_q, n_kv, d, page, [1, 1, 1, 1], [700, 65, 1, 129], fixed_splits=splits, **options)
    for ranges in (4, 2):
        chunked_case(ops, dtype, n_q, n_kv, d, page, [1, 1, 1, 1], [700, 64, 1, 128], fixed_splits=ranges, merge_in_workgroup=ranges, **options)


@pytest.mark.parametrize("halves,walk,per", [(1, None, 4), (2, None, 8), (2, None, 4), (1, 8, 8), (1, None, 8), (2, 8, 4)])
@pytest.mark.parametrize("form", range(len(FORMS)))
def test_every_way_of_the_prompt_kernel(ops, halves, walk, per, form, monkeypatch):
    from llmserver_amd.parts import attention as attention_module
    print(f"prompt kernel {halves} {walk} {per} {FORMS[form]}", flush=True)
    monkeypatch.setattr(attention_module, "_workgroup_tiles_that_pay", lambda *args, **kwargs: (per, halves, walk))
    plan = chunked_case(ops, torch.bfloat16, 4, 2, 64, 16, [400, 270], [400, 1333], **FORMS[form])
    assert len(plan.tiles) and plan.tile_halves == halves


@pytest.mark.parametrize("chunk", [1, 7, 16, 40, 64, 100])
@pytest.mark.parametrize("dtype", DTYPES)
def test_attention_at_the_edges_of_chunks(ops, dtype, chunk):
    """Contexts that end at, just before and just behind a chunk's edge, in prompts and one token at a time."""
    print(f"edges {dtype} {chunk}", flush=True)
    for ctx in (chunk, chunk + 1, 2 * chunk, 3 * chunk - 1, 3 * chunk + 1):
        chunked_case(ops, dtype, 4, 2, 32, 8, [1, min(ctx, 20)], [ctx, ctx], chunk=chunk)


def test_attention_refuses_slopes_it_cannot_take(ops):
    with pytest.raises(ValueError, match="positive scale"):
        z = torch.zeros(1, 64, device="cuda")
        ops.paged_attention(z, z, z, z, z, z, z, z, {}, 0.0, None, 16, 4, 4, 16, Ctx(), slopes=torch.zeros(4, device="cuda"))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rounded", [None, torch.bfloat16, torch.float32])
@pytest.mark.parametrize("width", [1, 100, 257, 1024, 4096, 5004, 9001])
def test_the_norm_behind_a_scaled_sum(ops, dtype, rounded, width):
    n = 9
    x, y, weight = torch.randn(n, width, device="cuda"), torch.randn(n, width, device="cuda").to(dtype), 1 + 0.3 * torch.randn(width, device="cuda")
    for in_place in (True, False):
        got, want = both(ops, lambda: (x.clone(), torch.zeros(n, width, device="cuda"), torch.zeros(n, width, device="cuda", dtype=rounded or dtype)),
                         lambda which, out: which.sum_norm(out[0], y, 2.5, weight, 1e-5, out[0] if in_place else out[1], rounded=out[2] if rounded else None))
        for a, b, kind in zip(got, want, (torch.float32, torch.float32, rounded or dtype)):
            close(a, b, kind, "sum_norm")
        if rounded:
            assert torch.equal(got[2], got[0 if in_place else 1].to(rounded))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,top,shared,inter,width", [(5, 2, 28, 32, 64), (8, 3, 64, 96, 128), (3, 3, None, 20, 50), (64, 6, 96, 64, 64), (1, 1, 32, 32, 32),
                                                            (9, 4, 17, 33, 77)])
@pytest.mark.parametrize("n", [1, 3, 9, 40, 200])
def test_routed_experts_without_gates(ops, dtype, experts, top, shared, inter, width, n):
    """Both ways of the products: pair by pair with the shared expert inside or ready made, and sorted by expert."""
    print(f"experts {dtype} {experts} top {top} shared {shared} {inter} {width} n {n}", flush=True)
    twin = TorchOps()
    x = torch.randn(n, width, device="cuda").to(dtype)
    chosen = torch.stack([torch.randperm(experts, device="cuda")[:top] for _ in range(n)]).to(torch.int32)
    weights = torch.rand(n, top, device="cuda")
    up = (0.2 * torch.randn(experts, inter, width, device="cuda")).to(dtype)
    down = (0.2 * torch.randn(experts, width, inter, device="cuda")).to(dtype)
    s_up = (0.2 * torch.randn(shared or 1, width, device="cuda")).to(dtype)
    s_down = (0.2 * torch.randn(width, shared or 1, device="cuda")).to(dtype)

    def pairs(which, inside, shared_y=None):
        hidden = torch.full((n * top, inter), float("nan"), device="cuda", dtype=dtype)
        s_hidden = torch.full((n, shared or 1), float("nan"), device="cuda", dtype=dtype)
        out = torch.full((n, width), float("nan"), device="cuda")
        use = bool(shared) and inside
        which.experts_gate_up(x, up, chosen, hidden, activation="relu2", shared=(s_up, s_hidden) if use else None)
        which.experts_down(hidden, down, chosen, weights, out, shared=(s_down, s_hidden) if use else None, shared_y=shared_y)
        return out, s_hidden

    want, s_hidden = pairs(twin, True)
    close(pairs(ops, True)[0], want, dtype, "shared expert inside")
    beside = {}
    if shared:
        beside["shared_y"] = (s_hidden.float() @ s_down.float().t()).to(dtype)
        close(pairs(ops, False, beside["shared_y"])[0], want, dtype, "shared expert ready made")
    out = torch.full((n, width), float("nan"), device="cuda")
    if ops.experts_sorted(x, up, down, chosen, weights, out, activation="relu2", **beside):
        close(out, want, dtype, "sorted by expert")
    else:
        assert dtype == torch.float32 or n * top <= experts or width % 32 or inter % 32
