"""The kernels that Setodra brought: recurrences with one decay per head (token by token and in chunks), the short convolution
and step sizes in front of a state-space mixer, the skip, gate and norm in parts behind it, heads turned in halves, the
stream in front of a pass, the rotary table's amplitude, a latent's rotated part turned in halves, and routed experts with a
corrected choice, identity experts and a shared expert; each against its plain torch twin, in float32 and in bfloat16, on
sizes that are no multiples of anything."""
import pytest
import torch

from test_latent_experts_kernels_gpu import batch, close
from torch_ops import TorchOps

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(scope="module")
def ops():
    from llmserver_amd.kernels import default_ops
    return default_ops()


def both(ops, outs, call):
    """``call(namespace, out)`` with the kernels and the twins; ``outs()`` makes one side's results."""
    made = [outs(), outs()]
    for which, out in zip((ops, TorchOps()), made):
        call(which, out)
    return made


@pytest.mark.parametrize("types", [(torch.float32, torch.float32), (torch.bfloat16, torch.bfloat16), (torch.float32, torch.bfloat16)])
@pytest.mark.parametrize("heads,key_heads,dim,vdim", [(3, 3, 24, 40), (4, 2, 64, 64), (5, 1, 7, 100), (1, 1, 130, 9), (2, 1, 300, 65), (4, 2, 128, 128), (6, 3, 48, 63)])
@pytest.mark.parametrize("chunked", [False, True])
def test_decayed_recurrences_over_steps_and_slots(ops, types, heads, key_heads, dim, vdim, chunked):
    """Rows of unequal portions, an empty row, single tokens, portions longer than the kernels' chunks; a request that starts
    again in a used slot starts from zeros.  Decays per token with step sizes, and constant ones without."""
    print(f"decayed_recurrence {types} {heads}/{key_heads} {dim} {vdim} chunked={chunked}", flush=True)
    twin = TorchOps()
    size = heads * dim * vdim
    constant = torch.log(torch.linspace(0.5, 0.9999, heads, device="cuda"))
    slots = torch.tensor([2, 0, 3], dtype=torch.int32, device="cuda")
    for per_token in (True, False):
        states = [torch.randn(4, size + 3, device="cuda") for _ in range(2)]
        states[1].copy_(states[0])
        firsts = [0, 0, 0]
        for step, lengths in enumerate(([5, 1, 37], [1, 1, 1], [18, 0, 2], [1, 1, 1], [64, 65, 128], [200, 0, 3])):
            if step == 3:
                firsts[1] = 0                          # the second request ends; another one starts in its slot
            _, _, row_start, row_len, row_ctx = batch(lengths, firsts, "cuda")
            n = sum(lengths)
            keys = (0.5 * torch.randn(n, 2 * key_heads * dim + 3, device="cuda")).to(types[0])
            q, k = keys[:, :key_heads * dim], keys[:, key_heads * dim:2 * key_heads * dim]
            v = torch.randn(n, heads * vdim + 2, device="cuda").to(types[1])[:, :heads * vdim]
            take = 2 * torch.rand(n, heads, device="cuda") if per_token else None
            log_keep = -take * torch.linspace(1e-3, 2.0, heads, device="cuda") if per_token else constant
            outs = [torch.zeros(n, heads * vdim, device="cuda") for _ in range(2)]
            scratch = {}
            if chunked:
                # (filled with what is no number: nothing may be read that has not been written)
                scratch = {"sums": torch.full((n // 64 + len(lengths), heads, dim, vdim), float("nan"), device="cuda"),
                           "totals": torch.full((n // 64 + len(lengths), heads), float("nan"), device="cuda")}
            for which, state, out in zip((ops, twin), states, outs):
                which.decayed_recurrence(q, k, v, log_keep, take, dim ** -0.5, state, slots, row_start, row_len, row_ctx, out, heads, key_heads,
                                         dim, vdim, **(scratch if which is ops else {}))
            close(outs[0], outs[1], torch.float32, f"read-out, step {step}")
            close(states[0], states[1], torch.float32, f"state, step {step}")
            assert torch.equal(states[0][1], states[1][1]) and torch.equal(states[0][:, size:], states[1][:, size:])
            firsts = [f + n for f, n in zip(firsts, lengths)]


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_recurrence_does_not_depend_on_how_its_tokens_are_cut(ops, dtype):
    """The same bits, state and read-out, whether 150 tokens come at once, in portions or one by one; in chunks, the same
    numbers."""
    heads, dim, vdim, n = 2, 48, 32, 150
    proj = torch.randn(n, 2 * heads * dim + heads * vdim, device="cuda").to(dtype)
    q, k, v = proj[:, :heads * dim], proj[:, heads * dim:2 * heads * dim], proj[:, 2 * heads * dim:]
    take = torch.rand(n, heads, device="cuda")
    log_keep = -0.05 * take
    make = lambda a: torch.tensor(a, dtype=torch.int32, device="cuda")
    results = []
    for cuts in ([150], [7, 16, 1, 64, 62], [1] * 150, "chunks"):
        state = torch.randn(1, heads * dim * vdim, device="cuda")       # (leftovers of whoever held the slot)
        out = torch.zeros(n, heads * vdim, device="cuda")
        at = 0
        for count in ([64, 86] if cuts == "chunks" else cuts):
            piece = slice(at, at + count)
            scratch = {}
            if cuts == "chunks":
                scratch = {"sums": torch.empty(count // 64 + 1, heads, dim, vdim, device="cuda"), "totals": torch.empty(count // 64 + 1, heads, device="cuda")}
            ops.decayed_recurrence(q[piece], k[piece], v[piece], log_keep[piece], take[piece], 0.2, state, make([0]), make([0]), make([count]),
                                   make([at + count]), out[piece], heads, heads, dim, vdim, **scratch)
            at += count
        results.append((out, state))
    for out, state in results[1:3]:
        assert torch.equal(out, results[0][0]) and torch.equal(state, results[0][1])
    close(results[3][0], results[0][0], torch.float32, "read-outs in chunks")
    close(results[3][1], results[0][1], torch.float32, "the state behind chunks")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("channels,taps,heads", [(37, 4, 3), (300, 1, 5), (64, 2, 1), (513, 3, 70), (100, 6, 2)])
def test_the_convolution_and_the_step_sizes_of_a_state_space_mixer(ops, dtype, channels, taps, heads):
    """Over several steps of unequal portions, tokens one by one with the state moved on inside the kernel, and a portion long
    enough for the form that gives a thread several tokens."""
    print(f"ssd_prepare {dtype} {channels} {taps} {heads}", flush=True)
    twin = TorchOps()
    weight, bias = torch.randn(channels, taps, device="cuda"), torch.randn(channels, device="cuda")
    dt_bias, a_log = 2 * torch.randn(heads, device="cuda"), torch.randn(heads, device="cuda")
    states = [torch.randn(4, 5 + (taps - 1) * channels + 2, device="cuda") for _ in range(2)]
    states[1].copy_(states[0])
    slots = torch.tensor([2, 0, 3], dtype=torch.int32, device="cuda")
    firsts = [0, 0, 0]
    for step, lengths in enumerate(([5, 1, 2], [1, 1, 1], [1, 0, 2], [1, 1, 1], [2, 40, 1], [1, 1, 1], [300, 260, 3])):
        if step == 3:
            firsts[1] = 0
        token_row, positions, row_start, row_len, row_ctx = batch(lengths, firsts, "cuda")
        n, single = sum(lengths), all(length == 1 for length in lengths)
        proj = torch.randn(n, 3 + channels + heads, device="cuda").to(dtype)
        x, dt = proj[:, 3:3 + channels], proj[:, 3 + channels:]
        dt.mul_(10.0)                                             # (softplus on both sides of its corner)
        results = []
        for which, state in zip((ops, twin), states):
            out = torch.zeros(n, channels, device="cuda", dtype=dtype)
            steps, logs = torch.zeros(n, heads, device="cuda"), torch.zeros(n, heads, device="cuda")
            which.ssd_prepare(x, weight, bias, state, 5, slots, token_row, positions, row_start, out, dt, dt_bias, a_log, steps, logs, keep=single)
            if not single and taps > 1:
                which.delta_conv_keep(x, channels, taps, state, 5, slots, row_start, row_len, row_ctx)
            results.append((out, steps, logs))
        close(results[0][0], results[1][0], dtype, f"convolution, step {step}")
        close(results[0][1], results[1][1], torch.float32, f"step sizes, step {step}")
        close(results[0][2], results[1][2], torch.float32, f"decays, step {step}")
        assert torch.equal(states[0], states[1]), f"state, step {step}"
        firsts = [f + n for f, n in zip(firsts, lengths)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,vdim,groups", [(4, 6, 3), (2, 64, 1), (10, 77, 2), (16, 64, 1), (70, 40, 2), (66, 64, 1)])
def test_the_skip_the_gate_and_the_norm_in_parts(ops, dtype, heads, vdim, groups):
    width, n = heads * vdim, 5
    y, skip, weight = torch.randn(n, width, device="cuda"), torch.randn(heads, device="cuda"), 1 + 0.3 * torch.randn(width, device="cuda")
    proj = torch.randn(n, 2 * width + 3, device="cuda").to(dtype)
    got, want = both(ops, lambda: torch.empty(n, width, device="cuda", dtype=dtype),
                     lambda which, out: which.gated_group_norm(y, proj[:, 3:3 + width], skip, proj[:, 3 + width:], weight, 1e-5, out, heads, groups))
    close(got, want, dtype, "normed in parts")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,pairs", [(3, 10, 3), (2, 64, 32), (5, 7, 0), (1, 130, 65)])
def test_heads_turned_in_halves(ops, dtype, heads, dim, pairs):
    n, width = 6, heads * dim
    proj = torch.randn(n, 2 * width + 5, device="cuda").to(dtype)
    positions = torch.tensor([0, 1, 2, 500, 7, 3000], dtype=torch.int32, device="cuda")
    freqs = 100.0 ** (-torch.arange(pairs, device="cuda").float() / max(pairs, 1))
    table = None
    if pairs:
        table = ops.rotary_table(positions, freqs, amplitude=1.37)
        close(table, TorchOps().rotary_table(positions, freqs, amplitude=1.37), torch.float32, "table")
        close(table, 1.37 * ops.rotary_table(positions, freqs), torch.float32, "the amplitude multiplies cosines and sines")
    got, want = both(ops, lambda: (torch.empty(n, width, device="cuda"), torch.empty(n, width, device="cuda")),
                     lambda which, out: which.rotate_heads(proj[:, :width], proj[:, width:2 * width], table, dim ** -0.5, out[0], out[1], heads))
    close(got[0], want[0], torch.float32, "queries")
    close(got[1], want[1], torch.float32, "keys")
    # a head's norm without a weight
    gate = torch.randn(n, width, device="cuda").to(dtype)
    got, want = both(ops, lambda: torch.empty(n, width, device="cuda", dtype=dtype),
                     lambda which, out: which.heads_norm_gate(want[0], None, False, 1e-5, gate, out, heads, dim))
    close(got, want, dtype, "normed, gated heads")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [100, 256, 1027, 4400])
def test_the_stream_in_front_of_a_pass(ops, dtype, width):
    n = 7
    table = torch.randn(19, width, device="cuda").to(dtype)
    ids = torch.randint(0, 19, (n,), device="cuda", dtype=torch.int32)
    x, vector, weight = torch.randn(n, width, device="cuda"), torch.randn(width, device="cuda"), 1 + 0.2 * torch.randn(width, device="cuda")
    for scale in (0.0, 2.5):
        for following in (True, False):
            got, want = both(ops, lambda: (x.clone(), torch.zeros(n, width, device="cuda", dtype=dtype)),
                             lambda which, out: which.stream_inject(out[0], table, ids, scale, vector, weight if following else None, 1e-5,
                                                                    out[1] if following else None))
            close(got[0], want[0], torch.float32, "stream")
            close(got[1], want[1], dtype, "the next norm")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("inside", [False, True])
def test_a_latents_rotated_part_turned_in_halves(ops, dtype, inside):
    heads, dim, rot_dim, rank, page, row, n = 3, 8, 12, 21, 8, 48, 11
    token_row, positions, _, _, _ = batch([9, 2], [0, 30], "cuda")
    table = torch.randperm(10, device="cuda").to(torch.int32).view(2, 5)
    proj = torch.randn(n, heads * (dim + rot_dim) + rank + rot_dim, device="cuda").to(dtype)
    up_keys = torch.randn(heads, dim, rank, device="cuda").to(dtype)
    q_latent = None if inside else torch.randn(heads, n, rank, device="cuda").to(dtype)
    weight = 1 + 0.2 * torch.randn(rank, device="cuda")
    cos_sin = ops.rotary_table(positions, 50.0 ** (-torch.arange(rot_dim // 2, device="cuda").float() / 6), amplitude=1.2)
    outs = lambda: (torch.zeros(n, heads * row, device="cuda", dtype=dtype), torch.zeros(10, 1, page, row, device="cuda", dtype=dtype),
                    torch.zeros(10, 1, row, page, device="cuda", dtype=dtype))
    got, want = both(ops, outs, lambda which, out: which.latent_prepare(proj, q_latent, weight, 1e-5, cos_sin, out[1], out[2], table, token_row, positions,
                                                                       page, out[0], heads, dim, rot_dim, rank, True,
                                                                       **({"up_keys": up_keys} if inside else {}), pairing="halves"))
    for a, b, what in zip(got, want, ("queries", "keys", "values")):
        close(a, b, dtype, what)
    q = proj[3].float().view(-1)[:heads * (dim + rot_dim)].view(heads, dim + rot_dim)[1, dim:]          # dimension i turns with i + 6
    c, s = cos_sin[3, :6], cos_sin[3, 6:]
    close(got[0][3].float().view(heads, row)[1, rank:rank + rot_dim], torch.cat([q[:6] * c - q[6:] * s, q[6:] * c + q[:6] * s]), dtype, "a query by hand")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,identity,top,shared", [(5, 3, 2, 28), (8, 0, 3, 64), (3, 4, 7, None), (64, 8, 6, 96), (1, 1, 1, 32), (70, 5, 4, 20)])
@pytest.mark.parametrize("n", [1, 3, 9, 40, 200])
def test_routed_experts_with_identity_and_shared_ones(ops, dtype, experts, identity, top, shared, n):
    """The router (choice corrected, weights not, the shared expert's gate beside it) and both ways of the products: pair by
    pair with the shared expert inside or ready made, and sorted by expert."""
    print(f"experts {dtype} {experts}+{identity} top {top} shared {shared} n {n}", flush=True)
    twin = TorchOps()
    width, inter, choices = 64, 32, experts + identity
    x = torch.randn(n, width, device="cuda").to(dtype)
    router = 0.2 * torch.randn(choices + (1 if shared else 0), width, device="cuda")
    correction = 0.3 * torch.rand(choices, device="cuda") / choices
    make = lambda: (torch.zeros(n, top, device="cuda", dtype=torch.int32), torch.zeros(n, top, device="cuda"), torch.zeros(n, device="cuda"))
    got, want = both(ops, make, lambda which, out: which.route_experts(x, router, top, out[0], out[1], scoring="softmax_all", correction=correction,
                                                                     weight_scale=1.7, gate_out=out[2] if shared else None))
    assert (got[0] == want[0]).float().mean() > 0.97          # (two choices a rounding apart may change places)
    close(got[1], want[1], torch.float32, "weights")
    close(got[2], want[2], torch.float32, "gate")
    chosen, weights, gate = want
    assert float((weights.sum(dim=1) - 1.7).abs().max()) < 1e-5
    gate_up = (0.2 * torch.randn(experts, 2 * inter, width, device="cuda")).to(dtype)
    down = (0.2 * torch.randn(experts, width, inter, device="cuda")).to(dtype)
    s_gate_up = (0.2 * torch.randn(2 * (shared or 1), width, device="cuda")).to(dtype)
    s_down = (0.2 * torch.randn(width, shared or 1, device="cuda")).to(dtype)

    def pairs(which, inside, shared_y=None):
        hidden = torch.full((n * top, inter), float("nan"), device="cuda", dtype=dtype)
        s_hidden = torch.full((n, shared or 1), float("nan"), device="cuda", dtype=dtype)
        out = torch.empty(n, width, device="cuda")
        use = bool(shared) and inside
        which.experts_gate_up(x, gate_up, chosen, hidden, identity=identity, shared=(s_gate_up, s_hidden) if use else None)
        which.experts_down(hidden, down, chosen, weights, out, x=x if identity else None, shared=(s_down, s_hidden) if use else None,
                           shared_y=shared_y, shared_gate=gate if shared else None)
        return out, s_hidden

    want_out, s_hidden = pairs(twin, True)
    close(pairs(ops, True)[0], want_out, dtype, "shared expert inside")
    if shared:
        shared_y = (s_hidden.float() @ s_down.float().t()).to(dtype)
        close(pairs(ops, False, shared_y)[0], want_out, dtype, "shared expert ready made")
    beside = {"shared_y": shared_y, "shared_gate": gate} if shared else {}
    out = torch.full((n, width), float("nan"), device="cuda")
    if ops.experts_sorted(x, gate_up, down, chosen, weights, out, identity=identity, **beside):
        close(out, want_out, dtype, "sorted by expert")
    else:
        assert dtype == torch.float32 or n * top <= experts
