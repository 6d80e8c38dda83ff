"""Fevolorn's mechanisms one by one, each kernel against the plain function of ``plain_fevolorn`` (float64), at sizes of the
tests' own: the streams' read and join with every form of a sublayer's output, the tanh norm, the recurrence with a fixed
decay in order and in chunks, the selective scan in order, in chunks and with its low-rank map in front, the convolution
with its activation, the router's correction, the gated shared unit, the norm over all heads together and the gated unit
around the tanh form of gelu."""

import numpy as np
import pytest
import torch

import plain_fevolorn as plain

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(scope="module")
def ops():
    from flyweight_amd.kernels import ops
    ops.library()
    return ops


def dev(a, dtype=torch.float32):
    return torch.tensor(np.asarray(a), dtype=dtype, device=DEV).contiguous()


def ints(a):
    return torch.tensor(np.asarray(a, dtype=np.int32), device=DEV)


def host(t):
    return t.detach().float().cpu().numpy().astype(np.float64)


def segments_of(lengths):
    row0 = np.concatenate([[0], np.cumsum(lengths)])
    row_seg = np.concatenate([np.full(n, s) for s, n in enumerate(lengths)])
    return ints(row_seg), ints(row0)


def chunks_of(lengths, long_rows=32, size=64):
    """What a step brings for its long segments (None: there is none)."""
    row0 = np.concatenate([[0], np.cumsum(lengths)])
    seg, first, begins = [], [], [0]
    for s, n in enumerate(lengths):
        for at in range(0, n if n > long_rows else 0, size):
            seg.append(s)
            first.append(row0[s] + at)
        begins.append(len(seg))
    return (ints(seg), ints(first), ints(begins), long_rows, min(lengths) > long_rows) if seg else None


def near(found, want, limit, what=""):
    scale = max(1.0, float(np.abs(want).max()))
    worst = float(np.abs(found - want).max())
    assert np.isfinite(found).all() and worst <= limit * scale, f"{what}: {worst:.3e} of {scale:.3e}"


# ---- the streams -------------------------------------------------------------------------------------------
STREAM_SHAPES = [(1, 8, 3), (2, 64, 5), (3, 96, 4), (4, 2048, 3), (4, 4100, 2), (5, 44, 4), (6, 128, 2), (8, 256, 2), (4, 97, 3), (32, 20, 2), (1, 5000, 2)]


def _norm(rng, hidden):
    return rng.uniform(0.5, 1.5, hidden), rng.normal(size=hidden), np.float32(rng.uniform(0.3, 1.2))


@pytest.mark.parametrize("streams,hidden,rows", STREAM_SHAPES)
def test_stream_read(ops, streams, hidden, rows):
    """A weighted sum and a plain one, with and without the norm, some of the rows alone; arguments from far inside tanh's
    straight part to far outside it."""
    rng = np.random.default_rng(streams * hidden)
    x = rng.normal(size=(rows, streams, hidden)) * np.exp(rng.normal(size=(rows, 1, 1)) * 2)
    x[0, :, :4] *= 1e-4
    w, (weight, bias, alpha) = rng.normal(size=streams), _norm(rng, hidden)
    x32 = np.asarray(x, dtype=np.float32).astype(np.float64)
    for given in (w, None):
        u = plain.read_streams(x32, np.float32(w).astype(np.float64) if given is not None else np.ones(streams))
        reader = None if given is None else dev(w)
        near(host(ops.stream_read(dev(x), reader, torch.float32)), u, 1e-6, "sum")
        want = plain.tanh_norm(u, float(alpha), weight, bias)
        for dtype, limit in ((torch.float32, 2e-6), (torch.bfloat16, 8e-3)):
            found = ops.stream_read(dev(x), reader, dtype, kind=ops.NEXT_TANH, weight=dev(weight), bias=dev(bias), alpha=dev(alpha))
            assert found.dtype == dtype
            near(host(found), want, limit, f"norm {dtype}")
    index = [rows - 1, 0, rows - 1]
    found = ops.stream_read(dev(x), dev(w), torch.float32, kind=ops.NEXT_TANH, weight=dev(weight), bias=dev(bias), alpha=dev(alpha), row_index=ints(index))
    near(host(found), plain.tanh_norm(plain.read_streams(x32, w), float(alpha), weight, bias)[index], 2e-6, "gathered")


def test_the_norm_keeps_small_numbers(ops):
    """tanh near zero is its argument: relative precision is kept over the whole range."""
    x = np.concatenate([10.0 ** np.linspace(-8, 1.5, 400), -(10.0 ** np.linspace(-8, 1.5, 400)), [0.0, 0.2499, 0.2501, 100.0]])
    x = np.float32(x).astype(np.float64)
    found = host(ops.stream_read(dev(x).view(1, 1, -1), None, torch.float32, kind=ops.NEXT_TANH, weight=dev(np.ones(x.size)),
                                 bias=dev(np.zeros(x.size)), alpha=dev(1.0)))[0]
    want = np.tanh(x)
    assert np.all(np.abs(found - want) <= 1.5e-6 * np.abs(want))


@pytest.mark.parametrize("streams,hidden,rows", STREAM_SHAPES)
@pytest.mark.parametrize("source", ["rows", "branches", "chosen", "chosen_gated"])
def test_stream_join(ops, streams, hidden, rows, source):
    """Every form of a sublayer's output joins the streams from their old rows, and the next reader's norm is formed of the new
    ones (into float32 and bfloat16; or nothing)."""
    rng = np.random.default_rng(streams + hidden)
    x = rng.normal(size=(rows, streams, hidden))
    mix, out, ls, w = rng.normal(size=(streams, streams)), rng.normal(size=streams), rng.uniform(0.2, 1.5, hidden), rng.normal(size=streams)
    weight, bias, alpha = _norm(rng, hidden)
    given = {}
    if source == "rows":
        a = rng.normal(size=(rows, hidden))
        y = a
    elif source == "branches":
        a, b = rng.normal(size=(rows, hidden)) * 3.0, rng.normal(size=(rows, hidden)) * 0.01
        wa, wb = rng.uniform(0.5, 1.5, hidden), rng.uniform(0.5, 1.5, hidden)
        y = 0.5 * plain.rms(a, 1e-5) * wa + 0.25 * plain.rms(b, 1e-5) * wb
        given["branches"] = (dev(b), dev(wa), dev(wb), 0.5, 0.25, 1e-5)
    else:
        top = 3
        a = rng.normal(size=(rows * top, hidden))
        choice = rng.uniform(0.1, 1.0, size=(rows, top))
        place = rng.permutation(rows * top).reshape(rows, top)
        y = np.einsum("rj,rjd->rd", choice, a[place])
        b = rng.normal(size=(rows, hidden)) if source == "chosen_gated" else None
        gate = rng.normal(size=(rows, 7)) * 2.0
        if b is not None:
            y = y + plain.sigmoid(gate[:, 2:3]) * b
        given["chosen"] = (dev(choice), ints(place), None if b is None else dev(b), None if b is None else dev(gate)[:, 2:3])
    want = plain.join_streams(x, ls * y, mix, out)
    seen = plain.tanh_norm(plain.read_streams(want, w), float(alpha), weight, bias)
    for dtype, limit in ((torch.float32, 3e-6), (torch.bfloat16, 8e-3)):
        streams_now = dev(x)
        found = ops.stream_join_(streams_now, dev(ls), dev(mix), dev(out), dev(a), next_kind=ops.NEXT_TANH, next_in=dev(w), next_weight=dev(weight),
                                 next_bias=dev(bias), next_alpha=dev(alpha), next_dtype=dtype, **given)
        near(host(streams_now), want, 3e-6, "streams")
        near(host(found), seen, limit * (1.0 + np.abs(weight).max()), f"next {dtype}")
    streams_now = dev(x)
    found = ops.stream_join_(streams_now, dev(ls), dev(mix), dev(out), dev(a), next_kind=ops.NEXT_SUM, next_dtype=torch.float32, **given)
    near(host(found), want.sum(axis=1), 3e-6 * streams, "plain sum")
    streams_now = dev(x)
    assert ops.stream_join_(streams_now, dev(ls), dev(mix), dev(out), dev(a), **given) is None
    near(host(streams_now), want, 3e-6, "streams alone")


def test_stream_join_does_not_depend_on_the_batch(ops):
    rng = np.random.default_rng(3)
    x, a, b = rng.normal(size=(40, 4, 256)), rng.normal(size=(40, 256)), rng.normal(size=(40, 256))
    mix, out, ls, ones = dev(rng.normal(size=(4, 4))), dev(rng.normal(size=4)), dev(rng.uniform(size=256)), dev(np.ones(256))
    together = dev(x)
    ops.stream_join_(together, ls, mix, out, dev(a), branches=(dev(b), ones, ones, 0.5, 0.5, 1e-6))
    alone = dev(x[17:18])
    ops.stream_join_(alone, ls, mix, out, dev(a[17:18]), branches=(dev(b[17:18]), ones, ones, 0.5, 0.5, 1e-6))
    assert torch.equal(together[17:18], alone)


def test_streams_refuse_what_does_not_fit(ops):
    x, v = torch.zeros((2, 3, 8), device=DEV), torch.zeros((8,), device=DEV)
    mix, out, a = torch.zeros((3, 3), device=DEV), torch.zeros((3,), device=DEV), torch.zeros((2, 8), device=DEV)
    for call in (lambda: ops.stream_join_(x, v, mix[:2, :2].contiguous(), out, a), lambda: ops.stream_join_(x, v, mix, out, a[:1]),
                 lambda: ops.stream_join_(x, v[:4], mix, out, a), lambda: ops.stream_join_(x[:, 0], v, mix, out, a),
                 lambda: ops.stream_join_(x, v, mix, out, a, next_kind=ops.NEXT_TANH),
                 lambda: ops.stream_read(x, out[:2], torch.float32), lambda: ops.stream_read(x, None, torch.float32, kind=7)):
        with pytest.raises(ops.KernelError):
            call()


def test_embedding_rows_in_copies(ops):
    rng = np.random.default_rng(4)
    ids = [3, 49, 0, 3]
    for width in (33, 2052):
        table = rng.normal(size=(50, width))
        for dtype in DTYPES:
            stored = dev(table, dtype)
            found = ops.embed_rows(stored, ints(ids), scale=1.5, copies=3)
            assert found.shape == (4, 3, width)
            for copy in range(3):
                near(host(found[:, copy]), host(stored)[ids] * 1.5, 1e-6)


# ---- the recurrence with a fixed decay ------------------------------------------------------------------------
@pytest.mark.parametrize("heads,dim,vdim,lengths", [(3, 32, 48, [1, 5, 1, 2]), (2, 16, 16, [1, 1, 1]), (1, 100, 12, [33, 3]), (4, 5, 70, [40, 1, 64]),
                                                    (2, 128, 128, [200, 7, 65]), (1, 256, 40, [130]), (2, 64, 256, [64, 128, 33]), (5, 24, 36, [700]),
                                                    (2, 129, 33, [97, 32])])
def test_decay_recurrence(ops, heads, dim, vdim, lengths):
    """Three steps over the same requests, states carried in slots: in order, in chunks of 64 rows (full ones, one row, the
    last one not full) beside short segments in order, then single rows. Decays of 0.2 to exactly 1."""
    rng = np.random.default_rng(heads * dim + vdim)
    decay = np.concatenate([[1.0, 0.2, 0.999, 0.9, 0.97]])[:heads]
    powers = ops.decay_powers(decay, DEV)
    slots = [4, 1, 0, 2][:len(lengths)]
    state = torch.zeros((6, heads, dim, vdim), dtype=torch.float32, device=DEV)
    carried = {slot: np.zeros((heads, dim, vdim)) for slot in slots}
    for step, cut in ((0, False), (1, True), (2, False), (3, True)):
        now = [1] * len(lengths) if step == 2 else lengths
        rows, width = sum(now), heads * (2 * dim + vdim)
        proj = rng.normal(size=(rows, width + 3))               # rows wider than what is read
        both = dev(proj)
        q, k, v = (both[:, at:at + n] for at, n in ((0, heads * dim), (heads * dim, heads * dim), (2 * heads * dim, heads * vdim)))
        _, seg_row0 = segments_of(now)
        found = host(ops.decay_recurrence(q, k, v, powers, state, seg_row0, ints(slots), len(now), heads, dim, vdim, chunks=chunks_of(now) if cut else None))
        at = 0
        for slot, n in zip(slots, now):
            part = plain.silu(proj[at:at + n])
            qq, kk = (part[:, o:o + heads * dim].reshape(n, heads, dim) for o in (0, heads * dim))
            vv = part[:, 2 * heads * dim:width].reshape(n, heads, vdim)
            want, carried[slot] = plain.decay_recurrence(qq, kk, vv, decay, carried[slot])
            near(found[at:at + n], want.reshape(n, -1), 4e-6, f"step {step} slot {slot}")
            near(host(state[slot]), carried[slot], 4e-6, f"state, step {step} slot {slot}")
            at += n
    assert float(state[[3, 5]].abs().max()) == 0.0              # nobody else's slot moved


def test_decay_recurrence_carries_one_key_across_chunks(ops):
    """A single token's key and value among empty ones: what the rows behind it read out is decay^(rows since), across chunk
    borders and into the next step."""
    decay, rows, at = 0.99, 200, 37
    big = 30.0                                                  # silu of it is itself
    q, k, v = np.full((rows, 16), big), np.zeros((rows, 16)), np.zeros((rows, 16))
    k[at], v[at, 3] = big, big
    state = torch.zeros((2, 1, 16, 16), dtype=torch.float32, device=DEV)
    _, seg_row0 = segments_of([rows])
    both = dev(np.concatenate([q, k, v], axis=1))
    parts = [both[:, i * 16:(i + 1) * 16] for i in range(3)]
    for cut in (chunks_of([rows]), None):
        state.zero_()
        found = host(ops.decay_recurrence(*parts, ops.decay_powers([decay], DEV), state, seg_row0, ints([1]), 1, 1, 16, 16, chunks=cut))
        want = np.zeros((rows, 16))
        want[at:, 3] = 16 * big ** 3 * decay ** np.arange(rows - at)
        near(found, want, 2e-6)
        assert np.all(np.abs(found[:, [c for c in range(16) if c != 3]]) == 0.0)


# ---- the selective scan -----------------------------------------------------------------------------------------
def _scan_inputs(rng, rows, channels, states):
    return rng.normal(size=(rows, channels)) * 2, rng.normal(size=(rows, channels)) * 4 - 2, rng.normal(size=(rows, 2 * states)), rng.normal(size=(rows, channels)) * 2


@pytest.mark.parametrize("out_dtype", DTYPES)
@pytest.mark.parametrize("channels,states,lengths", [(30, 1, [1, 5, 1, 2]), (120, 12, [70, 9]), (64, 16, [1, 1, 1]), (100, 9, [33, 17]), (200, 24, [130, 64, 65, 1]),
                                                     (65, 33, [40, 128]), (48, 64, [80]), (33, 128, [66, 2]), (256, 8, [700]), (72, 20, [32])])
def test_selective_scan(ops, channels, states, lengths, out_dtype):
    """Steps over the same requests, states carried in slots: in order, in chunks beside short segments in order, single rows. Decays
    from barely forgetting to forgetting at once, step sizes from 1e-6 to tens."""
    rng = np.random.default_rng(channels + states)
    A, D = -np.exp(rng.uniform(-3.0, 2.0, size=(channels, states))), rng.normal(size=channels)
    A2 = dev((A * np.log2(np.e)).T)
    slots = [4, 1, 0, 2][:len(lengths)]
    state = torch.zeros((6, states, channels), dtype=torch.float32, device=DEV)
    carried = {slot: np.zeros((channels, states)) for slot in slots}
    for step, cut in ((0, False), (1, True), (2, False), (3, True)):
        now = [1] * len(lengths) if step == 2 else lengths
        x, z, bc, gate = _scan_inputs(rng, sum(now), channels, states)
        z[0, 0], z[-1, 0] = -14.0, 25.0
        _, seg_row0 = segments_of(now)
        wide = dev(np.concatenate([z, bc], axis=1))            # rows that lie apart
        found = host(ops.selective_scan(dev(x), wide[:, :channels], wide[:, channels:], dev(gate), A2, dev(D), state, seg_row0, ints(slots), len(now),
                                        out_dtype, chunks=chunks_of(now) if cut else None))
        at = 0
        for slot, n in zip(slots, now):
            s = slice(at, at + n)
            want, carried[slot] = plain.selective_scan(x[s], plain.softplus(z[s]), A, bc[s, :states], bc[s, states:], D, carried[slot])
            near(found[s], want * plain.silu(gate[s]), 1e-5 if out_dtype == torch.float32 else 8e-3, f"step {step} slot {slot}")
            near(host(state[slot]), carried[slot].T, 1e-5, f"state, step {step} slot {slot}")
            at += n
    assert float(state[[3, 5]].abs().max()) == 0.0


@pytest.mark.parametrize("out_dtype", DTYPES)
@pytest.mark.parametrize("channels,states,rank,rows", [(30, 1, 1, 3), (120, 12, 6, 5), (64, 16, 64, 1), (100, 9, 7, 4), (200, 24, 128, 16), (65, 33, 10, 2), (48, 64, 5, 3),
                                                       (70, 128, 12, 2)])
def test_selective_scan_with_its_low_rank_map(ops, channels, states, rank, rows, out_dtype):
    """Single rows: the step sizes' map inside the scan against the map ahead of it; even and odd ranks."""
    rng = np.random.default_rng(channels + rank)
    A, D, bias = -np.exp(rng.uniform(-3.0, 2.0, size=(channels, states))), rng.normal(size=channels), rng.normal(size=channels)
    W = host(dev(rng.normal(size=(channels, rank)) / np.sqrt(rank), torch.bfloat16))
    weights = ops.low_rank_weights(dev(W, out_dtype))
    assert weights.dim() == (3 if out_dtype == torch.bfloat16 and rank % 2 == 0 else 2)
    slots = rng.permutation(rows + 2)[:rows]
    start = rng.normal(size=(rows + 3, states, channels))
    state = dev(start)
    x, gate = rng.normal(size=(rows, channels)), rng.normal(size=(rows, channels))
    low = rng.normal(size=(rows, rank + 2 * states))
    found = host(ops.selective_scan_low_rank(dev(x), dev(low), weights, dev(bias), dev(gate), dev((A * np.log2(np.e)).T), dev(D), state, ints(slots), out_dtype))
    for r in range(rows):
        dt = plain.softplus(low[r:r + 1, :rank] @ W.T + bias)
        want, S = plain.selective_scan(x[r:r + 1], dt, A, low[r:r + 1, rank:rank + states], low[r:r + 1, rank + states:], D, start[slots[r]].T)
        near(found[r:r + 1], want * plain.silu(gate[r:r + 1]), 1e-5 if out_dtype == torch.float32 else 8e-3, f"row {r}")
        near(host(state[int(slots[r])]), S.T, 1e-5, f"state of row {r}")
    untouched = [s for s in range(rows + 3) if s not in slots]
    assert np.array_equal(host(state[untouched]), host(dev(start)[untouched]))


# ---- the convolution ---------------------------------------------------------------------------------------
@pytest.mark.parametrize("channels,taps,lengths", [(40, 4, [1, 5, 1, 2]), (300, 4, [200, 1, 2, 90, 3]), (70, 2, [300]), (130, 3, [2, 2, 260]), (40, 7, [300, 9]), (64, 1, [280])])
def test_causal_conv_with_its_activation(ops, channels, taps, lengths):
    """silu behind the convolution, the result once more in bfloat16; steps of many rows walk runs of rows across segments'
    borders, whose first rows reach back into the slots."""
    rng = np.random.default_rng(channels + taps)
    w, bias = rng.normal(size=(channels, taps)), rng.normal(size=channels)
    slots = [5, 0, 3, 2, 6][:len(lengths)]
    state = torch.zeros((7, channels, taps - 1), dtype=torch.float32, device=DEV)
    before = {slot: np.zeros((taps - 1, channels)) for slot in slots}
    for step, single in ((0, False), (1, False), (2, True), (3, False)):
        now = [1] * len(lengths) if single else lengths
        x = rng.normal(size=(sum(now), channels + 5))
        row_seg, seg_row0 = segments_of(now)
        found, short = ops.causal_conv(dev(x)[:, :channels], dev(w), dev(bias), state, row_seg, seg_row0, ints(slots), len(now), single_rows=single,
                                       silu=True, rounded=True)
        assert torch.equal(short, found.to(torch.bfloat16))
        at = 0
        for slot, n in zip(slots, now):
            want, before[slot] = plain.causal_conv(x[at:at + n, :channels], w, bias, before[slot])
            near(host(found[at:at + n]), plain.silu(want), 3e-6, f"step {step} slot {slot}")
            at += n
        if taps > 1:
            for slot in slots:
                near(host(state[slot]), before[slot].T, 1e-6, "memory")


# ---- the mixture ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("experts,top", [(8, 2), (9, 3), (1, 1), (64, 8), (130, 5), (5, 5)])
def test_router_with_a_correction(ops, experts, top):
    """The choice is by score + correction, the weights are the scores alone times the scale, undivided; rows of logits that lie
    apart; ties go to the lowest id."""
    rng = np.random.default_rng(experts)
    z = rng.normal(size=(50, experts)) * 2
    z[3] = 0.0
    correction = rng.normal(size=experts) * 0.5
    correction[1:] = np.where(rng.random(experts - 1) < 0.3, correction[0], correction[1:])
    z, correction = np.float32(z).astype(np.float64), np.float32(correction).astype(np.float64)
    padded = np.concatenate([z, rng.normal(size=(50, 3)) + 50.0], axis=1)
    chosen, weight = ops.moe_route(dev(padded)[:, :experts], None, top, scores="sigmoid", correction=dev(correction), weight_scale=1.7, normalize=False)
    found = chosen.cpu().numpy()
    want, _ = plain.route(z, np.eye(experts), correction, top, 1.7)
    score = plain.sigmoid(z) + correction
    for r in range(50):
        same = found[r] == want[r]
        # (choices of one score to the last digit of float32 may change places)
        assert np.all(same | (np.abs(score[r, found[r]] - score[r, want[r]]) < 1e-6)), r
        assert len(set(found[r].tolist())) == top
    assert found[3].tolist() == np.argsort(-(0.5 + correction), kind="stable")[:top].tolist()
    near(host(weight), 1.7 * np.take_along_axis(plain.sigmoid(z), found.astype(np.int64), axis=1), 1e-6)
    # divided by their sum, and groups ranked by their corrected scores
    chosen, weight = ops.moe_route(dev(z), None, top, scores="sigmoid", correction=dev(correction), weight_scale=1.5)
    near(host(weight).sum(axis=1), np.full(50, 1.5), 1e-6)
    if experts == 64:
        chosen, _ = ops.moe_route(dev(z), None, 4, groups=8, keep=2, scores="sigmoid", correction=dev(correction), group_pair=True)
        pair = np.sort(score.reshape(50, 8, 8), axis=2)[:, :, -2:].sum(axis=2)
        for r in range(50):
            best = set(np.argsort(-pair[r], kind="stable")[:2].tolist())
            assert set((chosen[r].cpu().numpy() // 8).tolist()) <= best
    with pytest.raises(ops.KernelError):
        ops.moe_route(dev(z), None, top, scores="softmax_all", correction=dev(correction))


def test_combine_with_a_gated_shared_unit(ops):
    rng = np.random.default_rng(2)
    x, y, b, gate = rng.normal(size=(6, 40)), rng.normal(size=(18, 40)), rng.normal(size=(6, 40)), rng.normal(size=(6, 4))
    weight, place = rng.uniform(size=(6, 3)), rng.permutation(18).reshape(6, 3)
    found = ops.moe_combine_(dev(x), dev(y), dev(weight), ints(place), shared=dev(b), gate=dev(gate)[:, 1:2])
    near(host(found), x + np.einsum("rj,rjd->rd", weight, y[place]) + plain.sigmoid(gate[:, 1:2]) * b, 2e-6)


@pytest.mark.parametrize("width", [300, 1024, 1500, 4096, 5000])
@pytest.mark.parametrize("dtype", DTYPES)
def test_norm_over_all_heads_together(ops, width, dtype):
    rng = np.random.default_rng(width)
    o, gate, weight = rng.normal(size=(5, width)) * 3, rng.normal(size=(5, width + 2)), rng.uniform(0.5, 1.5, width)
    found = host(ops.gated_head_norm(dev(o), dev(gate)[:, 2:], dev(weight), 1, width, 1e-5, dtype))
    near(found, plain.rms(o, 1e-5) * weight * plain.sigmoid(gate[:, 2:]), 3e-6 if dtype == torch.float32 else 8e-3)


# ---- the gated unit around gelu ----------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,inner", [(1, 64, 96), (8, 256, 320), (16, 100, 72), (33, 512, 256), (64, 2048, 512), (100, 64, 40), (300, 512, 1024),
                                              (700, 1024, 4096), (2048, 256, 640)])
def test_gelu_gated_unit(ops, rows, width, inner, dtype):
    """gelu_tanh(gate) * up behind the products of every number of rows, in both dtypes."""
    from flyweight_amd.parts import Linear
    rng = np.random.default_rng(rows + inner)
    a = host(dev(rng.normal(size=(rows, width)), dtype))
    w = host(dev(rng.normal(size=(2 * inner, width)) * 2.0 / np.sqrt(width), dtype))
    found = host(Linear(dev(w, dtype)).swiglu(dev(a, dtype), gelu=True))
    want = plain.gelu_tanh(a @ w[:inner].T) * (a @ w[inner:].T)
    near(found, want, 1e-5 if dtype == torch.float32 else 6e-3, "gelu")
    found = host(Linear(dev(w, dtype)).swiglu(dev(a, dtype)))
    near(found, plain.silu(a @ w[:inner].T) * (a @ w[inner:].T), 1e-5 if dtype == torch.float32 else 6e-3, "silu")


def test_columns_of_wider_rows_alone(ops):
    x = np.random.default_rng(0).normal(size=(5, 30))
    for dtype in DTYPES:
        out = torch.zeros((5, 7), dtype=dtype, device=DEV)
        assert torch.equal(ops.place_rows(dev(x)[:, 3:10], out), dev(x)[:, 3:10].to(dtype))
