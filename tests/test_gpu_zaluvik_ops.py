"""Zaluvik's mechanisms one by one, each kernel against the plain function of ``plain_zaluvik`` (float64), at sizes of
the tests' own: attention whose weights are sigmoids that the heads mix (with inputs made so that a single key decides the
output just inside and just outside the window), the decode step that norms and stores in the same kernel, the layer norms
with biases around a sublayer, the gelu in the products' epilogues, the router, the latent's rotation by halves and the
gate per head."""

import numpy as np
import pytest
import torch

import plain_zaluvik as plain

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(scope="module")
def ops():
    from flyweight_amd.kernels import ops
    ops.library()
    ops.prepare_device(torch.device(DEV))
    return ops


def dev(a, dtype=torch.float32):
    return torch.tensor(np.asarray(a), dtype=dtype, device=DEV).contiguous()


def ints(a):
    return torch.tensor(np.asarray(a, dtype=np.int32), device=DEV)


def host(t):
    return t.detach().float().cpu().numpy().astype(np.float64)


def stored(a, dtype):
    """The values a tensor of ``dtype`` holds of ``a``, in float64."""
    return torch.tensor(np.asarray(a)).to(dtype).to(torch.float64).numpy()


# ---- attention -------------------------------------------------------------------------------------------------
def paged(keys, values, dtype, pages):
    """[T, G, d] keys and [T, G, dv] values -> pages of 64 tokens in the order ``pages``; the rest is NaN."""
    T, G, d = keys.shape
    dv = values.shape[2]
    k_pages = torch.full((max(pages) + 1, G, 64, d), float("nan"), dtype=torch.float64)
    v_pages = torch.full((max(pages) + 1, G, dv, 64), float("nan"), dtype=torch.float64)
    for t in range(T):
        k_pages[pages[t // 64], :, t % 64, :] = torch.from_numpy(keys[t])
        v_pages[pages[t // 64], :, :, t % 64] = torch.from_numpy(values[t])
    return k_pages.to(dtype).to(DEV), v_pages.to(dtype).to(DEV)


def one_row(ops, q, H, G, d, dv, k_pages, v_pages, table, position, scale, window, bias, mix, gate, dtype):
    """The row ``q`` at ``position`` through the plain kernel and, in bfloat16 with sizes they take, both matrix-core ones."""
    rest = (dev(bias), dev(mix))
    found = [ops.sigmoid_attention_generic(q, H, G, d, dv, k_pages, v_pages, table, ints([0]), ints([position]), scale, window, *rest, gate)]
    if dtype == torch.bfloat16 and ops.sigmoid_attention_is_tiled(H, d, dv):
        found.append(ops.sigmoid_attention_decode(H, G, d, dv, k_pages, v_pages, table, ints([0]), ints([position]), scale, window, *rest,
                                                  position + 1, gate=gate, q=q))
        for parts in (1, 2):
            found.append(ops.sigmoid_attention_prefill(q, H, G, d, dv, k_pages, v_pages, table, ints([0]), ints([0]), ints([0, 1]), ints([position]),
                                                       scale, window, *rest, gate, parts=parts))
    return [host(f)[0].reshape(H, dv) for f in found]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [40, 64, 65, 1, 130, 0])
def test_a_key_just_inside_and_just_outside_the_window(ops, dtype, window):
    """One key matches the query, all others score far below zero: the row at 299 sees it at 299 - window + 1 and not one
    place earlier; at page borders; far back without a window. Every head mixes the weights of another head."""
    H, G, d, dv, T = 4, 2, 32, 48, 300
    rng = np.random.default_rng(window)
    pages = [7, 2, 9, 0, 4]
    values = stored(rng.normal(size=(T, G, dv)), dtype)
    mix = np.roll(np.eye(H), 1, axis=0) * np.array([1.0, -2.0, 0.5, 3.0])[:, None]      # head h carries head h - 1's weights
    q = np.zeros((1, H * d)); q[0, 5::d] = 4.0
    edge = T - window if window else 0
    targets = [(edge, True), (edge - 1, False), (T - 1, True), (256, window == 0 or T - 1 - 256 < window), (255, window == 0 or T - 1 - 255 < window),
               (3, window == 0)]
    for target, seen in targets:
        if target < 0:
            continue
        keys = np.zeros((T, G, d))
        keys[:, :, 5] = -4.0
        keys[target, :, 5] = 4.0
        k_pages, v_pages = paged(keys, values, dtype, pages)
        for found in one_row(ops, dev(q, dtype), H, G, d, dv, k_pages, v_pages, ints([pages]), T - 1, 2.0, window, np.zeros(H), mix, None, dtype):
            for head in range(H):
                want = mix[head].sum() * values[target, head // 2] if seen else np.zeros(dv)
                assert np.abs(found[head] - want).max() < 0.06, f"window {window}, key {target}, head {head}"


# heads, key heads, sizes, window: groups of 1, 2, 3, 4 and more heads, heads in every padding, sizes in every class of the
# kernels, values wider and narrower than keys, and sizes that only the plain kernel takes
SHAPES = [(6, 3, 32, 48, 50), (4, 4, 16, 16, 33), (2, 1, 48, 32, 64), (3, 1, 20, 24, 0), (16, 4, 64, 64, 150), (12, 4, 80, 128, 70), (9, 3, 128, 96, 0),
          (5, 1, 256, 160, 90), (1, 1, 16, 16, 1), (13, 13, 32, 16, 100), (8, 1, 112, 64, 129), (20, 5, 32, 32, 60), (10, 2, 144, 256, 0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv,window", SHAPES)
def test_attention_against_the_plain_heads(ops, dtype, H, G, d, dv, window):
    """Rows at several positions of a sequence of 300 (in the first window, across page borders, at the end), and in
    bfloat16 the whole sequence as one prompt and as a portion behind cached keys, its keys shared by one to eight
    workgroups."""
    T = 300
    rng = np.random.default_rng(H + d)
    pages = [3, 6, 0, 2, 5]
    q_all = stored(plain.rms(rng.normal(size=(T, H, d)), 1e-6), dtype)
    keys, values = stored(plain.rms(rng.normal(size=(T, G, d)), 1e-6), dtype), stored(rng.normal(size=(T, G, dv)), dtype)
    bias, mix = stored(rng.normal(-1.0, 0.7, H), torch.float32), stored(rng.normal(size=(H, H)), torch.float32)
    gates = stored(rng.normal(size=(T, H * dv + 3)), torch.float32)
    scale = 2.3 * d ** -0.5
    expected = plain.mixed_heads(q_all, keys, values, 0, scale, bias, mix, window or None)
    expected = expected * plain.sigmoid(gates[:, 3:]).reshape(T, H, dv)
    k_pages, v_pages = paged(keys, values, dtype, pages)
    limit = (2e-5 if dtype == torch.float32 else 1.5e-2) * np.abs(expected).max()
    table, gate = ints([pages]), dev(gates)[:, 3:]
    for position in (0, 1, max(window - 1, 0), window, 63, 64, 65, 128, 299):
        q = dev(q_all[position].reshape(1, H * d), dtype)
        for found in one_row(ops, q, H, G, d, dv, k_pages, v_pages, table, position, scale, window, bias, mix, gate[position:position + 1], dtype):
            assert np.abs(found - expected[position]).max() <= limit, f"position {position}"
    if dtype == torch.bfloat16 and ops.sigmoid_attention_is_tiled(H, d, dv):
        for first in (0, 130, 283):
            seg_row0 = [0, T - first]
            tile_seg, tile_row0 = ops.query_tiles(seg_row0)
            q = dev(q_all[first:].reshape(T - first, H * d), dtype)
            for parts in (0, 1, 2, 8):
                found = ops.sigmoid_attention_prefill(q, H, G, d, dv, k_pages, v_pages, table, ints(tile_seg), ints(tile_row0), ints(seg_row0),
                                                      ints(np.arange(first, T)), scale, window, dev(bias), dev(mix), gate[first:], parts=parts)
                assert np.abs(host(found).reshape(-1, H, dv) - expected[first:]).max() <= limit, f"rows from {first}, {parts} parts"


def test_which_sizes_the_matrix_core_kernels_take(ops):
    taken = {shape[:4]: ops.sigmoid_attention_is_tiled(shape[0], shape[2], shape[3]) for shape in SHAPES}
    assert not taken[(3, 1, 20, 24)] and not taken[(20, 5, 32, 32)] and taken[(16, 4, 64, 64)] and taken[(5, 1, 256, 160)]
    assert ops.sigmoid_attention_is_tiled(16, 128, 128) and not ops.sigmoid_attention_is_tiled(16, 256, 256)
    assert not ops.sigmoid_attention_is_tiled(4, 272, 64) and not ops.sigmoid_attention_is_tiled(4, 64, 24)


@pytest.mark.parametrize("dtype", DTYPES)
def test_segments_of_unequal_length_and_a_decode_prefix(ops, dtype):
    """One step of single rows and portions: every row equals the row alone (the plain kernel), whichever kernels the
    step's rows go to."""
    H, G, d, dv, window = 6, 2, 32, 48, 100
    rng = np.random.default_rng(3)
    starts, counts = [200, 64, 0, 0, 77], [1, 1, 1, 130, 19]
    stride = 5
    table = rng.permutation(5 * stride).reshape(5, stride)
    k_pages, v_pages = dev(rng.normal(size=(26, G, 64, d)), dtype), dev(rng.normal(size=(26, G, dv, 64)), dtype)
    rows = sum(counts)
    q, gate = dev(rng.normal(size=(rows, H * d)), dtype), dev(rng.normal(size=(rows, H * dv)))
    bias, mix = dev(rng.normal(size=H)), dev(rng.normal(size=(H, H)))
    row_seg, row_pos = np.repeat(np.arange(5), counts), np.concatenate([np.arange(s, s + n) for s, n in zip(starts, counts)])
    seg_row0 = np.concatenate([[0], np.cumsum(counts)])
    tile_seg, tile_row0 = ops.query_tiles(seg_row0.tolist())

    class Ctx:
        all_decode, decode_prefix, max_context = False, 3, 201
    ctx = Ctx()
    ctx.row_seg, ctx.row_pos, ctx.seg_row0 = ints(row_seg), ints(row_pos), ints(seg_row0)
    found = ops.sigmoid_attention(q, H, G, d, dv, k_pages, v_pages, ints(table), ctx, 0.2, window, bias, mix, gate, tile_seg=ints(tile_seg),
                                  tile_row0=ints(tile_row0))
    want = ops.sigmoid_attention_generic(q.float(), H, G, d, dv, k_pages.float(), v_pages.float(), ints(table), ctx.row_seg, ctx.row_pos, 0.2, window,
                                         bias, mix, gate)
    limit = (1e-6 if dtype == torch.float32 else 1.5e-2) * float(want.abs().max())
    assert float((found.float() - want).abs().max()) <= limit


def test_the_decode_step_that_norms_and_stores(ops):
    """The raw projections through one kernel (per-head norm of queries and keys, cache write, attention, gate) give bit
    for bit what the two kernels apart give, and leave the same pages; with one to many workgroups a row."""
    for H, G, d, dv, window, B in ((4, 2, 32, 32, 50, 3), (16, 4, 128, 128, 0, 5), (3, 3, 48, 80, 70, 2), (12, 2, 96, 64, 300, 16)):
        rng = np.random.default_rng(H)
        positions = rng.integers(0, 320, size=B)
        positions[0] = 64
        table = ints(rng.permutation(B * 5).reshape(B, 5))
        k_pages, v_pages = dev(rng.normal(size=(B * 5 + 1, G, 64, d)), torch.bfloat16), dev(rng.normal(size=(B * 5 + 1, G, dv, 64)), torch.bfloat16)
        wide = dev(rng.normal(size=(B, (H + G) * d + G * dv + H * dv)))
        width = (H + G) * d + G * dv
        qkv, gate = wide[:, :width], wide[:, width:]
        bias, mix, ones = dev(rng.normal(size=H)), dev(rng.normal(size=(H, H))), dev(np.ones(d))
        k_apart, v_apart, k_one, v_one = k_pages.clone(), v_pages.clone(), k_pages.clone(), v_pages.clone()
        q = ops.qk_norm_rope_kv_write(qkv, H, G, d, ones, ones, 1e-5, None, None, 0, k_apart, v_apart, table, ints(np.arange(B)), ints(positions), v_dim=dv)
        unit = plain.rms(host(qkv)[:, :(H + G) * d].reshape(B, H + G, d), 1e-5)
        assert np.abs(host(q).reshape(B, H, d) - unit[:, :H]).max() <= 1e-2 * np.abs(unit).max()
        for r, p in enumerate(positions):
            assert np.abs(host(k_apart[int(table[r, p // 64]), :, p % 64]) - unit[r, H:]).max() <= 1e-2 * np.abs(unit).max()
        common = (table, ints(np.arange(B)), ints(positions), 0.3, window, bias, mix, 320)
        was = ops.SIGMOID_DECODE_WORKGROUPS
        try:
            for workgroups in (was, 1):
                ops.SIGMOID_DECODE_WORKGROUPS = workgroups
                apart = ops.sigmoid_attention_decode(H, G, d, dv, k_apart, v_apart, *common, gate=gate, q=q)
                k_one.copy_(k_pages), v_one.copy_(v_pages)
                one = ops.sigmoid_attention_decode(H, G, d, dv, k_one, v_one, *common, gate=gate, qkv=qkv, eps=1e-5)
                assert torch.equal(one, apart) and torch.equal(k_one, k_apart) and torch.equal(v_one, v_apart)
        finally:
            ops.SIGMOID_DECODE_WORKGROUPS = was


def test_refusals(ops):
    from flyweight_amd.kernels.ops import KernelError
    H, G, d = 4, 2, 32
    k, v = torch.zeros((2, G, 64, d), device=DEV), torch.zeros((2, G, d, 64), device=DEV)
    q, table, one = torch.zeros((1, H * d), device=DEV), ints([[0, 1]]), ints([0])
    bias, mix = torch.zeros(H, device=DEV), torch.zeros((H, H), device=DEV)
    ops.sigmoid_attention_generic(q, H, G, d, d, k, v, table, one, one, 1.0, 0, bias, mix)
    with pytest.raises(KernelError, match="mix"):
        ops.sigmoid_attention_generic(q, H, G, d, d, k, v, table, one, one, 1.0, 0, bias, mix[:2].contiguous())
    with pytest.raises(KernelError, match="gate"):
        ops.sigmoid_attention_generic(q, H, G, d, d, k, v, table, one, one, 1.0, 0, bias, mix, torch.zeros((1, 5), device=DEV))
    with pytest.raises(KernelError, match="window"):
        ops.sigmoid_attention_generic(q, H, G, d, d, k, v, table, one, one, 1.0, -1, bias, mix)
    with pytest.raises(KernelError, match="one of the two"):
        ops.sigmoid_attention_decode(H, G, d, d, k, v, table, one, one, 1.0, 0, bias, mix, 64)
    with pytest.raises(KernelError, match="bfloat16"):
        ops.sigmoid_attention_decode(H, G, d, d, k, v, table, one, one, 1.0, 0, bias, mix, 64, qkv=torch.zeros((1, (H + 2 * G) * d), device=DEV))
    with pytest.raises(KernelError, match="block table"):
        ops.sigmoid_attention_decode(H, G, d, d, k.bfloat16(), v.bfloat16(), table, one, one, 1.0, 0, bias, mix, 200, q=q.bfloat16())


# ---- norms, joined rows, gelu ------------------------------------------------------------------------------------
@pytest.mark.parametrize("hidden", [40, 1000, 1500, 3000, 5000])
def test_layer_norms_with_bias_around_a_sublayer(ops, hidden):
    rng = np.random.default_rng(hidden)
    rows = 6
    x, a = rng.normal(2.0, 1.5, size=(rows, hidden)), rng.normal(-1.0, 2.0, size=(rows, hidden))
    w, b, w2, b2 = (rng.normal(size=hidden) for _ in range(4))
    new = stored(x, torch.float32) - 0.7 * plain.layer_norm(stored(a, torch.float32), w, b, 1e-5)
    limit = 2e-5 * np.abs(new).max()
    found = host(ops.layernorm_rows(dev(x), dev(w), 1e-5, torch.float32, row_index=ints([4, 0, 4]), bias=dev(b)))
    assert np.abs(found - plain.layer_norm(x, w, b, 1e-5)[[4, 0, 4]]).max() <= 2e-5 * np.abs(found).max()
    for dtype in DTYPES:
        for kind in (ops.NEXT_NOTHING, ops.NEXT_ROUNDED, ops.NEXT_CENTERED, ops.NEXT_RMS):
            rows_x = dev(x)
            out = ops.norm_add_norm_(rows_x, dev(a), dev(w), True, 1e-5, bias=dev(b), mult=-0.7, next_kind=kind, next_weight=dev(w2), next_bias=dev(b2),
                                     next_eps=1e-6, next_dtype=dtype)
            assert np.abs(host(rows_x) - new).max() <= limit
            want = {ops.NEXT_NOTHING: None, ops.NEXT_ROUNDED: new, ops.NEXT_CENTERED: plain.layer_norm(new, w2, b2, 1e-6),
                    ops.NEXT_RMS: plain.rms(new, 1e-6) * w2 + b2}[kind]
            if want is not None:
                assert np.abs(host(out) - want).max() <= (2e-5 if dtype == torch.float32 else 1e-2) * np.abs(want).max()
        # the rows beside others: x's half of [x | x0], the other half untouched
        joined = ops.place_rows(dev(x), torch.zeros((rows, 2 * hidden), dtype=dtype, device=DEV), twice=True)
        assert np.array_equal(host(joined), stored(np.concatenate([x, x], axis=1).astype(np.float32), dtype))
        ops.norm_add_norm_(dev(x), dev(a), dev(w), True, 1e-5, bias=dev(b), mult=-0.7, next_kind=ops.NEXT_ROUNDED, next_dtype=dtype,
                           next_out=joined[:, :hidden])
        assert np.abs(host(joined)[:, :hidden] - new).max() <= (2e-5 if dtype == torch.float32 else 1e-2) * np.abs(new).max()
        assert np.array_equal(host(joined)[:, hidden:], stored(x.astype(np.float32), dtype))


# every product that stores: the fused one, the one that splits K, the skinny one (K no multiple of 32), the tiled ones
@pytest.mark.parametrize("rows,N,K", [(1, 40, 96), (8, 3200, 256), (13, 100, 40), (40, 300, 128), (64, 96, 2048), (100, 200, 64), (300, 1024, 512), (700, 4096, 256),
                                      (2048, 4096, 128), (200, 130, 44), (256, 6144, 4096)])
def test_gelu_in_the_products(ops, rows, N, K):
    from flyweight_amd.parts.linear import Linear
    rng = np.random.default_rng(rows)
    a, w = stored(rng.normal(size=(rows, K)), torch.bfloat16), stored(rng.normal(0, 1.5, size=(N, K)) * K ** -0.5, torch.bfloat16)
    want = plain.gelu_erf(a @ w.T)
    found = host(Linear(dev(w, torch.bfloat16)).gelu(dev(a, torch.bfloat16)))
    assert np.abs(found - want).max() <= 6e-3 * np.abs(want).max()
    if rows <= 100:
        found = host(Linear(dev(w)).gelu(dev(a)))
        assert np.abs(found - want).max() <= 5e-6 * np.abs(want).max()


def test_gelu_rows(ops):
    z = np.concatenate([np.linspace(-9.0, 9.0, 1001), [0.0, -0.0, 1e-8, 40.0, -40.0]])
    assert np.abs(host(ops.gelu_rows(dev(z), torch.float32)) - plain.gelu_erf(stored(z, torch.float32))).max() < 2e-6


# ---- the router ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("scores", ["sigmoid", "softmax_all"])
@pytest.mark.parametrize("experts,top,groups,keep", [(2, 1, 2, 1), (9, 3, 3, 2), (16, 2, 2, 1), (8, 4, 4, 2), (64, 4, 8, 3), (200, 9, 4, 1), (6, 6, 1, 1), (128, 3, 64, 5),
                                                     (400, 5, 4, 2)])
def test_route_by_pairs(ops, scores, experts, top, groups, keep):
    rng = np.random.default_rng(experts + top)
    logits = rng.normal(size=(57, experts)).astype(np.float32) * 2
    logits[3] = 0.0                                           # all equal: the lowest groups, then the lowest ids
    logits[4] = -1.0
    logits[4, experts - 1] = 3.0                              # the best expert sits beside poor ones
    if experts > groups > 1:
        logits[5] = -2.0
        logits[5, :2] = 1.0                                   # the two best are equal: a group's pair may be a tie
    chosen, weight = ops.moe_route(dev(logits), None, top, groups, keep, scores=scores, group_pair=True)
    if scores == "sigmoid":
        want_chosen, want_weight = plain.route(logits.astype(np.float64), np.eye(experts), top, groups, keep)
    else:       # the plain router on logits whose sigmoids are the softmax's scores
        s = np.exp(logits.astype(np.float64))
        s /= s.sum(axis=1, keepdims=True)
        want_chosen, want_weight = plain.route(np.log(s / (1.0 - s)), np.eye(experts), top, groups, keep)
    same = (host(chosen).astype(np.int64) == want_chosen).all(axis=1)
    assert same[[0, 1, 2, 4]].all() and same.mean() > 0.98      # (two groups' sums may differ by less than float32 holds)
    if scores == "sigmoid":
        assert same[3]
    assert np.abs(host(weight) - want_weight)[same].max() < 2e-6
    per_group = experts // groups
    assert all(len({e // per_group for e in row}) <= keep for row in host(chosen).astype(np.int64))


# ---- the latent's rotation by halves, the gate per head ---------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank,rot,turn", [(48, 16, 16), (32, 32, 8), (100, 2, 2), (24, 6, 0), (40, 12, 4)])
def test_latent_store_and_queries_with_halves_turned(ops, dtype, rank, rot, turn):
    rng = np.random.default_rng(rank)
    positions = np.array([0, 1, 63, 64, 130, 700])
    rows, heads, dim = len(positions), 3, 8
    raw, weight = rng.normal(size=(rows, rank + rot + 5)), rng.uniform(0.5, 1.5, rank)
    pages = [3, 0, 2, 5, 1, 4, 6, 7, 8, 9, 10]
    k_pages = torch.full((11, 1, 64, rank + rot), float("nan"), dtype=dtype, device=DEV)
    v_pages = torch.full((11, 1, rank, 64), float("nan"), dtype=dtype, device=DEV)
    inv_freq = dev(100.0 ** (-2.0 * np.arange(turn // 2) / max(turn, 1)), torch.float64)
    cos, sin = ops.rope_table(ints(positions), inv_freq) if turn else (None, None)
    ops.latent_norm_write(dev(raw)[:, :rank + rot], dev(weight), 1e-5, k_pages, v_pages, ints([pages] * rows), ints(np.arange(rows)), ints(positions),
                          rot=rot, cos=cos, sin=sin, turn=turn, interleaved=False)
    c, part = plain.rms(raw[:, :rank], 1e-5) * weight, plain.rotate_halves(raw[:, rank:rank + rot], positions, turn, 100.0)
    limit = (1e-5 if dtype == torch.float32 else 1e-2) * 4.0
    for r, p in enumerate(positions):
        key = host(k_pages[pages[p // 64], 0, p % 64])
        assert np.abs(key[:rank] - c[r]).max() <= limit and np.abs(key[rank:] - part[r]).max() <= limit
        assert np.abs(host(v_pages[pages[p // 64], 0, :, p % 64]) - c[r]).max() <= limit
    q = stored(rng.normal(size=(rows, heads * (dim + rot))), dtype)
    out = torch.zeros((rows, heads * (rank + rot)), dtype=dtype, device=DEV)
    ops.rotate_place(dev(q, dtype), heads, dim, rot, cos, sin, out, rank, turn=turn, interleaved=False)
    want = plain.rotate_halves(q.reshape(rows, heads, dim + rot)[..., dim:], positions, turn, 100.0)
    assert np.abs(host(out).reshape(rows, heads, rank + rot)[..., rank:] - want).max() <= limit


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [3, 40])
@pytest.mark.parametrize("heads,N,K", [(4, 16, 48), (3, 24, 40), (1, 12, 25), (5, 1, 16)])
def test_map_per_head_with_one_gate_a_head(ops, dtype, rows, heads, N, K):
    rng = np.random.default_rng(heads * N + rows)
    x, w = stored(rng.normal(size=(rows, heads * K)), dtype), stored(rng.normal(size=(heads, N, K)) * K ** -0.5, dtype)
    gate = stored(rng.normal(size=(rows, heads + 7)), torch.float32)
    found = host(ops.head_linear(dev(x, dtype), dev(w, dtype), dtype, gate=dev(gate)[:, 7:])).reshape(rows, heads, N)
    want = np.stack([x.reshape(rows, heads, K)[:, h] @ w[h].T for h in range(heads)], axis=1) * plain.sigmoid(gate[:, 7:])[:, :, None]
    assert np.abs(found - want).max() <= (2e-5 if dtype == torch.float32 else 1.5e-2) * max(1.0, np.abs(want).max())
