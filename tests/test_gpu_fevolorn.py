"""Fevolorn through the engine against the plain float64 model (tests/plain_fevolorn.py): whole prompts,
token-by-token decoding, portions down to two tokens, mixed batches on few pages and slots, each mixer alone, a key that
decides the output inside the window alone, a far token that stays in the state, long decoding, the streams after every
layer, greedy generation through the scheduler, trace replay and the command line. In 32-bit and bfloat16."""

import json
import subprocess

import numpy as np
import pytest

import plain_fevolorn as plain
from fevolorn_common import CONFIGS, assert_close, dense, layer, lightning, make_folder, model, moe, only_mixer, parallel, random_tokens

pytestmark = pytest.mark.gpu

DTYPES = ("float32", "bfloat16")


class Loaded:
    def __init__(self, folder, config, dtype, seed=0, change=None):
        from flyweight_amd.engine import load_model
        self.config = config
        self.weights = make_folder(folder, config, seed=seed, change=change)
        self.folder, self.dtype = folder, dtype
        _, self.model = load_model(folder, dtype=dtype)
        self._expected = {}

    def stepper(self, num_pages, max_requests=4):
        from flyweight_amd.engine import Stepper
        return Stepper(self.model, num_pages=num_pages, max_requests=max_requests, context_limit=num_pages * 64)

    def expected(self, tokens):
        key = tuple(tokens)
        if key not in self._expected:
            self._expected[key] = plain.forward(self.config, self.weights, list(tokens))
        return self._expected[key]


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    root = tmp_path_factory.mktemp("fevolorn")
    made = {}

    def get(name, dtype, variant=""):
        key = (name, dtype, variant)
        if key not in made:
            config = CONFIGS[name] if not variant else only_mixer(CONFIGS[name], variant)
            made[key] = Loaded(str(root / f"{name}{variant}_{dtype}"), config, dtype, seed=len(name) + len(variant))
        return made[key]
    return get


def feed(stepper, request, tokens, cuts):
    """Feeds ``tokens`` in portions of the given sizes (cycled) and returns the logits at every position."""
    from flyweight_amd.engine import StepEntry
    out, at, i = [], 0, 0
    while at < len(tokens):
        n = min(cuts[i % len(cuts)], len(tokens) - at)
        out.append(stepper.step([StepEntry(request, list(tokens[at:at + n]), list(range(n)))]).cpu().numpy())
        at, i = at + n, i + 1
    return np.concatenate(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["X", "Y", "Z"])
def test_whole_prompt(models, name, dtype):
    loaded = models(name, dtype)
    tokens = random_tokens(loaded.config["vocab"], 200, seed=1)
    stepper = loaded.stepper(num_pages=8)
    stepper.admit("a")
    assert_close(feed(stepper, "a", tokens, [len(tokens)]), loaded.expected(tokens), dtype, f"{name} whole")
    for count in (1, 2):        # the first tokens of a sequence alone
        stepper.admit(("short", count))
        assert_close(feed(stepper, ("short", count), tokens[:count], [count]), loaded.expected(tokens[:count]), dtype, f"{name} first {count}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["X", "Y", "Z"])
def test_token_by_token_against_prefill(models, name, dtype):
    """Every token decoded alone, 170 steps: the windows (1, 33, 50, 64, 130 keys) pass over decoded tokens and
    page borders, recorded steps are replayed through every pass of the loop."""
    loaded = models(name, dtype)
    tokens = random_tokens(loaded.config["vocab"], 170, seed=2)
    stepper = loaded.stepper(num_pages=6)
    stepper.admit(0)
    assert_close(feed(stepper, 0, tokens, [1]), loaded.expected(tokens), dtype, f"{name} decoded")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["X", "Y", "Z"])
@pytest.mark.parametrize("cuts", [[2], [3, 2, 64, 5, 2, 33, 65, 9], [63, 1, 1, 64, 2], [7]])
def test_portions(models, name, dtype, cuts):
    loaded = models(name, dtype)
    tokens = random_tokens(loaded.config["vocab"], 150, seed=3)
    stepper = loaded.stepper(num_pages=6)
    stepper.admit("p")
    assert_close(feed(stepper, "p", tokens, cuts), loaded.expected(tokens), dtype, f"{name} portions {cuts}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(models, dtype):
    """A short prompt and 330 tokens decoded one by one: five pages, ten windows of the shorter mask, pages of the
    windowed layers handed back in every pass, states moved on 330 times."""
    loaded = models("Y", dtype)
    tokens = random_tokens(loaded.config["vocab"], 340, seed=9)
    stepper = loaded.stepper(num_pages=6)
    stepper.admit("long")
    head = feed(stepper, "long", tokens[:10], [10])
    tail = feed(stepper, "long", tokens[10:], [1])
    assert_close(np.concatenate([head, tail]), loaded.expected(tokens), dtype, "Y long decoding")
    stepper.cache.check_invariants()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_key_that_decides_the_output_inside_the_window_alone(dtype, tmp_path):
    """One layer in which a marker token's key matches the queries of every token and no other key does: its value stands
    in the logits of exactly the rows whose window (70 keys) reaches it, whether the marker and the rows came in one
    prompt, in portions cut beside the edge, or decoded. (The scan beside the attention reads nothing here.)"""
    D, V, window, marker = 32, 20, 70, 19
    config = model(V, D, 2, [layer(parallel(2, 1, 16, 32, window, 4.0, 16, 4, 4, 2), None)])

    def change(weights):
        # embed: a component that every token has (channel 0) and one of the marker's alone (channel 1)
        rng = np.random.default_rng(5)
        weights["embed"][:] = 0.3 * rng.normal(size=(V, D))
        weights["embed"][:, 0] = 3.0
        weights["embed"][:, 1] = 0.0
        weights["embed"][marker, 1] = 6.0
        for name in ("l0.mix.left.q", "l0.mix.left.k", "l0.mix.right.in"):
            weights[name][:] = 0.0
        weights["l0.mix.left.q"][0::16, 0] = 4.0            # every query along channel 0 of its head
        weights["l0.mix.left.k"][0, 1], weights["l0.mix.left.k"][1, 0] = 16.0, 1.0     # the marker's key too; any other's beside it
        weights["l0.mix.left.q.norm"][:] = weights["l0.mix.left.k.norm"][:] = 1.0
        weights["l0.mix.right.conv.b"][:] = 0.0             # x and z are zero, and so is what the scan gives
    loaded = Loaded(str(tmp_path / "m"), config, dtype, seed=1, change=change)
    tokens = random_tokens(V - 1, 150, seed=6)
    at = 40
    without = loaded.expected(tokens)
    tokens = list(tokens[:at]) + [marker] + list(tokens[at + 1:])
    expected = loaded.expected(tokens)
    moved = np.abs(expected - without).max(axis=-1)
    inside, outside = moved[at:at + window], moved[at + window:]
    assert inside.min() > 10.0 * max(outside.max(), 1e-9) and inside.min() > 0.3       # the oracle: the edge shows
    for cuts in ([150], [1], [at, 1, window - 1, 1, 1, 50], [at + window - 2, 2, 2, 40], [2]):
        stepper = loaded.stepper(num_pages=3)
        stepper.admit("a")
        found = feed(stepper, "a", tokens, cuts)
        assert_close(found, expected, dtype, f"marker's key, cut {cuts[:4]}")
        seen = np.abs(found - without).max(axis=-1) > 0.5 * inside.min()
        assert seen[at:at + window].all() and not seen[at + window:].any() and not seen[:at].any()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["lightning", "mamba"])
def test_a_far_token_stays_in_the_state(kind, dtype, tmp_path):
    """One layer whose recurrence takes in a marker token's value alone and forgets nothing (or a hundredth a token): the rows far
    behind the marker still carry it, whatever the portions between, and none ahead of it does."""
    D, V, marker, at, count = 32, 20, 19, 30, 260
    config = model(V, D, 2, [layer(lightning(2, 16, 16, [1.0, 0.99]) if kind == "lightning" else parallel(1, 1, 16, 16, 1, 1.0, 32, 4, 4, 3), None)])

    def change(weights):
        rng = np.random.default_rng(5)
        weights["embed"][:] = 0.3 * rng.normal(size=(V, D))
        weights["embed"][:, 0] = 3.0
        weights["embed"][:, 1] = 0.0
        weights["embed"][marker, 1] = 6.0
        weights["l0.norm1.b"][:] = 0.0
        if kind == "lightning":
            for name in ("q", "k", "v"):
                weights["l0.mix." + name][:] = 0.0
            weights["l0.mix.q"][:, 0] = 3.0                 # queries that every token asks, a key and a value of the marker's alone
            weights["l0.mix.k"][:, 1] = weights["l0.mix.v"][:, 1] = 3.0
            weights["l0.mix.v"][::2, 1] = 1.0
        else:
            right = "l0.mix.right."
            weights[right + "in"][:32] = 0.0
            weights[right + "in"][:32, 1] = 4.0             # x is the marker's alone; z as drawn
            weights[right + "conv.b"][:] = 0.0
            weights[right + "A_log"][:] = -6.0              # forgets a thousandth a token
            weights[right + "D"][:] = 0.0
            weights[right + "x"][:] = np.abs(weights[right + "x"])
            weights[right + "dt.b"][:] = 0.5
            weights["l0.mix.left.o"][:] = 0.0
    loaded = Loaded(str(tmp_path / "m"), config, dtype, seed=1, change=change)
    tokens = random_tokens(V - 1, count, seed=6)
    without = loaded.expected(tokens)
    tokens = list(tokens[:at]) + [marker] + list(tokens[at + 1:])
    expected = loaded.expected(tokens)
    moved = np.abs(expected - without).max(axis=-1)
    if kind == "lightning":
        assert moved[at:].min() > 0.3 and moved[:at].max() < 1e-9       # the oracle: the state shows to the end
    for cuts in ([count], [1], [64, 2, 33, 32, 65, 1], [at + 1, 200, 2]):
        stepper = loaded.stepper(num_pages=5)
        stepper.admit("a")
        assert_close(feed(stepper, "a", tokens, cuts), expected, dtype, f"{kind} far token, cut {cuts[:4]}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_wider_model_through_the_prompt_kernels(models, dtype):
    """500 tokens of a model of width 512: whole (the tiled products with their gated gelu, the matrix-core attention, the
    grouped products of sixteen experts, eight chunks of either recurrence), cut at odd places, and its last 40 tokens
    decoded one by one beside a second request's portions."""
    from flyweight_amd.engine import StepEntry
    loaded = models("W", dtype)
    tokens = random_tokens(loaded.config["vocab"], 500, seed=7)
    other = random_tokens(loaded.config["vocab"], 300, seed=8)
    expected = loaded.expected(tokens)
    stepper = loaded.stepper(num_pages=26)
    stepper.admit("whole")
    assert_close(feed(stepper, "whole", tokens, [500]), expected, dtype, "W whole")
    stepper.release("whole")
    stepper.admit("cut")
    assert_close(feed(stepper, "cut", tokens, [257, 17, 100, 63, 63]), expected, dtype, "W cut")
    stepper.release("cut")
    stepper.admit("a")
    stepper.admit("b")
    head = feed(stepper, "a", tokens[:460], [460])
    rows, at = [], 0
    for i in range(460, 500):
        entries = [StepEntry("a", [tokens[i]], [0])]
        if at < len(other):
            entries.append(StepEntry("b", other[at:at + 9], []))
            at += 9
        rows.append(stepper.step(entries).cpu().numpy())
    assert_close(np.concatenate([head] + rows), expected, dtype, "W decoded beside another request")
    stepper.release("a")
    stepper.release("b")
    # and alone, so that decode steps are recorded and replayed
    stepper.admit("c")
    head = feed(stepper, "c", tokens[:480], [480])
    assert_close(np.concatenate([head, feed(stepper, "c", tokens[480:], [1])]), expected, dtype, "W decoded alone")


@pytest.mark.parametrize("dtype", DTYPES)
def test_many_single_rows_at_once(models, dtype):
    """24 requests decoded together (more than the fused decode steps take: the norm, the cache write and the step sizes' map are kernels of their own):
    every row equals its request alone."""
    from flyweight_amd.engine import StepEntry
    loaded = models("X", dtype)
    prompts = {i: random_tokens(loaded.config["vocab"], 3 + 4 * i, seed=100 + i) for i in range(24)}
    stepper = loaded.stepper(num_pages=60, max_requests=24)
    for i, tokens in prompts.items():
        stepper.admit(i)
        feed(stepper, i, tokens[:-2], [len(tokens)])
    steps = [stepper.step([StepEntry(i, [tokens[place]], [0]) for i, tokens in prompts.items()]).cpu().numpy() for place in (-2, -1)]
    for i, tokens in prompts.items():
        assert_close(np.stack([s[i] for s in steps]), loaded.expected(tokens)[-2:], dtype, f"request {i}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("variant", ["lightning", "parallel"])
@pytest.mark.parametrize("name", ["X", "Y", "Z"])
def test_each_mixer_alone(models, name, variant, dtype):
    loaded = models(name, dtype, variant)
    tokens = random_tokens(loaded.config["vocab"], 140, seed=4)
    stepper = loaded.stepper(num_pages=6)
    stepper.admit("w")
    assert_close(feed(stepper, "w", tokens, [len(tokens)]), loaded.expected(tokens), dtype, f"{name} {variant} whole")
    stepper.admit("c")
    assert_close(feed(stepper, "c", tokens, [5, 2, 70, 1, 1]), loaded.expected(tokens), dtype, f"{name} {variant} cut")


def random_config(seed):
    """One to five layers of either mixer in any order, every size drawn: heads and groups of 1..4 and more, head sizes on
    and off the matrix cores' steps of 16, windows of 1 token to longer than the prompt or none, decays from forgetting at once
    to never, scans of 1 to 40 states with ranks of 1 to 24 and 1 to 5 taps, gated units, experts with or without a
    shared unit or no feed-forward, one to nine streams, no loop or any run of layers passed one to three times. (Scans of forty
    channels and more: a sum over few of them can come out near nothing, and the norm behind it then makes its rounding large.)"""
    rng = np.random.default_rng(seed)
    pick = lambda *xs: xs[int(rng.integers(len(xs)))]
    layers = []
    for _ in range(int(rng.integers(1, 6))):
        if pick(0, 1):
            kv, dim = int(pick(1, 2, 3, 4)), int(pick(16, 20, 32, 48, 64, 128, 160))
            mixer = parallel(kv * int(pick(1, 2, 3, 4)), kv, dim, int(pick(dim, 16, 36, 64)), pick(None, 1, 7, 50, 64, 100, 128, 1000),
                             float(pick(dim ** -0.5, 0.1, 0.4)), int(pick(40, 64, 100, 200, 256)), int(pick(1, 4, 8, 11, 16, 24, 40)),
                             int(pick(1, 3, 8, 16, 24)), int(pick(1, 2, 3, 4, 5)))
        else:
            heads = int(pick(1, 2, 3, 5, 8))
            mixer = lightning(heads, int(pick(8, 16, 20, 32, 64, 128)), int(pick(8, 16, 40, 64, 80)),
                              [float(pick(0.1, 0.5, 0.9, 0.99, 0.999, 1.0)) for _ in range(heads)])
        mlp = pick(None, "dense", "moe", "moe")
        if mlp == "dense":
            mlp = dense(int(pick(12, 64, 100, 200)))
        elif mlp == "moe":
            experts = int(pick(1, 2, 4, 6, 16))
            mlp = moe(experts, int(pick(*[t for t in (1, 2, 4, 8) if t <= experts])), float(pick(0.5, 0.7, 1.0, 1.5)), int(pick(12, 40, 64, 100)),
                      shared=pick(None, 24, 64))
        layers.append(layer(mixer, mlp))
    start = int(rng.integers(len(layers)))
    loop = pick(None, (start, int(rng.integers(start + 1, len(layers) + 1)), int(pick(1, 2, 3))))
    return model(int(pick(97, 300, 512, 1000)), int(pick(40, 64, 96, 100, 128, 160, 192, 256, 320)), int(pick(1, 2, 3, 4, 5, 8, 9)), layers, loop=loop,
                 eps=float(pick(1e-5, 1e-6)), scale=float(pick(1.0, 2.0, 0.5)))


@pytest.mark.parametrize("seed", range(12))
def test_random_configurations(seed, tmp_path):
    """Whatever config.json gives is read from there: twelve drawn models, whole, token by token, in odd portions and
    with a decoded tail, in both dtypes, against the plain model."""
    config = random_config(seed)
    tokens = random_tokens(config["vocab"], 140, seed=seed)
    for dtype in DTYPES:
        loaded = Loaded(str(tmp_path / dtype), config, dtype, seed=seed)
        for cuts in ([140], [1], [3, 2, 64, 5, 2, 33, 65, 9], [120] + [1] * 20):
            stepper = loaded.stepper(num_pages=4, max_requests=2)
            stepper.admit("a")
            assert_close(feed(stepper, "a", tokens, cuts), loaded.expected(tokens), dtype, f"drawn model {seed} cut {cuts[:3]}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["X", "Y", "Z"])
def test_mixed_batches_on_few_pages_and_slots(models, name, dtype):
    """Eight requests of unequal length through four slots and a pool that holds four of them at most: portions
    of some beside single tokens of others, requests left out of steps, pages and slots handed on. Every row must
    equal the request run alone."""
    from flyweight_amd.engine import StepEntry
    loaded = models(name, dtype)
    rng = np.random.default_rng(5)
    vocab = loaded.config["vocab"]
    prompts = {i: random_tokens(vocab, n, seed=10 + i) for i, n in enumerate([130, 1, 67, 200, 2, 64, 97, 33])}
    stepper = loaded.stepper(num_pages=9, max_requests=4)
    waiting, live, at = list(prompts), [], {}
    got = {i: [] for i in prompts}
    steps = 0
    while waiting or live:
        while waiting and len(live) < 4:
            need = (len(prompts[waiting[0]]) + 63) // 64
            held = sum((len(prompts[r]) + 63) // 64 for r in live)
            if held + need > 9:
                break
            request = waiting.pop(0)
            stepper.admit(request)
            live.append(request)
            at[request] = 0
        entries = []
        for request in live:
            if len(live) > 1 and rng.random() < 0.25:
                continue
            left = len(prompts[request]) - at[request]
            n = 1 if left <= 20 else int(min(left - 20, rng.choice([2, 3, 17, 64, 40])))
            entries.append(StepEntry(request, prompts[request][at[request]:at[request] + n], list(range(n))))
        if not entries:
            continue
        if rng.random() < 0.5:
            entries.sort(key=lambda e: len(e.tokens) != 1)      # the scheduler's order: single tokens first
        logits = stepper.step(entries).cpu().numpy()
        row = 0
        for entry in entries:
            n = len(entry.tokens)
            got[entry.request].append(logits[row:row + n])
            row += n
            at[entry.request] += n
            if at[entry.request] == len(prompts[entry.request]):
                stepper.release(entry.request)
                live.remove(entry.request)
        steps += 1
        stepper.cache.check_invariants()
    assert steps > 40
    for request, tokens in prompts.items():
        assert_close(np.concatenate(got[request]), loaded.expected(tokens), dtype, f"{name} mixed request {request}")


def test_a_batch_does_not_change_a_request(models):
    """float32: a request's logits beside three others, on pages and slots that others have used before, are bit for bit those
    of the request alone in the same portions on a fresh cache (a recurrence's chunks begin with its portions, so another cut
    moves its sums by rounding: that is held against the plain model)."""
    from flyweight_amd.engine import StepEntry
    loaded = models("X", "float32")
    vocab = loaded.config["vocab"]
    mine = random_tokens(vocab, 120, seed=50)
    others = [random_tokens(vocab, n, seed=51 + n) for n in (90, 40, 75)]
    fresh = loaded.stepper(num_pages=4)
    fresh.admit("m")
    alone = feed(fresh, "m", mine, [50, 1, 1, 30, 38])
    stepper = loaded.stepper(num_pages=8)
    for i, tokens in enumerate(others):         # use pages and slots, then give them back
        stepper.admit(("old", i))
        feed(stepper, ("old", i), tokens, [len(tokens)])
    for i in range(len(others)):
        stepper.release(("old", i))
    for name in ("m", "o0", "o1", "o2"):
        stepper.admit(name)
    rows, at = [], 0
    for n in (50, 1, 1, 30, 38):
        entries = [StepEntry(f"o{i}", others[i][at:at + n], []) for i in range(3) if at + n <= len(others[i])]
        entries.insert(1 if entries else 0, StepEntry("m", mine[at:at + n], list(range(n))))
        rows.append(stepper.step(entries).cpu().numpy())
        at += n
    assert np.array_equal(np.concatenate(rows), alone)


@pytest.mark.parametrize("name", ["X", "Y"])
def test_greedy_generation_through_the_scheduler(models, name):
    """Several prompts at once through Runtime (admission, portions, decode steps, recorded steps): in float32 the
    tokens are the plain model's; in bfloat16 every chosen token is among the plain model's best."""
    import flyweight_amd
    from flyweight_amd.engine import EVENT_TOKEN
    loaded = models(name, "float32")
    vocab = loaded.config["vocab"]
    prompts = [random_tokens(vocab, n, seed=20 + n) for n in (37, 5, 90)]
    new = 12
    want = [plain.greedy(loaded.config, loaded.weights, prompt, new) for prompt in prompts]
    with flyweight_amd.Runtime(flyweight_amd.Model(loaded.folder, dtype="float32"), context_limit=256, parallel_sequences=3,
                               prefill_rows=16, max_batch_tokens=24) as runtime:
        tasks = [runtime.task_submit(prompt, new) for prompt in prompts]
        outputs = {task: [] for task in tasks}
        while runtime.scheduler.has_work():
            for task, value, kind in runtime.engine_step():
                if kind == EVENT_TOKEN:
                    outputs[task].append(value)
    for task, expected in zip(tasks, want):
        assert outputs[task] == expected
    with flyweight_amd.Runtime(flyweight_amd.Model(loaded.folder, dtype="bfloat16"), context_limit=256, parallel_sequences=2) as runtime:
        got = runtime.generate(prompts[0], new)
    context = list(prompts[0])
    for token in got:
        logits = plain.forward(loaded.config, loaded.weights, context)[-1]
        assert logits[token] >= logits.max() - 0.1 * np.abs(logits).max()
        context.append(token)


def test_serving_more_requests_than_slots_on_few_pages(models):
    """Seven requests through three slots and four pages a group, several decode steps per turn on the device:
    requests wait for a slot, slots and pages are handed on, recorded decode steps are replayed at changing batch
    sizes. The tokens are the plain model's (float32)."""
    import flyweight_amd
    loaded = models("Y", "float32")
    vocab = loaded.config["vocab"]
    prompts = [random_tokens(vocab, n, seed=60 + n) for n in (90, 3, 150, 64, 65, 1, 120)]
    new = [9, 14, 6, 11, 5, 16, 8]
    want = [plain.greedy(loaded.config, loaded.weights, p, n) for p, n in zip(prompts, new)]
    with flyweight_amd.Runtime(flyweight_amd.Model(loaded.folder, dtype="float32"), context_limit=192, parallel_sequences=3,
                               num_pages=4, prefill_rows=48, max_batch_tokens=56, decode_steps_per_turn=4) as runtime:
        tasks = [runtime.task_submit(p, n) for p, n in zip(prompts, new)]
        result = runtime.run()
        assert runtime.info["live_requests"] == 0
        runtime.stepper.cache.check_invariants()
    for task, expected in zip(tasks, want):
        assert result[task] == expected


def test_accounting_counts_every_pass(models):
    """A looped layer's products count as often as it runs, its weights once; the step sizes' map counts once."""
    from flyweight_amd.engine import accounting
    loaded = models("X", "bfloat16")
    shapes = plain.tensor_shapes(loaded.config)
    flops = 0
    for index in plain.layer_runs(loaded.config):
        mlp = loaded.config["layers"][index]["mlp"]
        for name, shape in shapes.items():
            parts = name.split(".")
            if parts[0] != f"l{index}" or len(shape) != 2 or parts[-1] in ("mix", "A_log", "conv", "sg", "router"):
                continue
            share = mlp["router"]["top"] / mlp["router"]["experts"] if len(parts) == 4 and parts[2].startswith("e") else 1.0
            flops += 2 * share * shape[0] * shape[1]
        if mlp is not None and mlp["kind"] == "moe":        # the router's product, the shared unit's gate in it, filled up to eights
            rows = mlp["router"]["experts"]
            flops += 2 * loaded.config["width"] * (-(-(rows + 1) // 8) * 8 if mlp.get("shared") else rows)
    assert accounting.product_flops_per_token(loaded.model) == pytest.approx(flops, rel=1e-9)
    total = sum(int(np.prod(shape)) for shape in shapes.values())
    assert accounting.step_weight_bytes(loaded.model, rows=10 ** 6) >= 2 * total       # every expert chosen: each weight once (vectors in 32-bit)
    assert accounting.step_weight_bytes(loaded.model, rows=10 ** 6) < 2.4 * total


def test_streams_after_every_layer(models):
    """The sum of the streams behind every layer run of a prompt, in both dtypes."""
    from flyweight_amd.engine import StepEntry
    for dtype, limit in (("float32", 2e-5), ("bfloat16", 3e-2)):
        loaded = models("X", dtype)
        tokens = random_tokens(loaded.config["vocab"], 50, seed=77)
        _, want = plain.PlainFevolorn(loaded.config, loaded.weights).forward(tokens, keep_layers=True)
        seen = []

        def watched(forward):
            def run(x, *args, **kwargs):
                left = forward(x, *args, **kwargs)
                seen.append(x.sum(dim=1).cpu().numpy())
                return left
            return run
        blocks = loaded.model.layers
        kept = [block.forward for block in blocks]
        try:
            for block, forward in zip(blocks, kept):
                block.forward = watched(forward)
            stepper = loaded.stepper(num_pages=2)
            stepper.admit("a")
            stepper.step([StepEntry("a", tokens, [])])
        finally:
            for block in blocks:
                del block.forward
        assert len(seen) == len(want) == 8
        for run, (found, expected) in enumerate(zip(seen, want)):
            assert np.abs(found - expected).max() <= limit * np.abs(expected).max(), f"{dtype} layer run {run}"


def test_trace_replay(models, tmp_path):
    """bin/trace_run chooses the model class by config.json and replays a mixed trace on four slots."""
    from helpers import TRACE_RUN
    loaded = models("X", "float32")
    vocab = loaded.config["vocab"]
    a, b = random_tokens(vocab, 70, seed=31), random_tokens(vocab, 9, seed=32)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:40], "want": [0, 39]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:8], "want": []}, {"id": "a", "tokens": a[40:69], "want": [28]}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[69:], "want": [0]}, {"id": "b", "tokens": b[8:], "want": [0]}], "end": ["a", "b"]},
        {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [8]}], "end": ["c"]},
    ]
    out = tmp_path / "out"
    process = subprocess.run([TRACE_RUN, "--model", loaded.folder, "--dtype", "float32", "--out", str(out), "--max-tokens", "192"],
                             input="".join(json.dumps(step) + "\n" for step in steps), capture_output=True, text=True, timeout=300)
    assert process.returncode == 0, process.stderr
    assert [line for line in process.stdout.splitlines() if line.startswith("done")] == [f"done {i}" for i in range(4)]
    full_a, full_b = loaded.expected(a), loaded.expected(b)
    read = lambda i: np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, vocab)
    assert_close(read(0), full_a[[0, 39]], "float32", "step 0")
    assert_close(read(1), full_a[[68]], "float32", "step 1")
    assert_close(read(2), np.stack([full_a[69], full_b[8]]), "float32", "step 2")
    assert_close(read(3), full_b[[8]], "float32", "step 3")


def test_command_line(models, capsys, tmp_path):
    """generate prints the plain model's greedy tokens; inspect names the architecture and its tensors;
    random-weights writes a folder from the configuration alone."""
    from flyweight_amd.cli import main
    from flyweight_amd.config import load_config
    loaded = models("Y", "float32")
    prompt = random_tokens(loaded.config["vocab"], 13, seed=40)
    expected = plain.greedy(loaded.config, loaded.weights, prompt, 5)
    assert main(["generate", loaded.folder, "--tokens", ",".join(map(str, prompt)), "--max-tokens", "5", "--temperature", "0",
                 "--dtype", "float32", "--ignore-eos", "--context", "128"]) == 0
    assert [int(t) for t in capsys.readouterr().out.split()] == expected
    assert main(["inspect", loaded.folder]) == 0
    shown = json.loads(capsys.readouterr().out)
    assert shown["architecture"] == "Fevolorn" and set(shown["tensors"]) == set(plain.tensor_shapes(loaded.config))
    (tmp_path / "config.json").write_text(json.dumps(load_config(loaded.folder).to_dict()))
    assert main(["random-weights", "--config", str(tmp_path / "config.json"), "--seed", "3", "--out", str(tmp_path / "drawn")]) == 0
    capsys.readouterr()
    assert main(["generate", str(tmp_path / "drawn"), "--tokens", "1,2,3", "--max-tokens", "4", "--temperature", "0",
                 "--ignore-eos", "--context", "128"]) == 0
    assert len(capsys.readouterr().out.split()) == 4
