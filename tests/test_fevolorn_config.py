"""Fevolorn on the CPU: its configuration and tensor names, the schedule of a looped run of layers, the cache entries it
asks for, the chunks of a step, and the plain model held against itself (a sequence in one piece against pieces with carried
state, the window's edges, the streams, the recurrences in closed form, the router's correction, the loop)."""

import copy
import types

import numpy as np
import pytest
import torch

import plain_fevolorn as plain
from fevolorn_common import CONFIG_X, CONFIG_Y, CONFIG_Z, make_folder, random_tokens


def test_config_lowers_to_parts_and_names(tmp_path):
    from flyweight_amd.config import ConfigError, FevolornConfig, load_config
    from flyweight_amd.engine.model import declared_tensors
    for name, raw in (("X", CONFIG_X), ("Y", CONFIG_Y), ("Z", CONFIG_Z)):
        folder = str(tmp_path / name)
        make_folder(folder, raw)
        config = load_config(folder)                         # the model class by config.json
        assert isinstance(config, FevolornConfig)
        spec = config.model_spec()
        assert {n: tuple(d.shape) for n, d in declared_tensors(spec).items()} == plain.tensor_shapes(raw)
        assert [layer.mixer.kind for layer in config.layers] == [entry["type"] for entry in raw["layers"]]
        assert spec.lm_head_name is None and spec.embedding_name == "embed" and spec.streams == raw["streams"]
        assert all(layer.arrangement == "stream_residual" for layer in spec.layers)
        assert FevolornConfig.from_dict(config.to_dict()) == config and config.to_dict() == raw
        assert spec.embedding_scale == raw["embedding"]["scale"]
    first, second, third, _ = FevolornConfig.from_dict(CONFIG_X).model_spec().layers
    assert first.mixer.kind == "lightning" and (first.mixer["num_heads"], first.mixer["head_dim"], first.mixer["v_head_dim"]) == (3, 32, 48)
    assert first.mixer["decay"] == (0.3, 0.93, 0.998) and first.mixer["norm_eps"] == 1e-5
    assert second.mixer.kind == "parallel_branches"
    (left_name, left, left_scale), (right_name, right, right_scale) = second.mixer["branches"]
    assert (left_name, left.kind, left_scale, right_name, right.kind, right_scale) == ("left", "gqa_attention", 0.5, "right", "mamba", 0.5)
    assert (left["num_heads"], left["num_kv_heads"], left["head_dim"], left["v_head_dim"], left["window"], left["softmax_scale"]) == (6, 3, 32, 48, 50, 0.5)
    assert left["position"].kind == "none" and left["qk_norm"] and left["qk_norm_eps"] == 1e-5
    assert (right["inner_size"], right["state_size"], right["dt_rank"], right["conv_taps"]) == (120, 12, 6, 4)
    assert second.mixer["norms"]["left"]["tensor"] == "l1.mix.left.out" and second.mixer["norms"]["right"]["tensor"] == "l1.mix.right.out"
    assert first.ffn.kind == "swiglu" and first.ffn["activation"] == "gelu_tanh" and first.ffn["intermediate_size"] == 120
    assert second.ffn.kind == "moe_swiglu" and (second.ffn["num_experts"], second.ffn["top"], second.ffn["weight_scale"]) == (9, 3, 1.7)
    assert second.ffn["router_scores"] == "sigmoid" and second.ffn["router_correction"] and not second.ffn["normalize"] and second.ffn["shared_gate"]
    assert second.ffn["shared_intermediate_size"] == 56 and third.ffn["shared_intermediate_size"] is None and not third.ffn["shared_gate"]
    assert first.mixer_norm.kind == "tanh" and first.mixer_norm["tensor"] == "l0.norm1" and second.ffn_norm["tensor"] == "l1.norm2"
    assert first.params["mixer_connection"].prefix == "l0.hc1." and second.params["ffn_connection"]["scale_tensor"] == "l1.ls2"
    spec_y = FevolornConfig.from_dict(CONFIG_Y).model_spec()
    assert spec_y.layers[2].ffn is None and "ffn_connection" not in spec_y.layers[2].params
    assert FevolornConfig.from_dict(CONFIG_Z).model_spec().layers[2].mixer["branches"][0][1]["window"] is None
    for path, value, match in ((("layers", 0, "type"), "serial", "type"), (("layers", 1, "mixer", "left", "heads"), 5, "multiple"),
                               (("layers", 0, "mixer", "decay"), [0.5], "decay"), (("layers", 0, "mixer", "decay"), 0.5, "decay"),
                               (("norm", "eps"), 0, "eps"), (("streams",), 0, "streams"), (("layers", 0, "mlp", "kind"), "glu", "kind"),
                               (("layers", 1, "mlp", "router", "top"), 10, "experts"), (("layers", 1, "mixer", "left", "mask", "size"), 0, "size"),
                               (("layers", 1, "mixer", "right", "state"), None, "state"), (("layers", 1, "mixer", "right", "conv"), 0, "conv"),
                               (("loop", "stop"), 5, "loop"), (("loop", "start"), 3, "loop"), (("loop", "times"), 0, "times"),
                               (("layers", 0, "mlp", "ff"), None, "ff"), (("vocab",), None, "vocab")):
        broken = copy.deepcopy(CONFIG_X)
        at = broken
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        with pytest.raises(ConfigError, match=match):
            FevolornConfig.from_dict(broken)


def test_parts_refuse_what_their_kernels_do_not_take():
    from flyweight_amd.config import ConfigError, FevolornConfig, LayerSpec, ModelSpec, PartSpec
    from flyweight_amd.config.spec import default_schedule
    from flyweight_amd.engine.model import CausalLM
    for path, value, match in ((("layers", 0, "mixer", "dim"), 257, "256"), (("layers", 1, "mixer", "right", "state"), 129, "128"),
                               (("layers", 1, "mixer", "right", "conv"), 17, "taps"), (("streams",), 33, "32")):
        broken = copy.deepcopy(CONFIG_X)
        at = broken
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        with pytest.raises(ConfigError, match=match):
            CausalLM(FevolornConfig.from_dict(broken).model_spec())
    # streams and layers that take them come together
    norm = PartSpec("tanh", {"size": 8, "tensor": "n"})
    one = LayerSpec("pre_norm_residual", norm, PartSpec("lightning"), norm, PartSpec("swiglu"))
    with pytest.raises(ConfigError, match="stream"):
        ModelSpec("a", 8, 8, 8, (one,), default_schedule(1), norm, "embed", None, streams=2).validate()
    with pytest.raises(ConfigError, match="stream"):
        ModelSpec("a", 8, 8, 8, (LayerSpec("stream_residual", norm, PartSpec("lightning"), None, None),), default_schedule(1), norm, "embed", None).validate()


def test_the_schedule_of_a_loop():
    """Every pass runs the looped layers with their weights and cache entries of its own."""
    from flyweight_amd.config import FevolornConfig
    spec = FevolornConfig.from_dict(CONFIG_X).model_spec()
    assert len(spec.layers) == 4
    assert [(e.layer, e.cache) for e in spec.schedule] == [(0, 0), (1, 1), (2, 2), (1, 3), (2, 4), (1, 5), (2, 6), (3, 7)]
    assert all(e.writes_cache and not e.joins_input for e in spec.schedule)
    assert [e.layer for e in FevolornConfig.from_dict(CONFIG_Y).model_spec().schedule] == [0, 0, 1, 2, 3]
    for config in (CONFIG_X, CONFIG_Y, CONFIG_Z):
        assert plain.layer_runs(config) == [e.layer for e in FevolornConfig.from_dict(config).model_spec().schedule]


def test_cache_entries():
    """A lightning layer keeps its heads' states in the request's slot, a parallel layer pages of its key heads within the
    window beside the scan's state and the convolution's last inputs; every run has its own."""
    from flyweight_amd.cache import CacheManager
    from flyweight_amd.config import FevolornConfig
    from flyweight_amd.engine.model import CausalLM
    needs = CausalLM(FevolornConfig.from_dict(CONFIG_X).model_spec()).cache_needs()
    assert set(needs) == set(range(8))
    assert needs[1] == needs[3] == needs[5] and needs[2] == needs[4] == needs[6]
    assert needs[0]["state"].shape == (3, 32, 48) and needs[2]["state"].shape == (5, 16, 16)
    left, right = needs[1]["left"], needs[1]["right"]
    assert (left.num_kv_heads, left.head_dim, left.v_head_dim, left.window) == (3, 32, 48, 50)
    assert right["state"].shape == (12, 120) and right["conv"].shape == (120, 3)
    needs_y = CausalLM(FevolornConfig.from_dict(CONFIG_Y).model_spec()).cache_needs()
    assert "conv" not in needs_y[3]["right"]                 # a convolution of one tap remembers nothing
    cache = CacheManager(needs, num_pages=6, max_requests=2, dtype=torch.float32, device=torch.device("cpu"))
    assert len(cache.groups) == 2                            # the passes' pages share a pool and a block table
    cache.admit("a")
    for length in (50, 130, 131, 200, 330):
        cache.reserve("a", length)
        cache.commit("a", length)
        cache.check_invariants()
    held = {group.need.window: [page != -1 for page in group.tables["a"]] for group in cache.groups}
    assert held[50] == [False, False, False, False, True, True] and held[130] == [False, False, False, True, True, True]
    state = cache.view((0, "state")).state
    slot = cache.describe(["a"], cache.natives_of(["a"]))[1][0]
    state[slot] = 7.0
    cache.release("a")
    assert all(group.pool.free_count == 6 for group in cache.groups)
    for name in ("b", "c"):                                  # whoever gets the slot starts from zero
        cache.admit(name)
    assert float(state[:2].abs().max()) == 0.0


def test_chunks_of_a_step():
    """Segments of more than 32 rows are cut every 64 rows from their own first row on; shorter ones are not, and a step of single
    rows asks for nothing."""
    from flyweight_amd.parts.chunks import RecurrenceChunks
    part = RecurrenceChunks()

    def arrays(lengths):
        row0 = np.concatenate([[0], np.cumsum(lengths)]).tolist()
        return part.step_arrays(types.SimpleNamespace(all_decode=all(n == 1 for n in lengths), host_seg_row0=row0))

    assert arrays([1, 1, 1]) == {}
    found = arrays([1, 32, 33, 64, 65, 2, 200])
    assert found["seg_chunk0"].tolist() == [0, 0, 0, 1, 2, 4, 4, 8]
    assert found["chunk_seg"].tolist() == [2, 3, 4, 4, 6, 6, 6, 6]
    assert found["chunk_row0"].tolist() == [33, 66, 130, 194, 197, 261, 325, 389]
    assert arrays([20, 3])["chunk_seg"].size == 0 and arrays([20, 3])["seg_chunk0"].tolist() == [0, 0, 0]


def _mix(config, index):
    entry = config["layers"][index]
    return entry, {name[len(f"l{index}.mix."):]: value for name, value in plain.random_weights(config, 3).items() if name.startswith(f"l{index}.mix.")}


def test_plain_mixers_in_one_piece_and_in_pieces():
    """Each mixer over 90 tokens at once equals the same tokens in pieces of 1, 2, 7 and 40 on the carried state."""
    rng = np.random.default_rng(0)
    for config, index in ((CONFIG_X, 0), (CONFIG_X, 1), (CONFIG_Y, 0), (CONFIG_Y, 2), (CONFIG_Z, 0), (CONFIG_Z, 1)):
        entry, w = _mix(config, index)
        h = rng.normal(size=(90, config["width"]))
        mixer = plain.lightning if entry["type"] == "lightning" else plain.parallel
        whole, _ = mixer(h, w, plain._mixer_sizes(entry), config["norm"]["eps"], None)
        for piece in (1, 2, 7, 40):
            state, parts = None, []
            for at in range(0, 90, piece):
                out, state = mixer(h[at:at + piece], w, plain._mixer_sizes(entry), config["norm"]["eps"], state)
                parts.append(out)
            assert np.allclose(np.concatenate(parts), whole, rtol=1e-10, atol=1e-10), (entry["type"], piece)


def test_plain_recurrences_in_closed_form():
    """o_t = sum_{s <= t} decay^(t - s) (q_t . k_s) v_s; a scan with one state and constant steps is a geometric sum; the
    convolution's last column is the current token's."""
    rng = np.random.default_rng(1)
    q, k, v = (rng.normal(size=(9, 2, n)) for n in (3, 3, 4))
    decay = np.array([0.5, 0.9])
    out, S = plain.decay_recurrence(q, k, v, decay, np.zeros((2, 3, 4)))
    for t in range(9):
        for h in range(2):
            want = sum(decay[h] ** (t - s) * (q[t, h] @ k[s, h]) * v[s, h] for s in range(t + 1))
            assert np.allclose(out[t, h], want)
    assert np.allclose(S[1], sum(0.9 ** (8 - s) * np.outer(k[s, 1], v[s, 1]) for s in range(9)))
    y, S = plain.selective_scan(np.ones((6, 1)), np.full((6, 1), 0.7), np.array([[-2.0]]), np.ones((6, 1)), np.full((6, 1), 3.0),
                                np.array([0.25]), np.zeros((1, 1)))
    g = np.exp(-1.4)
    assert np.allclose(y[:, 0], [3.0 * 0.7 * (1 - g ** (t + 1)) / (1 - g) + 0.25 for t in range(6)])
    y, kept = plain.causal_conv(np.array([[1.0], [10.0], [100.0]]), np.array([[2.0, 3.0, 5.0]]), np.array([0.5]), np.array([[7.0], [9.0]]))
    assert y[:, 0].tolist() == [2 * 7 + 3 * 9 + 5 * 1 + 0.5, 2 * 9 + 3 * 1 + 5 * 10 + 0.5, 2 * 1 + 3 * 10 + 5 * 100 + 0.5]
    assert kept[:, 0].tolist() == [10.0, 100.0]


def test_plain_window():
    """A key just inside the window counts, the one just outside does not, and the softmax is over the visible keys alone."""
    D = 4
    w = {"q": np.zeros((2, D)), "k": np.zeros((2, D)), "v": np.eye(D)[2:3], "o": np.eye(1), "q.norm": np.ones(2), "k.norm": np.ones(2)}
    w["q"][0, 0] = w["k"][0, 1] = w["k"][1, 0] = 1.0
    sizes = {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 1, "scale": 50.0, "window": 4}
    h = np.zeros((12, D))
    h[:, 0] = 1.0                                            # every query looks along channel 0; every key lies beside it
    h[5] = [0.0, 1.0, 8.0, 0.0]                              # but the marker's
    out, _ = plain.windowed_attention(h, w, sizes, 1e-6)
    assert np.allclose(out[6:9], 8.0) and np.allclose(out[9:], 0.0) and np.allclose(out[:5], 0.0)


def test_plain_streams():
    """All streams start equal; the mix is [from, to] and takes the old rows; with a unit mix, weights of one and one stream it
    is a plain residual sum."""
    rng = np.random.default_rng(2)
    x, y = rng.normal(size=(5, 3, 4)), rng.normal(size=(5, 4))
    mix, out = rng.normal(size=(3, 3)), rng.normal(size=3)
    joined = plain.join_streams(x, y, mix, out)
    for t in range(3):
        assert np.allclose(joined[:, t], sum(mix[s, t] * x[:, s] for s in range(3)) + out[t] * y)
    assert np.allclose(plain.join_streams(x[:, :1], y, np.eye(1), np.ones(1))[:, 0], x[:, 0] + y)
    assert np.allclose(plain.read_streams(x, np.array([1.0, -2.0, 0.5])), x[:, 0] - 2.0 * x[:, 1] + 0.5 * x[:, 2])


def test_plain_router_and_units():
    z = np.array([[2.0, 1.0, -1.0, 0.5], [0.0, 0.0, 0.0, 0.0]])
    chosen, weight = plain.route(z, np.eye(4), np.array([0.0, 0.0, 0.9, 0.0]), 2, 1.5)
    assert chosen.tolist() == [[2, 0], [2, 0]]               # the correction lifts expert 2; ties go to the lowest id
    s = plain.sigmoid(z)
    assert np.allclose(weight, 1.5 * np.array([[s[0, 2], s[0, 0]], [0.5, 0.5]]))       # and does not enter the weights
    one = np.ones((1, 1))
    tanh_form = 0.5 * 0.7 * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (0.7 + 0.044715 * 0.343)))
    assert np.isclose(plain.gelu_gated_unit(one, np.array([[0.7]]), np.array([[2.0]]), one)[0, 0], 2.0 * tanh_form)
    assert np.isclose(plain.silu_gated_unit(one, np.array([[0.7]]), np.array([[2.0]]), one)[0, 0], 1.4 / (1.0 + np.exp(-0.7)))
    unit = {"e0.gate": one, "e0.up": one, "e0.down": one, "shared.gate": one, "shared.up": one, "shared.down": 3.0 * one,
            "shared.sg": np.array([[-1.0]]), "router": np.array([[0.4]]), "correction": np.array([-5.0])}
    base = 1.0 / (1.0 + np.exp(-1.0))
    want = 2.0 * plain.sigmoid(np.array(0.4)) * base + plain.sigmoid(np.array(-1.0)) * 3.0 * base
    assert np.isclose(plain.mixture(one, unit, {"top": 1, "scale": 2.0})[0, 0], want)


def test_plain_loop_is_the_layers_one_after_the_other():
    weights = plain.random_weights(CONFIG_X, 2)
    tokens = random_tokens(300, 30, seed=3)
    unrolled = copy.deepcopy(CONFIG_X)
    del unrolled["loop"]
    order = [0, 1, 2, 1, 2, 1, 2, 3]
    unrolled["layers"] = [CONFIG_X["layers"][i] for i in order]
    copied = {name: value for name, value in weights.items() if not name.startswith("l")}
    for place, source in enumerate(order):
        copied.update({f"l{place}." + name[len(f"l{source}."):]: value for name, value in weights.items() if name.startswith(f"l{source}.")})
    assert np.allclose(plain.forward(CONFIG_X, weights, tokens), plain.forward(unrolled, copied, tokens), atol=1e-12)


def test_plain_model_is_causal_and_every_part_counts():
    for config in (CONFIG_X, CONFIG_Y, CONFIG_Z):
        weights = plain.random_weights(config, 5)
        tokens = random_tokens(config["vocab"], 60, seed=6)
        full = plain.forward(config, weights, tokens)
        assert np.isfinite(full).all()
        assert np.allclose(plain.forward(config, weights, tokens[:40]), full[:40], rtol=1e-9, atol=1e-9)
        model = plain.PlainFevolorn(config, weights)
        states = model.start()
        pieces = [model.forward(tokens[at:at + n], states) for at, n in ((0, 23), (23, 1), (24, 2), (26, 34))]
        assert np.allclose(np.concatenate(pieces), full, rtol=1e-9, atol=1e-9)
        short = tokens[:20]
        base = plain.forward(config, weights, short)
        for name in weights:
            changed = dict(weights)
            # (an expert that no token of the sequence chooses changes nothing, so the experts are changed together; a correction
            # that lifts every expert alike changes no choice, so its entries are moved on; where all experts are chosen it is idle)
            parts = name.split(".")
            if len(parts) == 4 and parts[1] == "mlp" and parts[2].startswith("e"):
                for other in weights:
                    if other.startswith(f"{parts[0]}.mlp.e") and other.endswith("." + parts[3]):
                        changed[other] = weights[other] * 1.3 + 0.05
            elif name.endswith(".correction"):
                router = config["layers"][int(parts[0][1:])]["mlp"]["router"]
                if router["top"] == router["experts"]:
                    continue
                changed[name] = np.roll(weights[name], 1) * 3.0
            elif name.endswith("left.q") or name.endswith("left.k") or name.endswith("q.norm") or name.endswith("k.norm"):
                if (config["layers"][int(parts[0][1:])]["mixer"]["left"].get("mask") or {}).get("size") == 1:
                    continue                                 # one visible key has the weight 1 whatever its score
                changed[name] = weights[name] * 1.3 + 0.05
            else:
                changed[name] = weights[name] * 1.3 + 0.05
            assert not np.allclose(plain.forward(config, changed, short), base, rtol=1e-7, atol=1e-7), f"{name} changes nothing"
