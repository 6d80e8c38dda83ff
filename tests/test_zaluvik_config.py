"""Zaluvik on the CPU: its configuration and tensor names, the schedule of a looped run of layers, the cache entries it
asks for, and the plain model held against itself (a sequence in one piece against pieces with carried state, the
windows' edges, weights that are no distribution, the heads' mix, the router's groups, the loop)."""

import copy

import numpy as np
import pytest

import plain_zaluvik as plain
from zaluvik_common import CONFIG_X, CONFIG_Y, CONFIG_Z, make_folder, random_tokens


def test_config_lowers_to_parts_and_names(tmp_path):
    from flyweight_amd.config import ConfigError, ZaluvikConfig, load_config
    from flyweight_amd.engine.model import declared_tensors
    for name, raw in (("X", CONFIG_X), ("Y", CONFIG_Y), ("Z", CONFIG_Z)):
        folder = str(tmp_path / name)
        make_folder(folder, raw)
        config = load_config(folder)                         # the model class by config.json
        assert isinstance(config, ZaluvikConfig)
        spec = config.model_spec()
        assert {n: tuple(d.shape) for n, d in declared_tensors(spec).items()} == plain.tensor_shapes(raw)
        assert [layer.mixer.kind for layer in config.layers] == [entry["type"] for entry in raw["layers"]]
        assert spec.lm_head_name is None and spec.embedding_name == "embed"
        assert all(layer.arrangement == "sandwich_norm_residual" and layer.params["residual_mult"] == raw["residual_mult"] for layer in spec.layers)
        assert ZaluvikConfig.from_dict(config.to_dict()) == config and config.to_dict() == raw
        assert spec.embedding_scale == raw["embedding"]["scale"]
    first, second, third, _ = ZaluvikConfig.from_dict(CONFIG_X).model_spec().layers
    assert first.mixer.kind == "sigmoid_attention" and (first.mixer["num_heads"], first.mixer["num_kv_heads"]) == (6, 3)
    assert (first.mixer["head_dim"], first.mixer["v_head_dim"], first.mixer["window"], first.mixer["softmax_scale"]) == (32, 48, 50, 0.5)
    assert second.mixer.kind == "latent_attention" and second.mixer["q_rank"] is None and second.mixer["output_gate"] == "per_head"
    assert (second.mixer["window"], second.mixer["kv_rank"], second.mixer["rot_dim"]) == (90, 48, 16)
    assert second.mixer["position"].kind == "rotary_neox" and second.mixer["position"]["rotary_dim"] == 16
    assert first.ffn.kind == "gelu_mlp" and first.ffn["intermediate_size"] == 120
    assert second.ffn.kind == "moe_swiglu" and (second.ffn["num_experts"], second.ffn["top"], second.ffn["router_groups"]) == (9, 3, (3, 2))
    assert (second.ffn["router_scores"], second.ffn["group_score"], second.ffn["shared_intermediate_size"]) == ("sigmoid", "pair", 56)
    assert third.ffn["shared_intermediate_size"] is None and not second.ffn["router_bias"]
    assert first.mixer_norm["tensor"] == "l0.norm1" and first.params["mixer_post_norm"]["tensor"] == "l0.norm1b"
    assert second.ffn_norm["tensor"] == "l1.norm2" and second.params["ffn_post_norm"]["tensor"] == "l1.norm2b" and second.ffn_norm["bias"]
    assert ZaluvikConfig.from_dict(CONFIG_Y).model_spec().layers[2].ffn is None
    spec_z = ZaluvikConfig.from_dict(CONFIG_Z).model_spec()
    assert spec_z.input_join is None and spec_z.layers[2].mixer["window"] is None
    for path, value, match in ((("layers", 0, "type"), "serial", "type"), (("layers", 0, "mixer", "heads"), 5, "multiple"),
                               (("layers", 1, "mixer", "rot", "dims"), 18, "rot"), (("norm", "eps"), 0, "eps"),
                               (("layers", 0, "mlp", "kind"), "glu", "kind"), (("layers", 1, "mlp", "router", "top"), 7, "groups"),
                               (("layers", 1, "mlp", "router", "groups", "count"), 5, "groups"), (("layers", 0, "mixer", "mask", "size"), 0, "size"),
                               (("loop", "stop"), 5, "loop"), (("loop", "start"), 3, "loop"), (("loop", "times"), 0, "times"),
                               (("layers", 0, "mlp", "ff"), None, "ff"), (("vocab",), None, "vocab")):
        broken = copy.deepcopy(CONFIG_X)
        at = broken
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        with pytest.raises(ConfigError, match=match):
            ZaluvikConfig.from_dict(broken)


def test_the_schedule_of_a_loop():
    """Every pass runs the looped layers with their weights and cache entries of its own; the input joins ahead of the
    first layer of every pass and nowhere else."""
    from flyweight_amd.config import ConfigError, LayerSpec, ModelSpec, PartSpec, ScheduleEntry, ZaluvikConfig
    spec = ZaluvikConfig.from_dict(CONFIG_X).model_spec()
    assert len(spec.layers) == 4 and spec.input_join["tensor"] == "loop.in"
    assert [(e.layer, e.cache, e.joins_input) for e in spec.schedule] == [
        (0, 0, False), (1, 1, True), (2, 2, False), (1, 3, True), (2, 4, False), (1, 5, True), (2, 6, False), (3, 7, False)]
    assert all(e.writes_cache for e in spec.schedule)
    spec = ZaluvikConfig.from_dict(CONFIG_Y).model_spec()
    assert [(e.layer, e.joins_input) for e in spec.schedule] == [(0, True), (0, True), (1, False), (2, False)]
    once = copy.deepcopy(CONFIG_X)
    once["loop"]["times"] = 1
    assert [(e.layer, e.joins_input) for e in ZaluvikConfig.from_dict(once).model_spec().schedule] == [(0, False), (1, True), (2, False), (3, False)]
    assert plain.layer_runs(CONFIG_X) == [(e.layer, e.joins_input) for e in ZaluvikConfig.from_dict(CONFIG_X).model_spec().schedule]
    # a schedule may not join an input that the model has no map for
    norm = PartSpec("layernorm", {"eps": 1e-5, "size": 8, "tensor": "n"})
    block = LayerSpec("sandwich_norm_residual", norm, PartSpec("sigmoid_attention"), None, None)
    with pytest.raises(ConfigError, match="joins"):
        ModelSpec("a", 8, 8, 8, (block,), (ScheduleEntry(0, 0, joins_input=True),), norm, "embed", None).validate()


def test_cache_entries():
    """An attention layer asks for pages of its key heads within its window, a latent layer for pages of one head whose
    keys hold the latent and the rotated part, its values the latent alone, within its window; every run has its own."""
    from flyweight_amd.cache import CacheManager
    from flyweight_amd.config import ZaluvikConfig
    from flyweight_amd.engine.model import CausalLM
    needs = CausalLM(ZaluvikConfig.from_dict(CONFIG_X).model_spec()).cache_needs()
    assert set(needs) == set(range(8))
    assert needs[1] == needs[3] == needs[5] and needs[2] == needs[4] == needs[6] and needs[0] == needs[7]
    assert (needs[0].num_kv_heads, needs[0].head_dim, needs[0].v_head_dim, needs[0].window) == (3, 32, 48, 50)
    assert (needs[1].num_kv_heads, needs[1].head_dim, needs[1].v_head_dim, needs[1].window) == (1, 48 + 16, 48, 90)
    assert (needs[2].num_kv_heads, needs[2].head_dim, needs[2].v_head_dim, needs[2].window) == (1, 48, 16, 130)
    needs_z = CausalLM(ZaluvikConfig.from_dict(CONFIG_Z).model_spec()).cache_needs()
    assert needs_z[0].window == 1 and needs_z[2].window is None and needs_z[2].v_head_dim is None
    cache = CacheManager(needs, num_pages=6, max_requests=2)
    assert len(cache.groups) == 3                            # equal needs share a pool and a block table
    cache.admit("a")
    for length in (50, 130, 131, 200, 330):
        cache.reserve("a", length)
        cache.commit("a", length)
        cache.check_invariants()
    held = {group.need.window: [page != -1 for page in group.tables["a"]] for group in cache.groups}
    # the next token sees itself and the window - 1 keys before it: earlier pages have gone back
    assert held[50] == [False, False, False, False, True, True] and held[90] == [False, False, False, True, True, True]
    assert held[130] == [False, False, False, True, True, True]
    cache.release("a")
    assert all(group.pool.free_count == 6 for group in cache.groups)


def _mix(config, index):
    entry = config["layers"][index]
    return entry, {name[len(f"l{index}.mix."):]: value for name, value in plain.random_weights(config, 3).items() if name.startswith(f"l{index}.mix.")}


def test_plain_mixers_in_one_piece_and_in_pieces():
    """Each mixer over 90 tokens at once equals the same tokens in pieces of 1, 2, 7 and 40 on the carried state."""
    rng = np.random.default_rng(0)
    for config, index in ((CONFIG_X, 0), (CONFIG_X, 1), (CONFIG_Y, 0), (CONFIG_Y, 1), (CONFIG_Z, 0), (CONFIG_Z, 3)):
        entry, w = _mix(config, index)
        h = rng.normal(size=(90, config["width"]))
        mixer = plain.latent_attention if entry["type"] == "latent_attention" else plain.sigmoid_attention
        whole, _ = mixer(h, w, plain._mixer_sizes(entry), config["norm"]["eps"], None)
        for piece in (1, 2, 7, 40):
            state, parts = None, []
            for at in range(0, 90, piece):
                out, state = mixer(h[at:at + piece], w, plain._mixer_sizes(entry), config["norm"]["eps"], state)
                parts.append(out)
            assert np.allclose(np.concatenate(parts), whole, rtol=1e-10, atol=1e-10), (entry["type"], piece)


def test_plain_weights_are_sigmoids_that_the_heads_mix():
    """A key just inside the window counts and the one just outside does not; equal keys add up (nothing divides by
    their number); a head that mixes another's weights alone carries that head's pattern to its own values."""
    d, T = 8, 12
    rng = np.random.default_rng(1)
    q = np.zeros((T, 2, d))
    q[:, 0, 0] = q[:, 1, 1] = 1.0
    keys = np.zeros((T, 2, d))
    values = rng.normal(size=(T, 2, 3))
    keys[5, 0, 0] = 100.0                       # head 0 finds key 5, head 1 finds key 7
    keys[7, 1, 1] = 100.0
    bias = np.full(2, -40.0)
    own = plain.mixed_heads(q, keys, values, 0, 1.0, bias, np.eye(2), 4)
    for t in range(T):
        assert np.allclose(own[t, 0], values[5, 0] if 5 <= t < 9 else 0.0, atol=1e-12)
        assert np.allclose(own[t, 1], values[7, 1] if 7 <= t < 11 else 0.0, atol=1e-12)
    swapped = plain.mixed_heads(q, keys, values, 0, 1.0, bias, np.array([[0.0, 1.0], [-2.0, 0.5]]), 4)
    assert np.allclose(swapped[8, 0], values[7, 0], atol=1e-12)                       # head 1's key, head 0's values
    assert np.allclose(swapped[8, 1], -2.0 * values[5, 1] + 0.5 * values[7, 1], atol=1e-12)
    level = plain.mixed_heads(q, np.zeros((T, 2, d)), np.ones((T, 2, 3)), 0, 1.0, np.zeros(2), np.eye(2), None)
    assert np.allclose(level[:, 0, 0], 0.5 * np.arange(1, T + 1))                     # sigmoid(0) for every key, summed


def test_plain_rotation_turns_halves_and_leaves_the_rest():
    x = np.arange(6.0)[None, :]
    out = plain.rotate_halves(x, np.array([3]), 4, 100.0)
    for i, f in ((0, 1.0), (1, 100.0 ** -0.5)):
        c, s = np.cos(3 * f), np.sin(3 * f)
        assert np.isclose(out[0, i], x[0, i] * c - x[0, i + 2] * s) and np.isclose(out[0, i + 2], x[0, i + 2] * c + x[0, i] * s)
    assert out[0, 4:].tolist() == [4.0, 5.0]


def test_plain_router_and_units():
    h = np.eye(8)[:3]
    z = np.zeros((3, 8))
    z[0] = [3.0, -3.0, -3.0, -3.0, 1.5, 1.4, 1.3, -5.0]     # the best expert is 0, the best pair is in the second group
    z[1] = [2.0, 1.9, -1.0, -1.0, 4.0, -4.0, -4.0, -4.0]    # the best expert is 4, the best pair in the first group
    chosen, weight = plain.route(z, np.eye(8), top=2, groups=2, keep=1)
    assert chosen.tolist() == [[4, 5], [0, 1], [0, 1]]        # (all equal: the lowest group, the lowest ids)
    free, _ = plain.route(z, np.eye(8), top=2, groups=2, keep=2)
    assert free.tolist() == [[0, 4], [4, 0], [0, 1]]
    s = plain.sigmoid(np.array([1.5, 1.4]))
    assert np.allclose(weight[0], s / s.sum()) and np.allclose(weight.sum(axis=1), 1.0)
    assert plain.route(z, np.eye(8), top=1, groups=8, keep=1)[0][:, 0].tolist() == [0, 4, 0]     # groups of one: its one score
    one = np.ones((1, 1))
    assert np.isclose(plain.gelu_unit(one, np.array([[0.7]]), one)[0, 0], 0.7 * 0.758036347776927)      # 0.7 Phi(0.7)
    assert np.isclose(plain.gated_unit(one, np.array([[0.7]]), np.array([[2.0]]), one)[0, 0], 1.4 / (1.0 + np.exp(-0.7)))
    assert h.shape == (3, 8)


def test_plain_loop_joins_the_input_ahead_of_every_pass():
    """W_in = [0 | 1]: every pass starts again from the embedding output, so the passes before the last leave nothing;
    W_in = [1 | 0]: the passes are the layers one after the other."""
    weights = plain.random_weights(CONFIG_X, 2)
    tokens = random_tokens(300, 30, seed=3)
    D = CONFIG_X["width"]
    again = dict(weights, **{"loop.in": np.concatenate([np.zeros((D, D)), np.eye(D)], axis=1)})
    once = copy.deepcopy(CONFIG_X)
    once["loop"]["times"] = 1
    assert np.allclose(plain.forward(CONFIG_X, again, tokens), plain.forward(once, again, tokens), atol=1e-12)
    through = dict(weights, **{"loop.in": np.concatenate([np.eye(D), np.zeros((D, D))], axis=1)})
    unrolled = copy.deepcopy(CONFIG_X)
    del unrolled["loop"]
    order = [0, 1, 2, 1, 2, 1, 2, 3]
    unrolled["layers"] = [CONFIG_X["layers"][i] for i in order]
    copied = {name: value for name, value in weights.items() if not name.startswith("l")}
    for place, source in enumerate(order):
        copied.update({f"l{place}." + name[len(f"l{source}."):]: value for name, value in weights.items() if name.startswith(f"l{source}.")})
    assert np.allclose(plain.forward(CONFIG_X, through, tokens), plain.forward(unrolled, copied, tokens), atol=1e-12)


def test_plain_model_is_causal_and_every_part_counts():
    for config in (CONFIG_X, CONFIG_Y, CONFIG_Z):
        weights = plain.random_weights(config, 5)
        tokens = random_tokens(config["vocab"], 60, seed=6)
        full = plain.forward(config, weights, tokens)
        assert np.isfinite(full).all()
        assert np.allclose(plain.forward(config, weights, tokens[:40]), full[:40], rtol=1e-9, atol=1e-9)
        model = plain.PlainZaluvik(config, weights)
        states = model.start()
        pieces = [model.forward(tokens[at:at + n], states) for at, n in ((0, 23), (23, 1), (24, 2), (26, 34))]
        assert np.allclose(np.concatenate(pieces), full, rtol=1e-9, atol=1e-9)
        short = tokens[:20]
        base = plain.forward(config, weights, short)
        for name in weights:
            changed = dict(weights)
            # (a router of which one expert is chosen gives the same choice and the weight 1 whatever its size: its rows are moved on instead;
            # an expert that no token of the sequence chooses changes nothing, so the experts are changed together)
            parts = name.split(".")
            if len(parts) == 4 and parts[1] == "mlp" and parts[2].startswith("e"):
                for other in weights:
                    if other.startswith(f"{parts[0]}.mlp.e") and other.endswith("." + parts[3]):
                        changed[other] = weights[other] * 1.3 + 0.05
            else:
                changed[name] = np.roll(weights[name], 1, axis=0) if name.endswith(".router") else weights[name] * 1.3 + 0.05
            assert not np.allclose(plain.forward(config, changed, short), base, rtol=1e-7, atol=1e-7), f"{name} changes nothing"
