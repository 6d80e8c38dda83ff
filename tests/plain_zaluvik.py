"""A plain, slow Zaluvik in float64 numpy, one function per mechanism, written from the design's
equations. It shares no code with the package: the tests hold the engine against it.

Notation: T tokens, D model width; a weight W is stored [out, in] and applied as x @ W.T. Every mixer
takes a whole sequence (position 0 first) and can also be walked in pieces: a piece gets the ``state``
that the piece before it returned (None at the start of a sequence).

The design: x = scale * embed[token] =: x0; a run of neighbouring layers is passed several times with the
same weights, and x <- W_in [x; x0] ahead of every pass; a layer does x += m N1b(mixer(N1(x))), then
x += m N2b(ff(N2(x))), N a layer norm with weight and bias and m one factor for the whole model. Mixers:
``attention`` (grouped heads without positions, unit queries and keys, a sliding window, weights that are
sigmoids of biased scores and no distribution over the keys, heads that mix their weights, an output
gate per channel) and ``latent_attention`` (softmax attention in a sliding window whose keys and values are maps
of one cached latent per token, plus a rotated key part shared by all heads, an output gate per head). The
feed-forward is a gelu unit or a mixture of gated units chosen per token among the best groups of experts,
with one unit that every token runs. The head is the embedding table behind a final norm.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import numpy as np


# ----- small pieces -------------------------------------------------------------------------
def rms(x: np.ndarray, eps: float) -> np.ndarray:
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def layer_norm(x: np.ndarray, weight: np.ndarray, bias: np.ndarray, eps: float) -> np.ndarray:
    d = x - np.mean(x, axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * weight + bias


def sigmoid(x: np.ndarray) -> np.ndarray:
    return 0.5 * (1.0 + np.tanh(0.5 * x))


def silu(x: np.ndarray) -> np.ndarray:
    return x * sigmoid(x)


def gelu_erf(x: np.ndarray) -> np.ndarray:
    return 0.5 * x * (1.0 + np.vectorize(math.erf, otypes=[np.float64])(x / math.sqrt(2.0)))


def visible(position: int, window: Optional[int]) -> int:
    """The first key that the row at ``position`` sees: itself and the window - 1 before it."""
    return 0 if window is None else max(0, position - window + 1)


# ----- attention with sigmoid weights that the heads mix -----------------------------------------------
def sigmoid_attention(h: np.ndarray, w: Dict[str, np.ndarray], sizes: Dict, eps: float, state=None):
    """sizes: heads, kv_heads, dim, vdim, scale, window. The state is (unit keys so far, values so far)."""
    H, G, d, dv = sizes["heads"], sizes["kv_heads"], sizes["dim"], sizes["vdim"]
    past_k, past_v = state if state is not None else (np.zeros((0, G, d)), np.zeros((0, G, dv)))
    T, start = h.shape[0], past_k.shape[0]
    q = rms((h @ w["q"].T).reshape(T, H, d), eps)
    keys = np.concatenate([past_k, rms((h @ w["k"].T).reshape(T, G, d), eps)], axis=0)
    values = np.concatenate([past_v, (h @ w["v"].T).reshape(T, G, dv)], axis=0)
    out = mixed_heads(q, keys, values, start, sizes["scale"], w["pb"], w["talk"], sizes["window"])
    gate = sigmoid(h @ w["g"].T)
    return (out.reshape(T, H * dv) * gate) @ w["o"].T, (keys, values)


def mixed_heads(q: np.ndarray, keys: np.ndarray, values: np.ndarray, start: int, scale: float, bias: np.ndarray,
                mix: np.ndarray, window: Optional[int]) -> np.ndarray:
    """q [T, H, d] are the rows at positions start .. start + T - 1 of a sequence whose keys [N, G, d] and values
    [N, G, dv] are given from position 0 on. a_g(i, j) = sigmoid(q_g . k * scale + bias_g) for the visible keys;
    head h weighs the values of key head h // (H / G) with sum_g mix[h, g] a_g(i, j). Returns [T, H, dv]."""
    T, H, _ = q.shape
    per = H // keys.shape[1]
    out = np.zeros((T, H, values.shape[2]))
    for t in range(T):
        p = start + t
        first = visible(p, window)
        a = np.stack([sigmoid((keys[first:p + 1, g // per] @ q[t, g]) * scale + bias[g]) for g in range(H)])
        mixed = mix @ a
        for head in range(H):
            out[t, head] = mixed[head] @ values[first:p + 1, head // per]
    return out


# ----- attention over a latent --------------------------------------------------------------------
def rotate_halves(x: np.ndarray, positions: np.ndarray, dims: int, base: float) -> np.ndarray:
    """x [T, ..., dim]: channels (i, i + dims / 2), i < dims / 2, turn by position * base^(-2i / dims); the
    channels from ``dims`` on pass."""
    out = x.copy()
    half = dims // 2
    if half == 0:
        return out
    freq = base ** (-2.0 * np.arange(half) / dims)
    angle = positions.astype(np.float64)[:, None] * freq[None, :]
    shape = (x.shape[0],) + (1,) * (x.ndim - 2) + (half,)
    c, s = np.cos(angle).reshape(shape), np.sin(angle).reshape(shape)
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def latent_attention(h: np.ndarray, w: Dict[str, np.ndarray], sizes: Dict, eps: float, state=None):
    """sizes: heads, dim, rot_dim, vdim, kv_rank, scale, rot_base, rot_dims, window. The state is (latents so far,
    rotated key parts so far): nothing else of a token is kept."""
    H, d, dr, dv, rk = sizes["heads"], sizes["dim"], sizes["rot_dim"], sizes["vdim"], sizes["kv_rank"]
    turn, base = sizes["rot_dims"], sizes["rot_base"]
    past_c, past_kr = state if state is not None else (np.zeros((0, rk)), np.zeros((0, dr)))
    T, start = h.shape[0], past_c.shape[0]
    positions = np.arange(start, start + T)
    q = (h @ w["q"].T).reshape(T, H, d + dr)
    q_plain, q_rot = q[..., :d], rotate_halves(q[..., d:], positions, turn, base)
    down = h @ w["dkv"].T
    c = np.concatenate([past_c, rms(down[:, :rk], eps) * w["dkv.norm"]], axis=0)
    kr = np.concatenate([past_kr, rotate_halves(down[:, rk:], positions, turn, base)], axis=0)
    k_plain = (c @ w["uk"].T).reshape(-1, H, d)
    v = (c @ w["uv"].T).reshape(-1, H, dv)
    gate = sigmoid(h @ w["g"].T)
    out = np.zeros((T, H, dv))
    for t in range(T):
        p = start + t
        first = visible(p, sizes["window"])
        for head in range(H):
            s = (k_plain[first:p + 1, head] @ q_plain[t, head] + kr[first:p + 1] @ q_rot[t, head]) * sizes["scale"]
            e = np.exp(s - s.max())
            out[t, head] = (e / e.sum()) @ v[first:p + 1, head] * gate[t, head]
    return out.reshape(T, H * dv) @ w["o"].T, (c, kr)


# ----- the feed-forward -------------------------------------------------------------------------
def gelu_unit(h: np.ndarray, up: np.ndarray, down: np.ndarray) -> np.ndarray:
    return gelu_erf(h @ up.T) @ down.T


def gated_unit(h: np.ndarray, gate: np.ndarray, up: np.ndarray, down: np.ndarray) -> np.ndarray:
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(h: np.ndarray, router: np.ndarray, top: int, groups: int, keep: int) -> Tuple[np.ndarray, np.ndarray]:
    """(chosen [T, top], weight [T, top]): every expert scores sigmoid(z); a group of neighbours scores the sum of its
    two best; experts outside the ``keep`` best groups cannot be chosen; the chosen scores are divided by their sum."""
    s = sigmoid(h @ router.T)
    T, E = s.shape
    size = E // groups
    chosen, weight = np.zeros((T, top), dtype=np.int64), np.zeros((T, top))
    for t in range(T):
        best = np.array([np.sort(s[t, g * size:(g + 1) * size])[-2:].sum() for g in range(groups)])
        allowed = np.full(E, -np.inf)
        for g in np.argsort(-best, kind="stable")[:keep]:
            allowed[g * size:(g + 1) * size] = s[t, g * size:(g + 1) * size]
        chosen[t] = np.argsort(-allowed, kind="stable")[:top]
        weight[t] = s[t, chosen[t]] / (s[t, chosen[t]].sum() + 1e-20)
    return chosen, weight


def mixture(h: np.ndarray, w: Dict[str, np.ndarray], sizes: Dict) -> np.ndarray:
    """sizes: experts, top, groups, keep."""
    chosen, weight = route(h, w["router"], sizes["top"], sizes["groups"], sizes["keep"])
    out = np.zeros((h.shape[0], w["e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, a in zip(chosen[t], weight[t]):
            out[t] += a * gated_unit(h[t:t + 1], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])[0]
    if "shared.gate" in w:
        out += gated_unit(h, w["shared.gate"], w["shared.up"], w["shared.down"])
    return out


# ----- the model ------------------------------------------------------------------------------
def layer_runs(config: Dict) -> List[Tuple[int, bool]]:
    """[(layer, whether a pass begins right ahead of it)] in the order in which the layers run."""
    count, loop = len(config["layers"]), config.get("loop")
    if loop is None:
        return [(i, False) for i in range(count)]
    start, stop = loop["start"], loop["stop"]
    passes = [(i, i == start) for _ in range(loop["times"]) for i in range(start, stop)]
    return [(i, False) for i in range(start)] + passes + [(i, False) for i in range(stop, count)]


def _under(tensors: Dict[str, np.ndarray], prefix: str) -> Dict[str, np.ndarray]:
    return {name[len(prefix):]: value for name, value in tensors.items() if name.startswith(prefix)}


def _mixer_sizes(entry: Dict) -> Dict:
    m = entry["mixer"]
    sizes = {"heads": m["heads"], "dim": m["dim"], "vdim": m["vdim"], "scale": m["scale"], "window": (m.get("mask") or {}).get("size")}
    if entry["type"] == "latent_attention":
        sizes.update(rot_dim=m["rot_dim"], kv_rank=m["kv_rank"], rot_base=m["rot"]["base"], rot_dims=m["rot"]["dims"])
    else:
        sizes["kv_heads"] = m["kv_heads"]
    return sizes


def _ff_sizes(mlp: Dict) -> Dict:
    router = mlp["router"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    return {"experts": router["experts"], "top": router["top"], "groups": groups["count"], "keep": groups["keep"]}


class PlainZaluvik:
    """``config``: the model's configuration as a dict; ``tensors``: name -> float64 array."""

    def __init__(self, config: Dict, tensors: Dict[str, np.ndarray]):
        self.config, self.tensors = config, {k: np.asarray(v, dtype=np.float64) for k, v in tensors.items()}
        self.eps, self.mult = float(config["norm"]["eps"]), float(config["residual_mult"])
        self.runs = layer_runs(config)

    def start(self) -> List:
        """One state for every run of a layer: the passes of a layer share weights, not keys."""
        return [None] * len(self.runs)

    def _norm(self, x: np.ndarray, name: str) -> np.ndarray:
        return layer_norm(x, self.tensors[name], self.tensors[name + ".b"], self.eps)

    def forward(self, tokens, states: Optional[List] = None, keep_layers: bool = False):
        """Logits [T, vocab] of the next ``tokens`` of one sequence; ``states`` (from ``start`` or an earlier
        call) is brought up to date in place."""
        if states is None:
            states = self.start()
        x0 = self.tensors["embed"][np.asarray(tokens, dtype=np.int64)] * self.config["embedding"]["scale"]
        x = x0
        after = []
        for run, (index, begins_pass) in enumerate(self.runs):
            if begins_pass:
                x = np.concatenate([x, x0], axis=-1) @ self.tensors["loop.in"].T
            entry, base = self.config["layers"][index], f"l{index}."
            mix = _under(self.tensors, base + "mix.")
            mixer = latent_attention if entry["type"] == "latent_attention" else sigmoid_attention
            y, states[run] = mixer(self._norm(x, base + "norm1"), mix, _mixer_sizes(entry), self.eps, states[run])
            x = x + self.mult * self._norm(y, base + "norm1b")
            if entry.get("mlp") is not None:
                ff, h = _under(self.tensors, base + "mlp."), self._norm(x, base + "norm2")
                y = gelu_unit(h, ff["up"], ff["down"]) if entry["mlp"]["kind"] == "dense" else mixture(h, ff, _ff_sizes(entry["mlp"]))
                x = x + self.mult * self._norm(y, base + "norm2b")
            after.append(x.copy())
        logits = self._norm(x, "final.norm") @ self.tensors["embed"].T
        return (logits, after) if keep_layers else logits


def forward(config: Dict, weights: Dict[str, np.ndarray], tokens) -> np.ndarray:
    """Logits [T, vocab] of a whole sequence."""
    return PlainZaluvik(config, weights).forward(list(tokens))


def greedy(config: Dict, weights: Dict[str, np.ndarray], prompt: List[int], new: int) -> List[int]:
    """The prompt once, then token by token on the carried states."""
    model = PlainZaluvik(config, weights)
    states = model.start()
    logits = model.forward(list(prompt), states)
    out = []
    for _ in range(new):
        out.append(int(np.argmax(logits[-1])))
        logits = model.forward([out[-1]], states)
    return out


# ----- tensors of a model --------------------------------------------------------------------------------
def tensor_shapes(config: Dict) -> Dict[str, Tuple[int, ...]]:
    D, V = config["width"], config["vocab"]
    shapes: Dict[str, Tuple[int, ...]] = {"embed": (V, D), "final.norm": (D,), "final.norm.b": (D,)}
    if config.get("loop") is not None:
        shapes["loop.in"] = (D, 2 * D)
    for index, layer in enumerate(config["layers"]):
        base, m, mlp = f"l{index}.", layer["mixer"], layer.get("mlp")
        for norm in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp is not None else ()):
            shapes[base + norm] = shapes[base + norm + ".b"] = (D,)
        mix = base + "mix."
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        if layer["type"] == "latent_attention":
            dr, rk = m["rot_dim"], m["kv_rank"]
            shapes.update({mix + "q": (H * (d + dr), D), mix + "dkv": (rk + dr, D), mix + "dkv.norm": (rk,), mix + "uk": (H * d, rk),
                           mix + "uv": (H * dv, rk), mix + "g": (H, D), mix + "o": (D, H * dv)})
        else:
            G = m["kv_heads"]
            shapes.update({mix + "q": (H * d, D), mix + "k": (G * d, D), mix + "v": (G * dv, D), mix + "talk": (H, H), mix + "pb": (H,),
                           mix + "g": (H * dv, D), mix + "o": (D, H * dv)})
        if mlp is None:
            continue
        ff = base + "mlp."
        if mlp["kind"] == "dense":
            shapes.update({ff + "up": (mlp["ff"], D), ff + "down": (D, mlp["ff"])})
            continue
        shapes[ff + "router"] = (mlp["router"]["experts"], D)
        units = [(f"e{e}.", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
        if mlp.get("shared"):
            units.append(("shared.", mlp["shared"]["ff"]))
        for unit, width in units:
            shapes.update({ff + unit + "gate": (width, D), ff + unit + "up": (width, D), ff + unit + "down": (D, width)})
    return shapes


def random_weights(config: Dict, seed: int, experts_alike: float = 0.9) -> Dict[str, np.ndarray]:
    """Weights that make every part count: matrices keep the size of what passes through them (the router's, the
    gates' and the experts' somewhat more), head mixes near no pattern of their own, score biases around -1 so that most
    keys weigh little and a few a lot, biases of visible size. The experts of a layer share ``experts_alike`` of their
    weights: where bfloat16 rounding turns a close call of the router the output then moves by a part of an expert, not
    by all of it, while in float32 any wrong choice still shows far above the comparison's limit."""
    rng = np.random.default_rng(seed)
    weights: Dict[str, np.ndarray] = {}
    common: Dict[Tuple[str, str], np.ndarray] = {}
    for name, shape in tensor_shapes(config).items():
        parts = name.split(".")
        leaf = parts[-1]
        if len(parts) == 4 and parts[1] == "mlp" and parts[2].startswith("e") and experts_alike:
            size = 1.0 if leaf == "down" else 1.5
            if (parts[0], leaf) not in common:
                common[parts[0], leaf] = rng.normal(0.0, size, shape) / math.sqrt(shape[-1])
            own = rng.normal(0.0, size, shape) / math.sqrt(shape[-1])
            weights[name] = experts_alike * common[parts[0], leaf] + (1.0 - experts_alike) * own
            continue
        if leaf.startswith("norm"):
            value = rng.uniform(0.6, 1.4, shape)
        elif leaf == "b":
            value = rng.normal(0.0, 0.3, shape)
        elif leaf == "pb":
            value = rng.normal(-1.0, 0.7, shape)
        elif leaf == "talk":
            value = rng.normal(0.0, 1.0, shape)
        elif name == "embed":
            value = rng.normal(0.0, 1.0, shape)
        elif leaf in ("router", "gate", "up", "g"):
            value = rng.normal(0.0, 1.5, shape) / math.sqrt(shape[-1])
        else:
            value = rng.normal(0.0, 1.0, shape) / math.sqrt(shape[-1])
        weights[name] = value
    return weights
