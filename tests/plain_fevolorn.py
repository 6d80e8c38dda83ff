"""A plain, slow Fevolorn in float64 numpy, one function per mechanism, written from the design's
equations. It shares no code with the package: the tests hold the engine against it.

Notation: T tokens, D model width; a weight W is stored [out, in] and applied as x @ W.T. Every mixer
takes a whole sequence (position 0 first) and can also be walked in pieces: a piece gets the ``state``
that the piece before it returned (None at the start of a sequence).

The design: the residual stream is ``streams`` rows side by side, all of them scale * embed[token] at the
start. A sublayer reads one weighted sum of the streams through its norm; its output, scaled channel by
channel, goes to every stream with a weight of that stream's own while the streams mix among themselves. The
norm is tanh(alpha x) w + b. Mixers: ``lightning`` (a linear recurrence over a matrix state per head with
a fixed decay) and ``parallel`` (windowed softmax attention without positions beside a selective scan, each
output brought to unit root mean square, half their sum). The feed-forward is a gated unit around a gelu
or a mixture of gated units chosen by sigmoid scores that a correction shifts for the choice alone, beside a
gated unit that every token runs and gates. A run of neighbouring layers is passed several times. The head
is the embedding table behind a final norm of the streams' sum.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import numpy as np


# ----- small pieces -------------------------------------------------------------------------
def rms(x: np.ndarray, eps: float) -> np.ndarray:
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def tanh_norm(x: np.ndarray, alpha: float, weight: np.ndarray, bias: np.ndarray) -> np.ndarray:
    return np.tanh(alpha * x) * weight + bias


def sigmoid(x: np.ndarray) -> np.ndarray:
    return 0.5 * (1.0 + np.tanh(0.5 * x))


def silu(x: np.ndarray) -> np.ndarray:
    return x * sigmoid(x)


def softplus(x: np.ndarray) -> np.ndarray:
    return np.logaddexp(0.0, x)


def gelu_tanh(x: np.ndarray) -> np.ndarray:
    return 0.5 * x * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


# ----- the streams --------------------------------------------------------------------------
def read_streams(x: np.ndarray, weights: np.ndarray) -> np.ndarray:
    """x [T, S, D] -> what a sublayer's norm sees, [T, D]."""
    return np.einsum("s,tsd->td", weights, x)


def join_streams(x: np.ndarray, y: np.ndarray, mix: np.ndarray, out: np.ndarray) -> np.ndarray:
    """x_t <- sum_s mix[s, t] x_s + out[t] y, all streams from the old ones. y [T, D]."""
    return np.einsum("st,nsd->ntd", mix, x) + out[None, :, None] * y[:, None, :]


# ----- a linear recurrence with a fixed decay per head -----------------------------------------
def decay_recurrence(q: np.ndarray, k: np.ndarray, v: np.ndarray, decay: np.ndarray, state: np.ndarray):
    """q, k [T, H, d], v [T, H, dv], state [H, d, dv]: S <- decay S + k v^T, then o = S^T q. Returns (o [T, H, dv], S)."""
    S = state.copy()
    out = np.zeros(v.shape)
    for t in range(q.shape[0]):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hde,hd->he", S, q[t])
    return out, S


def lightning(h: np.ndarray, w: Dict[str, np.ndarray], sizes: Dict, eps: float, state=None):
    """sizes: heads, dim, vdim, decay. The state is S."""
    H, d, dv = sizes["heads"], sizes["dim"], sizes["vdim"]
    T = h.shape[0]
    q, k = silu(h @ w["q"].T).reshape(T, H, d), silu(h @ w["k"].T).reshape(T, H, d)
    v = silu(h @ w["v"].T).reshape(T, H, dv)
    o, S = decay_recurrence(q, k, v, np.asarray(sizes["decay"], dtype=np.float64), state if state is not None else np.zeros((H, d, dv)))
    return (rms(o.reshape(T, H * dv), eps) * w["norm"] * sigmoid(h @ w["g"].T)) @ w["o"].T, S


# ----- windowed attention without positions -----------------------------------------------------
def visible(position: int, window: Optional[int]) -> int:
    """The first key that the row at ``position`` sees: itself and the window - 1 before it."""
    return 0 if window is None else max(0, position - window + 1)


def windowed_attention(h: np.ndarray, w: Dict[str, np.ndarray], sizes: Dict, eps: float, state=None):
    """sizes: heads, kv_heads, dim, vdim, scale, window. The state is (normed keys so far, values so far)."""
    H, G, d, dv = sizes["heads"], sizes["kv_heads"], sizes["dim"], sizes["vdim"]
    past_k, past_v = state if state is not None else (np.zeros((0, G, d)), np.zeros((0, G, dv)))
    T, start = h.shape[0], past_k.shape[0]
    q = rms((h @ w["q"].T).reshape(T, H, d), eps) * w["q.norm"]
    keys = np.concatenate([past_k, rms((h @ w["k"].T).reshape(T, G, d), eps) * w["k.norm"]], axis=0)
    values = np.concatenate([past_v, (h @ w["v"].T).reshape(T, G, dv)], axis=0)
    out = np.zeros((T, H, dv))
    for t in range(T):
        p = start + t
        first = visible(p, sizes["window"])
        for head in range(H):
            g = head // (H // G)
            s = keys[first:p + 1, g] @ q[t, head] * sizes["scale"]
            e = np.exp(s - s.max())
            out[t, head] = (e / e.sum()) @ values[first:p + 1, g]
    return out.reshape(T, H * dv) @ w["o"].T, (keys, values)


# ----- a selective scan ----------------------------------------------------------------------
def causal_conv(x: np.ndarray, taps: np.ndarray, bias: np.ndarray, before: np.ndarray):
    """x [T, C], taps [C, L] (the last column the current token's), before [L - 1, C]: the inputs ahead of x's first
    row. Returns (the convolution [T, C], the last L - 1 inputs)."""
    L = taps.shape[1]
    padded = np.concatenate([before, x], axis=0)
    y = np.zeros_like(x) + bias
    for j in range(L):
        y = y + taps[:, j] * padded[j:j + x.shape[0]]
    return y, padded[padded.shape[0] - (L - 1):]


def selective_scan(x: np.ndarray, dt: np.ndarray, A: np.ndarray, B: np.ndarray, C: np.ndarray, D: np.ndarray, state: np.ndarray):
    """x, dt [T, channels], A, state [channels, N], B, C [T, N]: S <- exp(dt A) S + dt x B, y = S C + D x."""
    S = state.copy()
    y = np.zeros_like(x)
    for t in range(x.shape[0]):
        S = np.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y, S


def mamba(h: np.ndarray, w: Dict[str, np.ndarray], sizes: Dict, state=None):
    """sizes: inner, state, dt_rank, conv. The state is (S, the convolution's last inputs)."""
    inner, N, rank, L = sizes["inner"], sizes["state"], sizes["dt_rank"], sizes["conv"]
    S, before = state if state is not None else (np.zeros((inner, N)), np.zeros((L - 1, inner)))
    both = h @ w["in"].T
    x, z = both[:, :inner], both[:, inner:]
    x, before = causal_conv(x, w["conv"], w["conv.b"], before)
    x = silu(x)
    low = x @ w["x"].T
    dt = softplus(low[:, :rank] @ w["dt"].T + w["dt.b"])
    y, S = selective_scan(x, dt, -np.exp(w["A_log"]), low[:, rank:rank + N], low[:, rank + N:], w["D"], S)
    return (y * silu(z)) @ w["o"].T, (S, before)


def parallel(h: np.ndarray, w: Dict[str, np.ndarray], sizes: Dict, eps: float, state=None):
    """sizes: left (windowed_attention's), right (mamba's). The state is both branches'."""
    left_state, right_state = state if state is not None else (None, None)
    left, left_state = windowed_attention(h, _under(w, "left."), sizes["left"], eps, left_state)
    right, right_state = mamba(h, _under(w, "right."), sizes["right"], right_state)
    return 0.5 * (rms(left, eps) * w["left.out"] + rms(right, eps) * w["right.out"]), (left_state, right_state)


# ----- the feed-forward -------------------------------------------------------------------------
def gelu_gated_unit(h: np.ndarray, gate: np.ndarray, up: np.ndarray, down: np.ndarray) -> np.ndarray:
    return (gelu_tanh(h @ gate.T) * (h @ up.T)) @ down.T


def silu_gated_unit(h: np.ndarray, gate: np.ndarray, up: np.ndarray, down: np.ndarray) -> np.ndarray:
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(h: np.ndarray, router: np.ndarray, correction: np.ndarray, top: int, scale: float) -> Tuple[np.ndarray, np.ndarray]:
    """(chosen [T, top], weight [T, top]): scores sigmoid(z); chosen by score + correction, weighed by score * scale."""
    s = sigmoid(h @ router.T)
    chosen = np.argsort(-(s + correction), axis=-1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=-1) * scale


def mixture(h: np.ndarray, w: Dict[str, np.ndarray], sizes: Dict) -> np.ndarray:
    """sizes: top, scale."""
    chosen, weight = route(h, w["router"], w["correction"], sizes["top"], sizes["scale"])
    out = np.zeros((h.shape[0], w["e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, a in zip(chosen[t], weight[t]):
            out[t] += a * silu_gated_unit(h[t:t + 1], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])[0]
    if "shared.gate" in w:
        out += sigmoid(h @ w["shared.sg"].T) * silu_gated_unit(h, w["shared.gate"], w["shared.up"], w["shared.down"])
    return out


# ----- the model ------------------------------------------------------------------------------
def layer_runs(config: Dict) -> List[int]:
    """The layers in the order in which they run."""
    order, loop = list(range(len(config["layers"]))), config.get("loop")
    if loop is None:
        return order
    start, stop = loop["start"], loop["stop"]
    return order[:start] + order[start:stop] * loop["times"] + order[stop:]


def _under(tensors: Dict[str, np.ndarray], prefix: str) -> Dict[str, np.ndarray]:
    return {name[len(prefix):]: value for name, value in tensors.items() if name.startswith(prefix)}


def _mixer_sizes(entry: Dict) -> Dict:
    m = entry["mixer"]
    if entry["type"] == "lightning":
        return m
    left = dict(m["left"], window=(m["left"].get("mask") or {}).get("size"))
    return {"left": left, "right": m["right"]}


class PlainFevolorn:
    """``config``: the model's configuration as a dict; ``tensors``: name -> float64 array."""

    def __init__(self, config: Dict, tensors: Dict[str, np.ndarray]):
        self.config, self.tensors = config, {k: np.asarray(v, dtype=np.float64) for k, v in tensors.items()}
        self.eps = float(config["norm"]["eps"])
        self.runs = layer_runs(config)

    def start(self) -> List:
        """One state for every run of a layer: the passes of a layer share weights, not states."""
        return [None] * len(self.runs)

    def _norm(self, x: np.ndarray, name: str) -> np.ndarray:
        t = self.tensors
        return tanh_norm(x, t[name + ".alpha"], t[name], t[name + ".b"])

    def forward(self, tokens, states: Optional[List] = None, keep_layers: bool = False):
        """Logits [T, vocab] of the next ``tokens`` of one sequence; ``states`` (from ``start`` or an earlier
        call) is brought up to date in place. ``keep_layers``: also the sum of the streams after every layer run."""
        if states is None:
            states = self.start()
        t = self.tensors
        x0 = t["embed"][np.asarray(tokens, dtype=np.int64)] * self.config["embedding"]["scale"]
        x = np.repeat(x0[:, None, :], self.config["streams"], axis=1)
        after = []
        for run, index in enumerate(self.runs):
            entry, base = self.config["layers"][index], f"l{index}."
            mixer = lightning if entry["type"] == "lightning" else parallel
            h = self._norm(read_streams(x, t[base + "hc1.in"]), base + "norm1")
            y, states[run] = mixer(h, _under(t, base + "mix."), _mixer_sizes(entry), self.eps, states[run])
            x = join_streams(x, y * t[base + "ls1"], t[base + "hc1.mix"], t[base + "hc1.out"])
            if entry.get("mlp") is not None:
                ff = _under(t, base + "mlp.")
                h = self._norm(read_streams(x, t[base + "hc2.in"]), base + "norm2")
                if entry["mlp"]["kind"] == "dense":
                    y = gelu_gated_unit(h, ff["gate"], ff["up"], ff["down"])
                else:
                    y = mixture(h, ff, entry["mlp"]["router"])
                x = join_streams(x, y * t[base + "ls2"], t[base + "hc2.mix"], t[base + "hc2.out"])
            after.append(x.sum(axis=1))
        logits = self._norm(x.sum(axis=1), "final.norm") @ t["embed"].T
        return (logits, after) if keep_layers else logits


def forward(config: Dict, weights: Dict[str, np.ndarray], tokens) -> np.ndarray:
    """Logits [T, vocab] of a whole sequence."""
    return PlainFevolorn(config, weights).forward(list(tokens))


def greedy(config: Dict, weights: Dict[str, np.ndarray], prompt: List[int], new: int) -> List[int]:
    """The prompt once, then token by token on the carried states."""
    model = PlainFevolorn(config, weights)
    states = model.start()
    logits = model.forward(list(prompt), states)
    out = []
    for _ in range(new):
        out.append(int(np.argmax(logits[-1])))
        logits = model.forward([out[-1]], states)
    return out


# ----- tensors of a model --------------------------------------------------------------------------------
def tensor_shapes(config: Dict) -> Dict[str, Tuple[int, ...]]:
    D, V, S = config["width"], config["vocab"], config["streams"]
    shapes: Dict[str, Tuple[int, ...]] = {"embed": (V, D), "final.norm": (D,), "final.norm.b": (D,), "final.norm.alpha": ()}
    for index, layer in enumerate(config["layers"]):
        base, m, mlp = f"l{index}.", layer["mixer"], layer.get("mlp")
        for q in (1, 2) if mlp is not None else (1,):
            shapes.update({f"{base}norm{q}": (D,), f"{base}norm{q}.b": (D,), f"{base}norm{q}.alpha": (), f"{base}ls{q}": (D,),
                           f"{base}hc{q}.in": (S,), f"{base}hc{q}.out": (S,), f"{base}hc{q}.mix": (S, S)})
        mix = base + "mix."
        if layer["type"] == "lightning":
            H, d, dv = m["heads"], m["dim"], m["vdim"]
            shapes.update({mix + "q": (H * d, D), mix + "k": (H * d, D), mix + "v": (H * dv, D), mix + "g": (H * dv, D),
                           mix + "norm": (H * dv,), mix + "o": (D, H * dv)})
        else:
            a, b = m["left"], m["right"]
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            left, right = mix + "left.", mix + "right."
            C, N, R = b["inner"], b["state"], b["dt_rank"]
            shapes.update({left + "q": (H * d, D), left + "k": (G * d, D), left + "v": (G * dv, D), left + "q.norm": (d,),
                           left + "k.norm": (d,), left + "o": (D, H * dv), left + "out": (D,), right + "out": (D,),
                           right + "in": (2 * C, D), right + "conv": (C, b["conv"]), right + "conv.b": (C,),
                           right + "x": (R + 2 * N, C), right + "dt": (C, R), right + "dt.b": (C,), right + "A_log": (C, N),
                           right + "D": (C,), right + "o": (D, C)})
        if mlp is None:
            continue
        ff = base + "mlp."
        units = [("", mlp.get("ff"))]
        if mlp["kind"] == "moe":
            shapes.update({ff + "router": (mlp["router"]["experts"], D), ff + "correction": (mlp["router"]["experts"],)})
            units = [(f"e{e}.", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
            if mlp.get("shared"):
                units.append(("shared.", mlp["shared"]["ff"]))
                shapes[ff + "shared.sg"] = (1, D)
        for unit, width in units:
            shapes.update({ff + unit + "gate": (width, D), ff + unit + "up": (width, D), ff + unit + "down": (D, width)})
    return shapes


def random_weights(config: Dict, seed: int, experts_alike: float = 0.9) -> Dict[str, np.ndarray]:
    """Weights that make every part count: matrices keep the size of what passes through them (the router's, the
    gates' and the experts' somewhat more); the streams' mixes lie near the unit matrix with visible crossings;
    corrections are large enough to change choices; step sizes spread over what a scan forgets quickly and slowly.
    The experts of a layer share ``experts_alike`` of their weights: where bfloat16 rounding turns a close call of the
    router the output then moves by a part of an expert, not by all of it, while in float32 any wrong choice still shows
    far above the comparison's limit."""
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
        if leaf == "alpha":
            value = rng.uniform(0.5, 1.0, shape)
        elif leaf.startswith("norm") or (leaf == "out" and parts[-2] in ("left", "right")):
            value = rng.uniform(0.6, 1.4, shape)
        elif leaf.startswith("ls"):
            value = rng.uniform(0.3, 1.0, shape)
        elif leaf == "in" and parts[1].startswith("hc"):
            value = rng.uniform(0.1, 0.6, shape)
        elif leaf == "out" and parts[1].startswith("hc"):
            value = rng.uniform(0.4, 1.2, shape)
        elif leaf == "mix" and parts[1].startswith("hc"):
            value = 0.7 * np.eye(shape[0]) + rng.normal(0.0, 0.12, shape)
        elif name.endswith("dt.b"):
            value = rng.uniform(-3.0, 0.0, shape)
        elif leaf == "b":
            value = rng.normal(0.0, 0.2, shape)
        elif leaf == "A_log":
            value = rng.uniform(-1.5, 2.0, shape)
        elif leaf in ("D", "conv"):
            value = rng.normal(0.0, 0.6, shape)
        elif leaf == "correction":
            value = rng.normal(0.0, 0.15, shape)
        elif name == "embed":
            value = rng.normal(0.0, 1.0, shape)
        elif leaf in ("router", "gate", "up", "g", "sg"):
            value = rng.normal(0.0, 1.5, shape) / math.sqrt(shape[-1])
        else:
            value = rng.normal(0.0, 1.0, shape) / math.sqrt(shape[-1])
        weights[name] = value
    return weights
