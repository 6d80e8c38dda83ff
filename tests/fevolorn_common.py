"""Shared by the Fevolorn tests: small configurations that differ from each other in every size and option,
model folders with random weights that make every part count, and the comparison's limits."""

from __future__ import annotations

import copy
import json
import os
from typing import List, Optional

import numpy as np

import plain_fevolorn as plain


def lightning(heads, dim, vdim, decay):
    return {"type": "lightning", "mixer": {"decay": list(decay), "dim": dim, "heads": heads, "vdim": vdim}}


def parallel(heads, kv_heads, dim, vdim, window, scale, inner, state, dt_rank, conv):
    left = {"dim": dim, "heads": heads, "kv_heads": kv_heads, "scale": scale, "vdim": vdim}
    if window is not None:
        left["mask"] = {"size": window}
    return {"type": "parallel", "mixer": {"left": left, "right": {"conv": conv, "dt_rank": dt_rank, "inner": inner, "state": state}}}


def dense(ff):
    return {"ff": ff, "kind": "dense"}


def moe(experts, top, scale, ff, shared=None):
    out = {"expert": {"ff": ff}, "kind": "moe", "router": {"experts": experts, "scale": scale, "top": top}}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer, mlp):
    return {**copy.deepcopy(mixer), "mlp": copy.deepcopy(mlp)}


def model(vocab, width, streams, layers, loop=None, eps=1e-5, scale=1.0):
    out = {"architecture": "Fevolorn", "embedding": {"scale": scale}, "vocab": vocab, "width": width, "streams": streams,
           "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


# X: both mixers and both feed-forwards, a loop of two layers passed three times with a layer before and one behind it,
# three streams, windows of 50 and 130 that cross page borders, values wider and narrower than keys, three key heads under
# six, decays from forgetting at once to barely forgetting, nine experts of which three are chosen with a shared unit.
CONFIG_X = model(300, 96, 3, [
    layer(lightning(3, 32, 48, [0.3, 0.93, 0.998]), dense(120)),
    layer(parallel(6, 3, 32, 48, 50, 0.5, 120, 12, 6, 4), moe(9, 3, 1.7, 40, shared=56)),
    layer(lightning(5, 16, 16, [0.99, 0.5, 0.9, 0.97, 0.7]), moe(8, 2, 0.8, 48)),
    layer(parallel(5, 1, 48, 16, 130, 0.4, 72, 20, 10, 3), dense(72)),
], loop=(1, 3, 3), scale=1.4)

# Y: the loop begins at the first layer and is one layer passed twice, one stream, scale 1; windows of 64 and 33, a key
# head to every head, one expert chosen, as many chosen as there are, no shared unit, a layer without feed-forward, a
# decay of exactly 1, keys and values of one size, a convolution of two taps and one of one, a power of two of states.
CONFIG_Y = model(200, 64, 1, [
    layer(parallel(4, 4, 16, 16, 64, 0.8, 64, 16, 16, 2), moe(4, 1, 1.0, 64, shared=32)),
    layer(lightning(2, 64, 64, [1.0, 0.95]), moe(3, 3, 2.5, 32)),
    layer(parallel(2, 1, 32, 32, 33, 0.6, 32, 8, 4, 1), None),
    layer(lightning(1, 16, 32, [0.99]), None),
], loop=(0, 1, 2), eps=1e-6)

# Z: the corners. No loop; five streams, a window of one key, a window longer than any prompt here, none at all, one head,
# heads of 8 and of 20 channels (off the matrix-core kernels), a width that is no multiple of eight, one state a channel, 33
# of them, an odd rank and a rank of one, seven taps, more channels in a head's keys than in its values and the other way.
CONFIG_Z = model(97, 44, 5, [
    layer(parallel(1, 1, 8, 12, 1, 1.0, 30, 1, 1, 7), None),
    layer(lightning(3, 5, 70, [0.9, 0.2, 0.985]), moe(2, 1, 0.5, 50)),
    layer(parallel(6, 3, 20, 20, None, 0.9, 44, 33, 5, 4), dense(30)),
    layer(lightning(1, 100, 12, [0.97]), moe(9, 4, 1.5, 12, shared=12)),
    layer(parallel(3, 3, 24, 8, 500, 0.7, 100, 9, 7, 4), moe(4, 2, 1.0, 16)),
], scale=0.8)

# W: wide enough that a prompt of some hundred tokens goes through the tiled prompt products, the matrix-core attention
# kernels, the grouped products and chunks of both recurrences in which every wave has work.
_W_MIX = moe(16, 4, 1.2, 256, shared=384)
CONFIG_W = model(1000, 512, 4, [
    layer(lightning(4, 128, 128, [0.8, 0.95, 0.99, 0.999]), dense(1024)),
    layer(parallel(8, 2, 64, 64, 150, 0.25, 1024, 16, 32, 4), _W_MIX),
    layer(lightning(2, 64, 256, [0.9, 0.995]), _W_MIX),
], loop=(0, 2, 2))

CONFIGS = {"X": CONFIG_X, "Y": CONFIG_Y, "Z": CONFIG_Z, "W": CONFIG_W}

# Largest difference from the plain float64 model, as a fraction of the largest logit compared, and the same for the
# root mean square. float32 shows the logic right; the bfloat16 limits have to tell rounding (2e-3 at every stored
# activation) from a fault, and the configurations make faults large. In bfloat16 a router's choice between two
# experts of nearly equal scores can fall the other way; the experts of a layer are drawn alike in most of their
# weights, so that such a row moves by a part of an expert and by the difference of the two corrections, and the rows that
# read its state or keys by less: one row in fifteen may pass the largest difference, the root mean square over all
# rows has to hold.
MAX_TOL = {"float32": 4e-5, "bfloat16": 8e-2}
RMS_TOL = {"float32": 8e-6, "bfloat16": 2e-2}
ROWS_OVER = {"float32": 0.0, "bfloat16": 0.067}


def only_mixer(config: dict, kind: str) -> dict:
    """The same model with the layers of one mixer alone, no feed-forward and no loop: one mechanism between its norms."""
    out = copy.deepcopy(config)
    out["layers"] = [dict(entry, mlp=None) for entry in out["layers"] if entry["type"] == kind]
    out.pop("loop", None)
    return out


def make_folder(folder: str, config: dict, seed: int = 0, change=None):
    """Writes config.json and model.safetensors (everything in bfloat16) and returns the weights as the plain model
    reads them: the stored values, in float64. ``change``: called with the weights before they are stored."""
    import torch
    from safetensors.torch import save_file
    weights = plain.random_weights(config, seed)
    if change is not None:
        change(weights)
    stored = {name: torch.from_numpy(np.asarray(value)).to(torch.bfloat16) for name, value in weights.items()}
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as handle:
        json.dump(config, handle)
    save_file({name: value.contiguous() for name, value in stored.items()}, os.path.join(folder, "model.safetensors"))
    return {name: value.to(torch.float64).numpy() for name, value in stored.items()}


def random_tokens(vocab: int, count: int, seed: int) -> List[int]:
    return np.random.default_rng(seed).integers(0, vocab, size=count).tolist()


def assert_close(found: np.ndarray, expected: np.ndarray, dtype: str, what: str = "", scale: Optional[float] = None) -> None:
    assert found.shape == expected.shape, f"{what}: shape {found.shape} vs {expected.shape}"
    assert np.isfinite(found).all(), f"{what}: non-finite values"
    scale = max(1.0, float(np.abs(expected).max())) if scale is None else scale
    error = np.abs(found.astype(np.float64) - expected)
    worst, rms = float(error.max()), float(np.sqrt(np.mean(error ** 2)))
    over = error.reshape(error.shape[0], -1).max(axis=-1) > MAX_TOL[dtype] * scale
    allowed = int(ROWS_OVER[dtype] * error.shape[0])
    assert int(over.sum()) <= allowed, (f"{what}: largest difference {worst:.3e} exceeds {MAX_TOL[dtype] * scale:.3e} in {int(over.sum())} rows "
                                        f"({allowed} allowed; first row over: {int(np.argmax(over))})")
    assert rms <= RMS_TOL[dtype] * scale, f"{what}: rms difference {rms:.3e} exceeds {RMS_TOL[dtype] * scale:.3e}"
