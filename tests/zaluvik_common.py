"""Shared by the Zaluvik tests: small configurations that differ from each other in every size and option,
model folders with random weights that make every part count, and the comparison's limits."""

from __future__ import annotations

import copy
import json
import os
from typing import List, Optional

import numpy as np

import plain_zaluvik as plain


def attention(heads, kv_heads, dim, vdim, window, scale):
    out = {"dim": dim, "heads": heads, "kv_heads": kv_heads, "scale": scale, "vdim": vdim}
    if window is not None:
        out["mask"] = {"size": window}
    return {"type": "attention", "mixer": out}


def latent(heads, dim, rot_dim, vdim, kv_rank, window, scale, base=10000.0, rot_dims=None):
    out = {"dim": dim, "heads": heads, "kv_rank": kv_rank, "rot": {"base": base, "dims": rot_dim if rot_dims is None else rot_dims},
           "rot_dim": rot_dim, "scale": scale, "vdim": vdim}
    if window is not None:
        out["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": out}


def dense(ff):
    return {"ff": ff, "kind": "dense"}


def moe(experts, top, groups, keep, ff, shared=None):
    out = {"expert": {"ff": ff}, "kind": "moe", "router": {"experts": experts, "groups": {"count": groups, "keep": keep}, "top": top}}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer, mlp):
    return {**copy.deepcopy(mixer), "mlp": copy.deepcopy(mlp)}


def model(vocab, width, layers, loop=None, eps=1e-5, mult=0.6, scale=1.0):
    out = {"architecture": "Zaluvik", "embedding": {"scale": scale}, "vocab": vocab, "width": width, "norm": {"eps": eps},
           "residual_mult": mult, "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


# X: both mixers and both feed-forwards, a loop of two layers passed three times with a layer before and one behind it,
# windows of 50 and 90 that cross page borders, values wider and narrower than keys, three key heads under six, a latent
# of 48 channels with a rotated part of 16, nine experts in three groups of which two are kept, with a shared unit.
CONFIG_X = model(300, 96, [
    layer(attention(6, 3, 32, 48, 50, 0.5), dense(120)),
    layer(latent(4, 16, 16, 32, 48, 90, 0.3), moe(9, 3, 3, 2, 40, shared=56)),
    layer(attention(5, 1, 48, 16, 130, 0.4), moe(8, 2, 4, 2, 48)),
    layer(attention(6, 3, 32, 48, 50, 0.5), dense(72)),
], loop=(1, 3, 3), scale=0.8)

# Y: the loop begins at the first layer and is one layer passed twice, the stream taken as it comes (factor 1, scale 1);
# windows of 64 and 33, a key head to every head, one key head, a rotated part of which a quarter turns, one group (every
# expert can be chosen), one expert chosen, as many chosen as there are, no shared unit, a layer without feed-forward.
CONFIG_Y = model(200, 64, [
    layer(latent(2, 32, 32, 16, 32, 64, 0.25, base=100.0, rot_dims=8), moe(4, 1, 1, 1, 64, shared=32)),
    layer(attention(4, 4, 16, 16, 33, 0.8), moe(3, 3, 1, 1, 32)),
    layer(attention(2, 1, 48, 32, 64, 0.6), None),
], loop=(0, 1, 2), eps=1e-6, mult=1.0)

# Z: the corners. No loop; a window of one key, a window longer than any prompt here, none at all, one head, heads of 8
# and of 20 channels and seventeen heads (off the matrix-core kernels), a latent of 24 with a rotated part of 2, a width
# that is no multiple of eight, groups of one expert, the whole stream turned round (a negative factor).
CONFIG_Z = model(97, 44, [
    layer(attention(1, 1, 8, 12, 1, 1.0), None),
    layer(latent(1, 12, 2, 20, 24, 500, 0.6), moe(2, 1, 2, 1, 50)),
    layer(attention(6, 3, 20, 20, None, 0.9), dense(30)),
    layer(latent(3, 8, 4, 8, 20, None, 0.4), moe(9, 4, 3, 2, 12, shared=12)),
    layer(attention(17, 17, 16, 16, 40, 0.7), moe(4, 2, 4, 2, 16)),
], mult=-0.7, scale=1.3)

# W: wide enough that a prompt of some hundred tokens goes through the tiled prompt products and the matrix-core
# attention kernels (sixteen heads of 64 channels on four key heads, two of 128 on two; a latent of 128 + 64 channels).
_W_MIX = moe(16, 4, 4, 2, 256, shared=384)
CONFIG_W = model(1000, 512, [
    layer(attention(16, 4, 64, 64, 150, 0.25), dense(1024)),
    layer(latent(8, 64, 64, 64, 128, 200, 0.09), _W_MIX),
    layer(attention(2, 2, 128, 64, 100, 0.2), _W_MIX),
], loop=(0, 2, 2))

CONFIGS = {"X": CONFIG_X, "Y": CONFIG_Y, "Z": CONFIG_Z, "W": CONFIG_W}

# Largest difference from the plain float64 model, as a fraction of the largest logit compared, and the same for the
# root mean square. float32 shows the logic right; the bfloat16 limits have to tell rounding (2e-3 at every stored
# activation) from a fault, and the configurations make faults large. In bfloat16 a router's choice between two
# experts (or two groups) of nearly equal scores can fall the other way; the experts of a layer are drawn alike in most
# of their weights, so that such a row moves by a part of an expert: one row in twenty may pass the largest difference,
# the root mean square over all rows has to hold.
MAX_TOL = {"float32": 3e-5, "bfloat16": 8e-2}
RMS_TOL = {"float32": 6e-6, "bfloat16": 2e-2}
ROWS_OVER = {"float32": 0.0, "bfloat16": 0.05}


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
