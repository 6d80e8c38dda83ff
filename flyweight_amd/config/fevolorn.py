"""Typed configuration of Fevolorn, read from its config.json keys.

Fevolorn is a decoder whose residual stream is ``streams`` rows side by side that every sublayer reads as one weighted sum and
writes to all (see ``parts/streams.py``); its norm is tanh(alpha x) w + b, and each sublayer's output is scaled channel by
channel. ``layers`` lists the layers, each with its ``type``: ``lightning`` (a linear recurrence with a fixed ``decay`` per head:
``heads``, ``dim``, ``vdim``, see ``parts/lightning.py``) or ``parallel`` (``left``: grouped softmax attention without positions
in a sliding window ``mask.size``, with a norm per query and key head; ``right``: a selective scan, ``inner``, ``state``,
``dt_rank``, ``conv`` taps, see ``parts/mamba.py``; the output is half the sum of both, each RMS-normed). ``mlp`` is ``null``,
``{"kind": "dense", "ff"}`` (a gated unit around the tanh form of gelu) or ``{"kind": "moe", "router": {"experts", "top",
"scale"}, "expert": {"ff"}, "shared": {"ff"}}`` (sigmoid scores, a correction for the choice alone, weights times ``scale``, a
gated unit that every token runs and gates). ``loop`` names a run of neighbouring layers (``start`` .. ``stop`` - 1) that every
token passes ``times`` times, one set of weights, pages and slots of its own for each pass. The embedding rows are scaled
(``embedding.scale``); the head is the table itself behind the final norm. A checkpoint names its tensors ``l<i>.<part>``
without a ".weight" suffix.
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Any, Dict, List, Mapping, Optional, Tuple

from .spec import ConfigError, LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from .vavelorn import _get, _groups, _int, _number, _or, _scale
from .zaluvik import NO_POSITION_LIMIT, LoopSizes, _window

LAYER_TYPES = ("lightning", "parallel")
FF_KINDS = ("dense", "moe")


@dataclass(frozen=True)
class LightningSizes:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]

    kind = "lightning"

    @classmethod
    def from_dict(cls, data, where) -> "LightningSizes":
        heads, dim = _int(data, "heads", where), _int(data, "dim", where)
        decay = _get(data, "decay", where)
        if not isinstance(decay, list) or len(decay) != heads or any(isinstance(d, bool) or not isinstance(d, (int, float)) for d in decay):
            raise ConfigError(f"config.json: {where}.decay must be a list of {heads} numbers, one per head")
        return cls(heads=heads, dim=dim, vdim=_or(data, "vdim", where, dim), decay=tuple(float(d) for d in decay))

    def to_dict(self) -> Dict[str, Any]:
        return {"decay": list(self.decay), "dim": self.dim, "heads": self.heads, "vdim": self.vdim}


@dataclass(frozen=True)
class ParallelSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int]               # None: every earlier key
    inner: int
    state: int
    dt_rank: int
    conv: int

    kind = "parallel"

    @classmethod
    def from_dict(cls, data, where) -> "ParallelSizes":
        left, right = _get(data, "left", where), _get(data, "right", where)
        at = where + ".left"
        heads, dim = _int(left, "heads", at), _int(left, "dim", at)
        sizes = cls(heads=heads, kv_heads=_or(left, "kv_heads", at, heads), dim=dim, vdim=_or(left, "vdim", at, dim),
                    scale=_scale(left, at, dim), window=_window(left, at), inner=_int(right, "inner", where + ".right"),
                    state=_int(right, "state", where + ".right"), dt_rank=_int(right, "dt_rank", where + ".right"),
                    conv=_int(right, "conv", where + ".right"))
        _groups(sizes.heads, sizes.kv_heads, at)
        return sizes

    def to_dict(self) -> Dict[str, Any]:
        left: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.vdim}
        if self.window is not None:
            left["mask"] = {"size": self.window}
        return {"left": left, "right": {"conv": self.conv, "dt_rank": self.dt_rank, "inner": self.inner, "state": self.state}}


@dataclass(frozen=True)
class FeedForwardSizes:
    kind: str                           # "dense" or "moe"
    ff: int                             # of the dense unit, or of one expert
    experts: int = 0
    top: int = 0
    scale: float = 1.0
    shared_ff: Optional[int] = None

    @classmethod
    def from_dict(cls, data, where) -> "FeedForwardSizes":
        kind = _get(data, "kind", where)
        if kind not in FF_KINDS:
            raise ConfigError(f"config.json: {where}.kind is {kind!r}; known: {', '.join(FF_KINDS)}")
        if kind == "dense":
            return cls(kind=kind, ff=_int(data, "ff", where))
        router, shared = _get(data, "router", where), data.get("shared")
        sizes = cls(kind=kind, ff=_int(_get(data, "expert", where), "ff", where + ".expert"),
                    experts=_int(router, "experts", where + ".router"), top=_int(router, "top", where + ".router"),
                    scale=_number(router, "scale", where + ".router") if router.get("scale") is not None else 1.0,
                    shared_ff=_int(shared, "ff", where + ".shared") if shared is not None else None)
        if sizes.top > sizes.experts:
            raise ConfigError(f"config.json: {where}.router: {sizes.top} of {sizes.experts} experts")
        return sizes

    def to_dict(self) -> Dict[str, Any]:
        if self.kind == "dense":
            return {"ff": self.ff, "kind": "dense"}
        out: Dict[str, Any] = {"expert": {"ff": self.ff}, "kind": "moe", "router": {"experts": self.experts, "scale": self.scale, "top": self.top}}
        if self.shared_ff is not None:
            out["shared"] = {"ff": self.shared_ff}
        return out


_MIXERS = {cls.kind: cls for cls in (LightningSizes, ParallelSizes)}


@dataclass(frozen=True)
class FevolornLayer:
    mixer: Any                          # LightningSizes or ParallelSizes; its ``kind`` is the layer's type
    mlp: Optional[FeedForwardSizes]     # None: the layer has no feed-forward


@dataclass(frozen=True)
class FevolornConfig:
    vocab: int
    width: int
    streams: int
    norm_eps: float
    embedding_scale: float
    layers: Tuple[FevolornLayer, ...]
    loop: Optional[LoopSizes] = None    # None: every layer once

    architecture = "Fevolorn"

    @classmethod
    def from_dict(cls, data: Mapping[str, Any]) -> "FevolornConfig":
        if not isinstance(data, Mapping):
            raise ConfigError("config.json must hold a JSON object")
        listed = _get(data, "layers", "the model")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json: 'layers' must be a list of at least one layer")
        layers: List[FevolornLayer] = []
        for index, entry in enumerate(listed):
            where = f"layers[{index}]"
            kind = _get(entry, "type", where)
            if kind not in _MIXERS:
                raise ConfigError(f"config.json: {where}.type is {kind!r}; known: {', '.join(LAYER_TYPES)}")
            mlp = entry.get("mlp")
            layers.append(FevolornLayer(mixer=_MIXERS[kind].from_dict(_get(entry, "mixer", where), where + ".mixer"),
                                        mlp=FeedForwardSizes.from_dict(mlp, where + ".mlp") if mlp is not None else None))
        loop = None
        if data.get("loop") is not None:
            loop = LoopSizes(start=_int(data["loop"], "start", "loop", least=0), stop=_int(data["loop"], "stop", "loop"),
                             times=_int(data["loop"], "times", "loop"))
            if not loop.start < loop.stop <= len(layers):
                raise ConfigError(f"config.json: loop runs layers {loop.start} .. {loop.stop - 1} of {len(layers)}")
        embedding = data.get("embedding") or {}
        return cls(vocab=_int(data, "vocab", "the model"), width=_int(data, "width", "the model"), streams=_or(data, "streams", "the model", 1),
                   norm_eps=_number(_get(data, "norm", "the model"), "eps", "norm", positive=True),
                   embedding_scale=_number(embedding, "scale", "embedding") if embedding.get("scale") is not None else 1.0,
                   layers=tuple(layers), loop=loop)

    def to_dict(self) -> Dict[str, Any]:
        layers = [{"mixer": layer.mixer.to_dict(), "mlp": None if layer.mlp is None else layer.mlp.to_dict(), "type": layer.mixer.kind}
                  for layer in self.layers]
        data: Dict[str, Any] = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale}, "layers": layers,
                                "norm": {"eps": self.norm_eps}, "streams": self.streams, "vocab": self.vocab, "width": self.width}
        if self.loop is not None:
            data["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        return data

    def save(self, folder: str) -> None:
        os.makedirs(folder, exist_ok=True)
        with open(os.path.join(folder, "config.json"), "w", encoding="utf-8") as handle:
            json.dump(self.to_dict(), handle, indent=1)

    # sizes the engine's command line and scheduler ask any configuration for
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def max_position_embeddings(self) -> int:
        return NO_POSITION_LIMIT

    def _mixer_spec(self, sizes, prefix: str) -> PartSpec:
        if sizes.kind == "lightning":
            return PartSpec("lightning", {"hidden_size": self.width, "num_heads": sizes.heads, "head_dim": sizes.dim, "v_head_dim": sizes.vdim,
                                          "decay": sizes.decay, "norm_eps": self.norm_eps}, prefix=prefix)
        left = PartSpec("gqa_attention", {
            "hidden_size": self.width, "num_heads": sizes.heads, "num_kv_heads": sizes.kv_heads, "head_dim": sizes.dim,
            "v_head_dim": sizes.vdim, "qk_norm": True, "qk_norm_eps": self.norm_eps, "window": sizes.window, "softmax_scale": sizes.scale,
            "position": PartSpec("none"), "names": {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"},
            "weight_suffix": ""}, prefix=prefix + "left.")
        right = PartSpec("mamba", {"hidden_size": self.width, "inner_size": sizes.inner, "state_size": sizes.state, "dt_rank": sizes.dt_rank,
                                   "conv_taps": sizes.conv}, prefix=prefix + "right.")
        norms = {name: PartSpec("rmsnorm", {"eps": self.norm_eps, "size": self.width, "tensor": f"{prefix}{name}.out"})
                 for name in ("left", "right")}
        return PartSpec("parallel_branches", {"branches": (("left", left, 0.5), ("right", right, 0.5)), "norms": norms}, prefix=prefix)

    def _ffn_spec(self, mlp: FeedForwardSizes, prefix: str) -> PartSpec:
        if mlp.kind == "dense":
            return PartSpec("swiglu", {"hidden_size": self.width, "intermediate_size": mlp.ff, "activation": "gelu_tanh",
                                       "names": {"gate": "gate", "up": "up", "down": "down"}, "weight_suffix": ""}, prefix=prefix)
        return PartSpec("moe_swiglu", {
            "hidden_size": self.width, "num_experts": mlp.experts, "top": mlp.top, "intermediate_size": mlp.ff,
            "shared_intermediate_size": mlp.shared_ff, "shared_gate": mlp.shared_ff is not None, "router_bias": False,
            "router_scores": "sigmoid", "router_correction": True, "weight_scale": mlp.scale, "normalize": False}, prefix=prefix)

    def model_spec(self) -> ModelSpec:
        def norm(tensor: str) -> PartSpec:
            return PartSpec("tanh", {"size": self.width, "tensor": tensor})

        def connection(base: str, number: int) -> PartSpec:
            return PartSpec("stream_connection", {"hidden_size": self.width, "streams": self.streams, "scale_tensor": f"{base}ls{number}"},
                            prefix=f"{base}hc{number}.")

        layers: List[LayerSpec] = []
        for index, layer in enumerate(self.layers):
            base = f"l{index}."
            params: Dict[str, Any] = {"mixer_connection": connection(base, 1)}
            if layer.mlp is not None:
                params["ffn_connection"] = connection(base, 2)
            layers.append(LayerSpec(
                arrangement="stream_residual", mixer_norm=norm(base + "norm1"), mixer=self._mixer_spec(layer.mixer, base + "mix."),
                ffn_norm=None if layer.mlp is None else norm(base + "norm2"),
                ffn=None if layer.mlp is None else self._ffn_spec(layer.mlp, base + "mlp."), params=params))
        order = list(range(len(layers)))
        if self.loop is not None:
            order[self.loop.start:self.loop.stop] = order[self.loop.start:self.loop.stop] * self.loop.times
        schedule = tuple(ScheduleEntry(layer=index, cache=run) for run, index in enumerate(order))      # every run keeps its own
        spec = ModelSpec(
            architecture=self.architecture, hidden_size=self.width, vocab_size=self.vocab, max_positions=NO_POSITION_LIMIT,
            layers=tuple(layers), schedule=schedule, final_norm=norm("final.norm"), embedding_name="embed", lm_head_name=None,
            embedding_scale=self.embedding_scale, streams=self.streams)
        spec.validate()
        return spec
