"""Typed configuration of Zaluvik, read from its config.json keys.

Zaluvik is a decoder with a layer norm (weight and bias) before and behind every sublayer, x += m N1b(mixer(N1(x))), then
x += m N2b(ff(N2(x))), with one factor m for the model (``residual_mult``). ``loop`` names a run of neighbouring layers
(``start`` .. ``stop`` - 1) that every token passes ``times`` times, one set of weights, pages of its own for each pass;
ahead of every pass the residual stream becomes ``loop.in`` times [stream; embedding output]. ``layers`` lists the layers, each
with its ``type``: ``attention`` (grouped heads without positions whose weights are sigmoids that the heads mix, see
``parts/sigmoid_attention.py``) or ``latent_attention`` (softmax attention over a cached latent with a rotated key part that
all heads share, one map for the queries, a gate per head, see ``parts/latent.py``), both in a sliding window ``mask.size``.
``mlp`` is ``null``, ``{"kind": "dense", "ff"}`` (two maps around a gelu) or ``{"kind": "moe", "router": {"experts", "top",
"groups": {"count", "keep"}}, "expert": {"ff"}, "shared": {"ff"}}`` (sigmoid scores, groups scored by their two best experts).
The embedding rows are scaled (``embedding.scale``); the head is the table itself behind the final norm. A checkpoint names
its tensors ``l<i>.<part>`` without a ".weight" suffix.
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Any, Dict, List, Mapping, Optional, Tuple

from .spec import ConfigError, LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from .vavelorn import _get, _groups, _int, _number, _or, _scale

LAYER_TYPES = ("attention", "latent_attention")
FF_KINDS = ("dense", "moe")
NO_POSITION_LIMIT = 1 << 30


def _window(data, where) -> Optional[int]:
    mask = data.get("mask")
    return _int(mask, "size", where + ".mask") if mask is not None else None


@dataclass(frozen=True)
class MixedHeadSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int]               # None: every earlier key

    kind = "attention"

    @classmethod
    def from_dict(cls, data, where) -> "MixedHeadSizes":
        heads, dim = _int(data, "heads", where), _int(data, "dim", where)
        sizes = cls(heads=heads, kv_heads=_or(data, "kv_heads", where, heads), dim=dim, vdim=_or(data, "vdim", where, dim),
                    scale=_scale(data, where, dim), window=_window(data, where))
        _groups(sizes.heads, sizes.kv_heads, where)
        return sizes

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.vdim}
        if self.window is not None:
            out["mask"] = {"size": self.window}
        return out


@dataclass(frozen=True)
class WindowedLatentSizes:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    window: Optional[int]
    rot_dims: int
    rot_base: float

    kind = "latent_attention"

    @classmethod
    def from_dict(cls, data, where) -> "WindowedLatentSizes":
        rot = data.get("rot") if isinstance(data, Mapping) else None
        dim, rot_dim = _int(data, "dim", where), _or(data, "rot_dim", where, 0, least=0)
        sizes = cls(heads=_int(data, "heads", where), dim=dim, rot_dim=rot_dim, vdim=_or(data, "vdim", where, dim),
                    kv_rank=_int(data, "kv_rank", where), scale=_scale(data, where, dim + rot_dim), window=_window(data, where),
                    rot_dims=_or(rot, "dims", where + ".rot", rot_dim, least=0) if rot is not None else 0,
                    rot_base=_number(rot, "base", where + ".rot", positive=True) if rot is not None else 1.0)
        if sizes.rot_dim % 2 or sizes.rot_dims % 2 or sizes.rot_dims > sizes.rot_dim:
            raise ConfigError(f"config.json: {where}: rot_dim {sizes.rot_dim} and rot.dims {sizes.rot_dims} must be even, rot.dims at most rot_dim")
        return sizes

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "rot": {"base": self.rot_base, "dims": self.rot_dims},
                               "rot_dim": self.rot_dim, "scale": self.scale, "vdim": self.vdim}
        if self.window is not None:
            out["mask"] = {"size": self.window}
        return out


@dataclass(frozen=True)
class FeedForwardSizes:
    kind: str                           # "dense" or "moe"
    ff: int                             # of the dense unit, or of one expert
    experts: int = 0
    top: int = 0
    groups: int = 1
    keep: int = 1
    shared_ff: Optional[int] = None

    @classmethod
    def from_dict(cls, data, where) -> "FeedForwardSizes":
        kind = _get(data, "kind", where)
        if kind not in FF_KINDS:
            raise ConfigError(f"config.json: {where}.kind is {kind!r}; known: {', '.join(FF_KINDS)}")
        if kind == "dense":
            return cls(kind=kind, ff=_int(data, "ff", where))
        router, shared = _get(data, "router", where), data.get("shared")
        groups = router.get("groups") if isinstance(router, Mapping) else None
        count = _int(groups, "count", where + ".router.groups") if groups is not None else 1
        sizes = cls(kind=kind, ff=_int(_get(data, "expert", where), "ff", where + ".expert"),
                    experts=_int(router, "experts", where + ".router"), top=_int(router, "top", where + ".router"), groups=count,
                    keep=_or(groups, "keep", where + ".router.groups", count) if groups is not None else 1,
                    shared_ff=_int(shared, "ff", where + ".shared") if shared is not None else None)
        if sizes.experts % sizes.groups or sizes.keep > sizes.groups or sizes.top > sizes.keep * (sizes.experts // sizes.groups):
            raise ConfigError(f"config.json: {where}.router: {sizes.top} of {sizes.experts} experts from {sizes.keep} of {sizes.groups} equal groups")
        return sizes

    def to_dict(self) -> Dict[str, Any]:
        if self.kind == "dense":
            return {"ff": self.ff, "kind": "dense"}
        out: Dict[str, Any] = {"expert": {"ff": self.ff}, "kind": "moe",
                               "router": {"experts": self.experts, "groups": {"count": self.groups, "keep": self.keep}, "top": self.top}}
        if self.shared_ff is not None:
            out["shared"] = {"ff": self.shared_ff}
        return out


_MIXERS = {cls.kind: cls for cls in (MixedHeadSizes, WindowedLatentSizes)}


@dataclass(frozen=True)
class ZaluvikLayer:
    mixer: Any                          # MixedHeadSizes or WindowedLatentSizes; its ``kind`` is the layer's type
    mlp: Optional[FeedForwardSizes]     # None: the layer has no feed-forward


@dataclass(frozen=True)
class LoopSizes:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class ZaluvikConfig:
    vocab: int
    width: int
    norm_eps: float
    residual_mult: float
    embedding_scale: float
    layers: Tuple[ZaluvikLayer, ...]
    loop: Optional[LoopSizes] = None    # None: every layer once, and no map of the input

    architecture = "Zaluvik"

    @classmethod
    def from_dict(cls, data: Mapping[str, Any]) -> "ZaluvikConfig":
        if not isinstance(data, Mapping):
            raise ConfigError("config.json must hold a JSON object")
        listed = _get(data, "layers", "the model")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json: 'layers' must be a list of at least one layer")
        layers: List[ZaluvikLayer] = []
        for index, entry in enumerate(listed):
            where = f"layers[{index}]"
            kind = _get(entry, "type", where)
            if kind not in _MIXERS:
                raise ConfigError(f"config.json: {where}.type is {kind!r}; known: {', '.join(LAYER_TYPES)}")
            mlp = entry.get("mlp")
            layers.append(ZaluvikLayer(mixer=_MIXERS[kind].from_dict(_get(entry, "mixer", where), where + ".mixer"),
                                       mlp=FeedForwardSizes.from_dict(mlp, where + ".mlp") if mlp is not None else None))
        loop = None
        if data.get("loop") is not None:
            loop = LoopSizes(start=_int(data["loop"], "start", "loop", least=0), stop=_int(data["loop"], "stop", "loop"),
                             times=_int(data["loop"], "times", "loop"))
            if not loop.start < loop.stop <= len(layers):
                raise ConfigError(f"config.json: loop runs layers {loop.start} .. {loop.stop - 1} of {len(layers)}")
        embedding = data.get("embedding") or {}
        return cls(vocab=_int(data, "vocab", "the model"), width=_int(data, "width", "the model"),
                   norm_eps=_number(_get(data, "norm", "the model"), "eps", "norm", positive=True),
                   residual_mult=_number(data, "residual_mult", "the model") if data.get("residual_mult") is not None else 1.0,
                   embedding_scale=_number(embedding, "scale", "embedding") if embedding.get("scale") is not None else 1.0,
                   layers=tuple(layers), loop=loop)

    def to_dict(self) -> Dict[str, Any]:
        layers = [{"mixer": layer.mixer.to_dict(), "mlp": None if layer.mlp is None else layer.mlp.to_dict(), "type": layer.mixer.kind}
                  for layer in self.layers]
        data: Dict[str, Any] = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale}, "layers": layers,
                                "norm": {"eps": self.norm_eps}, "residual_mult": self.residual_mult, "vocab": self.vocab, "width": self.width}
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
        if sizes.kind == "latent_attention":
            position = PartSpec("rotary_neox", {"theta": sizes.rot_base, "rotary_dim": sizes.rot_dims, "head_dim": max(sizes.rot_dim, 2)})
            return PartSpec("latent_attention", {
                "hidden_size": self.width, "num_heads": sizes.heads, "head_dim": sizes.dim, "v_head_dim": sizes.vdim, "q_rank": None,
                "kv_rank": sizes.kv_rank, "norm_eps": self.norm_eps, "softmax_scale": sizes.scale, "output_gate": "per_head",
                "window": sizes.window, "rot_dim": sizes.rot_dim, "position": position}, prefix=prefix)
        return PartSpec("sigmoid_attention", {
            "hidden_size": self.width, "num_heads": sizes.heads, "num_kv_heads": sizes.kv_heads, "head_dim": sizes.dim,
            "v_head_dim": sizes.vdim, "softmax_scale": sizes.scale, "window": sizes.window, "qk_norm": True, "qk_norm_eps": self.norm_eps,
            "output_gate": True}, prefix=prefix)

    def _ffn_spec(self, mlp: FeedForwardSizes, prefix: str) -> PartSpec:
        if mlp.kind == "dense":
            return PartSpec("gelu_mlp", {"hidden_size": self.width, "intermediate_size": mlp.ff, "names": {"up": "up", "down": "down"},
                                         "weight_suffix": ""}, prefix=prefix)
        return PartSpec("moe_swiglu", {
            "hidden_size": self.width, "num_experts": mlp.experts, "top": mlp.top, "intermediate_size": mlp.ff,
            "shared_intermediate_size": mlp.shared_ff, "router_bias": False, "router_scores": "sigmoid",
            "router_groups": (mlp.groups, mlp.keep), "group_score": "pair"}, prefix=prefix)

    def model_spec(self) -> ModelSpec:
        def norm(tensor: str) -> PartSpec:
            return PartSpec("layernorm", {"eps": self.norm_eps, "size": self.width, "tensor": tensor, "bias": True})

        layers: List[LayerSpec] = []
        for index, layer in enumerate(self.layers):
            base = f"l{index}."
            params: Dict[str, Any] = {"mixer_post_norm": norm(base + "norm1b"), "residual_mult": self.residual_mult}
            if layer.mlp is not None:
                params["ffn_post_norm"] = norm(base + "norm2b")
            layers.append(LayerSpec(
                arrangement="sandwich_norm_residual", mixer_norm=norm(base + "norm1"), mixer=self._mixer_spec(layer.mixer, base + "mix."),
                ffn_norm=None if layer.mlp is None else norm(base + "norm2"),
                ffn=None if layer.mlp is None else self._ffn_spec(layer.mlp, base + "mlp."), params=params))
        # the order in which layers run, a pass that begins marked as one that joins the input; every run has a cache entry of its own
        order = [(index, False) for index in range(len(layers))]
        if self.loop is not None:
            once = [(index, index == self.loop.start) for index in range(self.loop.start, self.loop.stop)]
            order[self.loop.start:self.loop.stop] = once * self.loop.times
        schedule = tuple(ScheduleEntry(layer=index, cache=run, joins_input=joins) for run, (index, joins) in enumerate(order))
        spec = ModelSpec(
            architecture=self.architecture, hidden_size=self.width, vocab_size=self.vocab, max_positions=NO_POSITION_LIMIT,
            layers=tuple(layers), schedule=schedule, final_norm=norm("final.norm"), embedding_name="embed", lm_head_name=None,
            embedding_scale=self.embedding_scale,
            input_join=None if self.loop is None else PartSpec("input_join", {"hidden_size": self.width, "tensor": "loop.in"}))
        spec.validate()
        return spec
