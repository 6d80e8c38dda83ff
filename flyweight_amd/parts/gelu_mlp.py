"""Feed-forward of two maps around a gelu: f = W_down gelu(W_up h), no biases, gelu the error-function form z Phi(z). The
unit is formed from the float32 sums as the product stores them, and rounded once."""

from __future__ import annotations

from typing import Dict

import torch

from ..weights.loader import TensorDecl
from .base import FeedForward, register_feed_forward
from .linear import Linear

_DEFAULT_NAMES = {"up": "up_proj", "down": "down_proj"}


@register_feed_forward("gelu_mlp")
class GeluMLP(FeedForward):
    graph_safe = True

    def __init__(self, spec):
        super().__init__(spec)
        self.hidden = int(spec["hidden_size"])
        self.intermediate = int(spec["intermediate_size"])
        self.names = {**_DEFAULT_NAMES, **dict(spec.get("names", {}))}
        self.weight_suffix = spec.get("weight_suffix", ".weight")

    def _name(self, which: str) -> str:
        return f"{self.prefix}{self.names[which]}{self.weight_suffix}"

    def tensors(self) -> Dict[str, TensorDecl]:
        return {self._name("up"): TensorDecl((self.intermediate, self.hidden)),
                self._name("down"): TensorDecl((self.hidden, self.intermediate))}

    def bind(self, tensors, dtype, device) -> None:
        super().bind(tensors, dtype, device)
        self.up = Linear(tensors[self._name("up")])
        self.down = Linear(tensors[self._name("down")])

    def forward(self, h, residual, ctx):
        return self.down.accumulate(self.up.gelu(h), residual, then=getattr(ctx, "upcoming_norm", None))

    def output(self, h, ctx) -> torch.Tensor:
        """The feed-forward's output as float32 rows of its own (for arrangements that do something to
        it before it joins the residual stream)."""
        return self.down.forward(self.up.gelu(h), out_dtype=torch.float32)
