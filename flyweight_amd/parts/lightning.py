"""Lightning attention: a linear recurrence over a matrix state per head with one fixed decay per head.

q = silu(W_q h), k = silu(W_k h) (heads of ``head_dim`` channels), v = silu(W_v h) (heads of ``v_head_dim``). Per head, from S = 0:

    S <- decay S + k v^T;   o = S^T q

The heads' o side by side are divided by their common root mean square, times a weight per channel, times
sigmoid(W_g h); out = W_o of that. The decays are constants of the model. The state and everything that enters the
recurrence behind the projections is float32 in either run dtype; a request's slot keeps S.
"""

from __future__ import annotations

from typing import Dict

import torch

from ..cache.needs import FixedState
from ..config.spec import ConfigError
from ..kernels import ops
from ..weights.loader import TensorDecl
from .base import Mixer, register_mixer
from .chunks import RecurrenceChunks
from .linear import Linear

_DEFAULT_NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "norm": "norm", "o": "o"}


@register_mixer("lightning")
class LightningAttention(RecurrenceChunks, Mixer):
    graph_safe = True

    def __init__(self, spec):
        super().__init__(spec)
        self.hidden = int(spec["hidden_size"])
        self.heads = int(spec["num_heads"])
        self.dim = int(spec["head_dim"])
        self.vdim = int(spec["v_head_dim"])
        self.decays = tuple(float(d) for d in spec["decay"])
        self.eps = float(spec["norm_eps"])
        self.names = {**_DEFAULT_NAMES, **dict(spec.get("names", {}))}
        if len(self.decays) != self.heads:
            raise ConfigError(f"{len(self.decays)} decays for {self.heads} heads")
        if not 1 <= self.dim <= ops.MAX_DECAY_DIM or self.vdim < 1:
            raise ConfigError(f"the recurrence's head sizes ({self.dim}, {self.vdim}): keys of 1..{ops.MAX_DECAY_DIM} channels")

    def cache_need(self):
        return {"state": FixedState((self.heads, self.dim, self.vdim), torch.float32)}

    def _name(self, which: str) -> str:
        return self.prefix + self.names[which]

    def mixing_flops(self, rows: int, keys_before: int = 0) -> int:
        """Per token and head a write and a read of the state, a multiply and an add each (the write two multiplies)."""
        return 5 * self.heads * self.dim * self.vdim * rows

    def tensors(self) -> Dict[str, TensorDecl]:
        D, qk, vw = self.hidden, self.heads * self.dim, self.heads * self.vdim
        return {self._name("q"): TensorDecl((qk, D)), self._name("k"): TensorDecl((qk, D)), self._name("v"): TensorDecl((vw, D)),
                self._name("g"): TensorDecl((vw, D)), self._name("norm"): TensorDecl((vw,), "vector", "norm"),
                self._name("o"): TensorDecl((D, vw))}

    def bind(self, tensors, dtype, device) -> None:
        super().bind(tensors, dtype, device)
        # one operand for everything that reads h (float32 sums out: the recurrence and the gate read them as they are)
        self.in_proj = Linear(torch.cat([tensors[self._name(n)] for n in ("q", "k", "v", "g")], dim=0))
        self.out = Linear(tensors[self._name("o")])
        self.norm_weight = tensors[self._name("norm")]
        self.powers = ops.decay_powers(self.decays, device)

    def heads_output(self, h, ctx, cache) -> torch.Tensor:
        """The heads' normed and gated read-outs [rows, heads * vdim] in the activation dtype; the request's state moves on."""
        proj = self.in_proj.forward(h, out_dtype=torch.float32)
        qk, vw = self.heads * self.dim, self.heads * self.vdim
        o = ops.decay_recurrence(proj[:, :qk], proj[:, qk:2 * qk], proj[:, 2 * qk:2 * qk + vw], self.powers, cache["state"].state,
                                 ctx.seg_row0, ctx.seg_slot, ctx.num_segments, self.heads, self.dim, self.vdim, **self.chunk_arguments(ctx))
        return ops.gated_head_norm(o, proj[:, 2 * qk + vw:], self.norm_weight, 1, vw, self.eps, self.dtype)

    def output(self, h, ctx, cache) -> torch.Tensor:
        return self.out.forward(self.heads_output(h, ctx, cache), out_dtype=torch.float32)

    def forward(self, h, residual, ctx, cache):
        return self.out.accumulate(self.heads_output(h, ctx, cache), residual, then=getattr(ctx, "upcoming_norm", None))
