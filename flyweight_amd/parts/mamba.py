"""The selective scan block (Mamba: Gu and Dao, "Mamba: Linear-Time Sequence Modeling with Selective State Spaces").

[x | z] = W_in h, ``inner`` channels each; x passes a short causal convolution per channel (with a bias) and silu.
[low | B | C] = W_x x, dt = softplus(W_dt low + b), one step size per channel. With A = -exp(A_log), per channel c and state n,
from S = 0:

    S <- exp(dt_c A[c, n]) S + dt_c x_c B_n;   y_c = sum_n S C_n + D_c x_c

and out = W_o (y * silu(z)). A request's slot keeps S (float32 [state, inner]) and the convolution's last taps - 1 inputs.
The convolution, the step sizes, the decays and the state are float32 in either run dtype; x is rounded for W_x, the low
part for W_dt (not in steps of a few single rows, whose scan forms that map itself), and y * silu(z) for W_o.
"""

from __future__ import annotations

import math
from typing import Dict

import torch

from ..cache.needs import FixedState
from ..config.spec import ConfigError
from ..kernels import ops
from ..weights.loader import TensorDecl
from .base import Mixer, register_mixer
from .chunks import RecurrenceChunks
from .linear import Linear

_DEFAULT_NAMES = {"in": "in", "conv": "conv", "conv_bias": "conv.b", "x": "x", "dt": "dt", "dt_bias": "dt.b", "A_log": "A_log", "D": "D",
                  "o": "o"}


@register_mixer("mamba")
class Mamba(RecurrenceChunks, Mixer):
    graph_safe = True
    # up to so many single rows the scan forms the step sizes' map itself: two launches fewer, but every row reads the map
    LOW_RANK_ROWS = 16

    def __init__(self, spec):
        super().__init__(spec)
        self.hidden = int(spec["hidden_size"])
        self.inner = int(spec["inner_size"])
        self.states = int(spec["state_size"])
        self.rank = int(spec["dt_rank"])
        self.taps_count = int(spec["conv_taps"])
        self.names = {**_DEFAULT_NAMES, **dict(spec.get("names", {}))}
        if not 1 <= self.states <= ops.MAX_SCAN_STATES:
            raise ConfigError(f"a scan of {self.states} states a channel (1..{ops.MAX_SCAN_STATES})")
        if not 1 <= self.taps_count <= 16:
            raise ConfigError(f"a short convolution of {self.taps_count} taps (1..16)")

    def cache_need(self):
        need = {"state": FixedState((self.states, self.inner), torch.float32)}
        if self.taps_count > 1:
            need["conv"] = FixedState((self.inner, self.taps_count - 1), torch.float32)
        return need

    def _name(self, which: str) -> str:
        return self.prefix + self.names[which]

    def mixing_flops(self, rows: int, keys_before: int = 0) -> int:
        """The convolution, and per channel and state the decay's exponential and product, the write and the read."""
        return rows * self.inner * (2 * self.taps_count + 7 * self.states + 8)

    def gathered_tensors(self):
        """The step sizes' map in its second layout: a step reads one of the two (counted once)."""
        return (self.low_rank,)

    def tensors(self) -> Dict[str, TensorDecl]:
        D, C, N, R = self.hidden, self.inner, self.states, self.rank
        return {
            self._name("in"): TensorDecl((2 * C, D)),
            self._name("conv"): TensorDecl((C, self.taps_count), "vector", "conv"), self._name("conv_bias"): TensorDecl((C,), "vector", "bias"),
            self._name("x"): TensorDecl((R + 2 * N, C)),
            self._name("dt"): TensorDecl((C, R)), self._name("dt_bias"): TensorDecl((C,), "vector", "bias"),
            self._name("A_log"): TensorDecl((C, N), "vector", "bias"), self._name("D"): TensorDecl((C,), "vector", "norm"),
            self._name("o"): TensorDecl((D, C)),
        }

    def bind(self, tensors, dtype, device) -> None:
        super().bind(tensors, dtype, device)
        t = {which: tensors[self._name(which)] for which in self.names}
        self.in_proj = Linear(t["in"])
        self.x_proj = Linear(t["x"])
        self.dt_proj = Linear(t["dt"], t["dt_bias"])
        self.low_rank = ops.low_rank_weights(t["dt"])
        self.dt_bias = t["dt_bias"]
        self.out = Linear(t["o"])
        self.taps, self.conv_bias, self.D = t["conv"], t["conv_bias"], t["D"]
        # exp(dt A) is taken as 2^(dt A log2 e); a state's row holds all channels
        self.A2 = (-torch.exp(t["A_log"].to(torch.float64)) * math.log2(math.e)).to(torch.float32).t().contiguous()
        self._no_conv_state = None

    def _conv_state(self, cache):
        if "conv" in cache:
            return cache["conv"].state
        slots = cache["state"].state.shape[0]
        if self._no_conv_state is None or self._no_conv_state.shape[0] != slots:
            self._no_conv_state = torch.zeros((slots, self.inner, 0), dtype=torch.float32, device=self.device)
        return self._no_conv_state

    def scanned(self, h, ctx, cache) -> torch.Tensor:
        """y * silu(z) [rows, inner] in the activation dtype; the request's state and convolution memory move on."""
        both = self.in_proj.forward(h, out_dtype=torch.float32)
        short = self.dtype == torch.bfloat16
        x = ops.causal_conv(both[:, :self.inner], self.taps, self.conv_bias, self._conv_state(cache), ctx.row_seg, ctx.seg_row0,
                            ctx.seg_slot, ctx.num_segments, single_rows=ctx.all_decode, silu=True, rounded=short)
        x, rounded = x if short else (x, x)
        low = self.x_proj.forward(rounded, out_dtype=torch.float32)
        if ctx.all_decode and ctx.num_rows <= self.LOW_RANK_ROWS:
            return ops.selective_scan_low_rank(x, low, self.low_rank, self.dt_bias, both[:, self.inner:], self.A2, self.D, cache["state"].state,
                                               ctx.seg_slot, self.dtype)
        rank = torch.empty((low.shape[0], self.rank), dtype=self.dtype, device=low.device)
        ops.place_rows(low[:, :self.rank], rank)
        z = self.dt_proj.forward(rank, out_dtype=torch.float32)
        return ops.selective_scan(x, z, low[:, self.rank:], both[:, self.inner:], self.A2, self.D, cache["state"].state, ctx.seg_row0,
                                  ctx.seg_slot, ctx.num_segments, self.dtype, **self.chunk_arguments(ctx))

    def output(self, h, ctx, cache) -> torch.Tensor:
        return self.out.forward(self.scanned(h, ctx, cache), out_dtype=torch.float32)

    def forward(self, h, residual, ctx, cache):
        return self.out.accumulate(self.scanned(h, ctx, cache), residual, then=getattr(ctx, "upcoming_norm", None))
