"""Attention whose weights are sigmoids and whose heads mix them, over the paged cache.

q = W_q h, k = W_k h, v = W_v h, heads of ``head_dim`` channels (values ``v_head_dim``), query head i on key/value head
i // (num_heads / num_kv_heads); with ``qk_norm`` every head of q and k is divided by its root mean square,
x / sqrt(mean(x^2) + eps), no weight. No positions. For row i and every key j it sees (causal, optionally the last ``window``
keys only, itself among them)

    a_g(i, j) = sigmoid(q_g . k * softmax_scale + b_g)              (``names["bias"]``, [heads]; each key on its own)
    o_h(i)    = sum_j (sum_g M[h, g] a_g(i, j)) v_j                 (``names["mix"]``, [heads, heads]; v of h's own group)

and out = W_o (o * sigmoid(W_g h)), a gate per channel (``output_gate``). Scores, sigmoids and the mix are float32. Nothing
is summed over the keys but the values, so parts of a row's keys simply add up. What reads h is one operand, [q | k | v | gate]
rows, whose float32 sums the kernels read as they are.
"""

from __future__ import annotations

from typing import Dict

import torch

from ..cache.needs import PagedKV
from ..config.spec import ConfigError
from ..kernels import ops
from ..weights.loader import TensorDecl
from .attention import QueryTileArrays
from .base import Mixer, register_mixer
from .linear import Linear

_DEFAULT_NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "mix": "talk", "bias": "pb"}


@register_mixer("sigmoid_attention")
class SigmoidAttention(QueryTileArrays, Mixer):
    graph_safe = True
    # Up to this many rows a decode step forms queries and keys inside the attention kernel.
    FUSED_DECODE_ROWS = 16

    def __init__(self, spec):
        super().__init__(spec)
        self.hidden = int(spec["hidden_size"])
        self.num_heads = int(spec["num_heads"])
        self.num_kv_heads = int(spec["num_kv_heads"])
        self.head_dim = int(spec["head_dim"])
        self.v_head_dim = int(spec.get("v_head_dim") or self.head_dim)
        self.scale = float(spec.get("softmax_scale", self.head_dim ** -0.5))
        self.window = None if spec.get("window") is None else int(spec["window"])
        self.qk_norm = bool(spec.get("qk_norm", True))
        self.eps = float(spec.get("qk_norm_eps", 1e-6))
        self.gated = bool(spec.get("output_gate", True))
        self.names = {**_DEFAULT_NAMES, **dict(spec.get("names", {}))}
        if min(self.num_heads, self.num_kv_heads, self.head_dim, self.v_head_dim) < 1 or self.num_heads % self.num_kv_heads:
            raise ConfigError(f"{self.num_heads} heads are not a multiple of {self.num_kv_heads} kv heads, or a size is not positive")
        if self.num_heads > ops.SIGMOID_MAX_HEADS or max(self.head_dim, self.v_head_dim) > ops.MAX_PLAIN_HEAD_DIM:
            raise ConfigError(f"{self.num_heads} heads of {self.head_dim} / {self.v_head_dim} channels exceed the kernels' limits of "
                              f"{ops.SIGMOID_MAX_HEADS} heads and {ops.MAX_PLAIN_HEAD_DIM} channels")
        if self.window is not None and self.window < 1:
            raise ConfigError("an attention window must be positive (or None for all keys)")

    def cache_need(self):
        return PagedKV(self.num_kv_heads, self.head_dim, self.window, None if self.v_head_dim == self.head_dim else self.v_head_dim)

    def _name(self, which: str) -> str:
        return self.prefix + self.names[which]

    def tensors(self) -> Dict[str, TensorDecl]:
        D, H, G, d, dv = self.hidden, self.num_heads, self.num_kv_heads, self.head_dim, self.v_head_dim
        declared = {
            self._name("q"): TensorDecl((H * d, D)), self._name("k"): TensorDecl((G * d, D)), self._name("v"): TensorDecl((G * dv, D)),
            self._name("mix"): TensorDecl((H, H), "vector", "conv"), self._name("bias"): TensorDecl((H,), "vector", "bias"),
            self._name("o"): TensorDecl((D, H * dv)),
        }
        if self.gated:
            declared[self._name("g")] = TensorDecl((H * dv, D))
        return declared

    def bind(self, tensors, dtype, device) -> None:
        super().bind(tensors, dtype, device)
        self.qkvg = Linear(torch.cat([tensors[self._name(n)] for n in (("q", "k", "v", "g") if self.gated else ("q", "k", "v"))], dim=0))
        self.out = Linear(tensors[self._name("o")])
        self.mix, self.bias = tensors[self._name("mix")], tensors[self._name("bias")]
        # the per-head norm has no weight; the kernel that norms for a prompt multiplies by this one
        self.unit_weight = torch.ones((self.head_dim,), dtype=torch.float32, device=device) if self.qk_norm else None

    def uses_query_tiles(self) -> bool:
        return getattr(self, "dtype", None) == torch.bfloat16 and ops.sigmoid_attention_is_tiled(self.num_heads, self.head_dim, self.v_head_dim)

    def mixing_flops(self, rows: int, keys_before: int = 0) -> int:
        """Scores, the mix and weighted sums for rows that follow ``keys_before`` cached tokens."""
        window = self.window or (keys_before + rows)
        full = max(0, min(rows, window - keys_before - 1))      # rows that still see fewer than a window
        pairs = full * keys_before + full * (full + 1) // 2 + (rows - full) * window
        return 2 * self.num_heads * (self.head_dim + self.v_head_dim + self.num_heads) * pairs

    def attend(self, h, ctx, cache) -> torch.Tensor:
        """The gated heads [rows, heads * v_head_dim] in the activation dtype; the step's keys and values join the cache."""
        H, G, d, dv = self.num_heads, self.num_kv_heads, self.head_dim, self.v_head_dim
        projected = self.qkvg.forward(h, out_dtype=torch.float32)
        width = (H + G) * d + G * dv
        qkv, gate = projected[:, :width], projected[:, width:] if self.gated else None
        window = self.window or 0
        if ctx.all_decode and ctx.num_rows <= self.FUSED_DECODE_ROWS and self.uses_query_tiles():
            # a few single-token segments on the matrix cores: norm, cache write, attention and gate in one kernel
            return ops.sigmoid_attention_decode(
                H, G, d, dv, cache.k_pages, cache.v_pages, cache.block_table, ctx.row_seg, ctx.row_pos, self.scale, window, self.bias, self.mix,
                ctx.max_context, gate=gate, qkv=qkv, qk_norm=self.qk_norm, eps=self.eps, write_kv=cache.writes)
        q = ops.qk_norm_rope_kv_write(qkv, H, G, d, self.unit_weight, self.unit_weight, self.eps, None, None, 0, cache.k_pages, cache.v_pages,
                                      cache.block_table, ctx.row_seg, ctx.row_pos, write_kv=cache.writes, v_dim=dv)
        own = ctx.step_arrays(self) if self.step_arrays_key() is not None else {}
        return ops.sigmoid_attention(q, H, G, d, dv, cache.k_pages, cache.v_pages, cache.block_table, ctx, self.scale, window, self.bias, self.mix,
                                     gate, tile_seg=own.get("tile_seg"), tile_row0=own.get("tile_row0"))

    def output(self, h, ctx, cache) -> torch.Tensor:
        """The mixer's output as float32 rows of its own (for arrangements that do something to it
        before it joins the residual stream)."""
        return self.out.forward(self.attend(h, ctx, cache), out_dtype=torch.float32)

    def forward(self, h, residual, ctx, cache):
        return self.out.accumulate(self.attend(h, ctx, cache), residual, then=getattr(ctx, "upcoming_norm", None))
