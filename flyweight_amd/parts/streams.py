"""A residual stream of several rows side by side ("hyper-connections": Zhu, Huang et al., "Hyper-Connections").

Instead of one x there are ``streams`` rows x_1 .. x_S, float32 [rows, streams, hidden], all equal to the embedding output at
the start. A sublayer reads one weighted sum of them through its norm and writes to all of them while they mix:

    u = sum_s in[s] x_s;   y = ls * sublayer(norm(u));   x_t <- sum_s mix[s, t] x_s + out[t] y

(all t from the old rows; ls is a vector, the sublayer's own scale per channel). What stands between two sublayers, the
join of one and the read of the next, is one kernel; so are two branches brought to unit size and summed, and the outputs
of a token's experts, where a sublayer leaves those (:class:`SublayerOutput`).

:class:`StreamReader` is what reads the streams next: the weights ``in`` of a sublayer, or plain ones for the model's end, and
the norm behind them. :class:`StreamConnection` is one sublayer's own tensors, ``in``, ``mix`` ([from, to]), ``out`` and ``ls``.
"""

from __future__ import annotations

from typing import Dict, Optional

import torch

from ..config.spec import ConfigError
from ..kernels import ops
from ..weights.loader import TensorDecl
from .base import Norm, Part, SublayerOutput


class StreamRows:
    """What the kernel that last changed the streams has already formed for ``reader``. (``norm`` is None: a block that
    looks for a prepared norm finds none here.)"""
    norm = None

    def __init__(self, reader: "StreamReader", activations: torch.Tensor):
        self.reader, self.activations = reader, activations


class StreamReader:
    """A weighted sum of the streams (``weights`` None: their plain sum) and the norm that reads it."""

    def __init__(self, norm: Norm):
        self.norm = norm
        self.weights: Optional[torch.Tensor] = None

    def _norm_arguments(self) -> dict:
        if not hasattr(self.norm, "tanh_parameters"):
            return {}
        weight, bias, alpha = self.norm.tanh_parameters()
        return {"weight": weight, "bias": bias, "alpha": alpha}

    def read(self, x: torch.Tensor, ctx, row_index: Optional[torch.Tensor] = None) -> torch.Tensor:
        """The norm's output for the streams' rows, in the activation dtype."""
        given = self._norm_arguments()
        if given:
            return ops.stream_read(x, self.weights, self.norm.dtype, kind=ops.NEXT_TANH, row_index=row_index, **given)
        return self.norm.forward(ops.stream_read(x, self.weights, torch.float32, row_index=row_index), ctx)

    def take(self, x: torch.Tensor, ctx, prepared) -> torch.Tensor:
        """``read``, or what was prepared for this very reader."""
        if isinstance(prepared, StreamRows) and prepared.reader is self and prepared.activations.shape[0] == x.shape[0]:
            return prepared.activations
        return self.read(x, ctx)

    def join_arguments(self) -> dict:
        """What a kernel that joins the streams is told about this reader."""
        given = self._norm_arguments()
        if given:
            return {"next_kind": ops.NEXT_TANH, "next_in": self.weights, "next_dtype": self.norm.dtype,
                    **{"next_" + key: value for key, value in given.items()}}
        return {"next_kind": ops.NEXT_SUM, "next_in": self.weights, "next_dtype": torch.float32}

    def finish(self, formed: torch.Tensor, ctx) -> torch.Tensor:
        """What the join left for this reader, through the norm where the kernel does not know it."""
        return formed if hasattr(self.norm, "tanh_parameters") else self.norm.forward(formed, ctx)


class StreamConnection(Part):
    """One sublayer's place in the streams. ``scale_tensor``: the name of ls (None: ones)."""
    graph_safe = True

    def __init__(self, spec):
        super().__init__(spec)
        self.hidden = int(spec["hidden_size"])
        self.streams = int(spec["streams"])
        self.scale_tensor = spec.get("scale_tensor")
        if not 1 <= self.streams <= ops.MAX_STREAMS:
            raise ConfigError(f"a residual stream of {self.streams} rows (1..{ops.MAX_STREAMS})")

    def tensors(self) -> Dict[str, TensorDecl]:
        S, p = self.streams, self.prefix
        declared = {p + "in": TensorDecl((S,), "vector", "share"), p + "out": TensorDecl((S,), "vector", "norm"),
                    p + "mix": TensorDecl((S, S), "vector", "unit")}
        if self.scale_tensor is not None:
            declared[self.scale_tensor] = TensorDecl((self.hidden,), "vector", "norm")
        return declared

    def bind(self, tensors, dtype, device) -> None:
        super().bind(tensors, dtype, device)
        self.weights_in, self.weights_out, self.mix = (tensors[self.prefix + n] for n in ("in", "out", "mix"))
        self.scale = tensors[self.scale_tensor] if self.scale_tensor is not None else torch.ones((self.hidden,), dtype=torch.float32, device=device)

    def join(self, x: torch.Tensor, y: SublayerOutput, reader: Optional[StreamReader], ctx) -> Optional[torch.Tensor]:
        """The sublayer's output joins the streams (in place); returns what ``reader`` sees of them (None for no reader)."""
        formed = ops.stream_join_(x, self.scale, self.mix, self.weights_out, y.rows, branches=y.branches, chosen=y.chosen,
                                  **(reader.join_arguments() if reader is not None else {}))
        return None if reader is None else reader.finish(formed, ctx)
