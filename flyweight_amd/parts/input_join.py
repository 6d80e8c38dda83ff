"""The model's input once more, in the middle of it: ahead of a run of layers the residual stream becomes a linear map of
itself and of the embedding output x0,

    x <- W_in [x; x0]

(W_in [hidden, 2 hidden], x's columns first). A model whose layers are passed several times joins its input ahead of every
pass. The product reads rows [x | x0] in the activation dtype that live as long as the step: x0's half is written once, and
the kernel that last sums into x ahead of a pass leaves x in the other half (:class:`JoinedRows`). The new x is float32.
"""

from __future__ import annotations

from typing import Dict

import torch

from ..kernels import ops
from ..weights.loader import TensorDecl
from .base import Part
from .linear import Linear


class JoinedRows:
    """The rows [x | x0] of one step: what a block is given as the reader of the residual stream after it. ``norm`` is
    None: a block that looks for a prepared norm finds none here."""
    norm = None

    def __init__(self, rows: torch.Tensor):
        self.rows = rows
        self.current = True             # whether x's half holds the stream as it is now

    @property
    def place(self) -> torch.Tensor:
        return self.rows[:, :self.rows.shape[1] // 2]

    def placed(self) -> "JoinedRows":
        """Returned by the block whose last sum has left x in its half."""
        self.current = True
        return self


class InputJoin(Part):
    graph_safe = True

    def __init__(self, spec):
        super().__init__(spec)
        self.hidden = int(spec["hidden_size"])
        self.tensor_name = str(spec["tensor"])

    def tensors(self) -> Dict[str, TensorDecl]:
        return {self.tensor_name: TensorDecl((self.hidden, 2 * self.hidden))}

    def bind(self, tensors, dtype, device) -> None:
        super().bind(tensors, dtype, device)
        self.map = Linear(tensors[self.tensor_name])

    def start(self, x: torch.Tensor) -> JoinedRows:
        """The step's rows, from the embedding output (float32): both halves hold it, x being x0 at the model's start."""
        rows = torch.empty((x.shape[0], 2 * self.hidden), dtype=self.dtype, device=x.device)
        return JoinedRows(ops.place_rows(x, rows, twice=True))

    def forward(self, x: torch.Tensor, joined: JoinedRows) -> torch.Tensor:
        """The new residual stream, float32 rows of its own."""
        if not joined.current:
            ops.place_rows(x, joined.rows)
        joined.current = False          # of the stream as it will be from here on
        return self.map.forward(joined.rows, out_dtype=torch.float32)
