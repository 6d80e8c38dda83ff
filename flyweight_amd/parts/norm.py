"""RMS norm: y = x * rsqrt(mean(x^2) + eps) * w, sums in float32; the weight multiplies
directly (native/include/flyweight_v2_qwen_kernels.hpp:425-447 with one_centered = 0).
Layer norm: the row's mean is taken off first, y = (x - m) * rsqrt(mean((x - m)^2) + eps) * w, plus a bias vector where
the design has one.
The tanh norm takes no statistics of the row: y = tanh(alpha x) w + b, alpha one number."""

from __future__ import annotations

from typing import Dict, NamedTuple, Optional

import torch

from ..kernels import ops
from ..weights.loader import TensorDecl
from .base import Norm, register_norm


class RowNorm(NamedTuple):
    """A norm over a whole row as a kernel applies it beside other work on the row: v / sqrt(mean(v^2) + eps) * weight
    (+ bias), v the row, or with ``centered`` the row less its mean."""
    weight: torch.Tensor
    eps: float
    centered: bool
    bias: Optional[torch.Tensor] = None


class Prepared:
    """What the product that last added to the residual stream left for the norm after it:
    ``activations`` bfloat16 [rows, size] = x * w of that norm and ``squares`` [tiles, 16],
    partial sums of x^2 per row, from which a product's kernel forms the row's 1/rms itself."""

    def __init__(self, norm: Norm, activations: torch.Tensor, squares: torch.Tensor):
        self.norm, self.activations, self.squares = norm, activations, squares


class NormedRows:
    """Rows that the kernel which last changed the residual stream has already passed through ``norm``
    (``activations``, in the activation dtype): whoever is about to apply that very norm to those
    very rows takes them instead."""

    def __init__(self, norm: Norm, activations: torch.Tensor):
        self.norm, self.activations = norm, activations


class LazyNorm:
    """A norm that has not run yet: the rows ``x`` (optionally gathered through ``row_index``)
    and the norm to apply. A product that can apply an RMS norm in its own kernel takes it as
    it is (``rms_parameters``, or ``prepared`` when the rows' producer already did most of it);
    anything else calls ``tensor()``, which runs the norm once."""

    def __init__(self, norm: Norm, x: torch.Tensor, ctx, row_index: Optional[torch.Tensor] = None,
                 prepared: Optional[Prepared] = None):
        self.norm, self.x, self.ctx, self.row_index = norm, x, ctx, row_index
        # only what was made for this very norm and these rows counts
        ok = prepared is not None and prepared.norm is norm and row_index is None \
            and prepared.activations.shape == x.shape
        self._tensor = None
        if ok and isinstance(prepared, NormedRows):     # the norm has run already
            self._tensor, ok = prepared.activations, False
        self.prepared = prepared if ok else None

    @property
    def rows(self) -> int:
        return self.row_index.numel() if self.row_index is not None else self.x.shape[0]

    @property
    def dtype(self) -> torch.dtype:
        return self.norm.dtype

    def rms_parameters(self):
        """(weight, eps, one_centered) if the norm is a plain RMS norm, else None."""
        return self.norm.rms_parameters() if hasattr(self.norm, "rms_parameters") else None

    def tensor(self) -> torch.Tensor:
        if self._tensor is None:
            self._tensor = self.norm.forward(self.x, self.ctx, row_index=self.row_index)
        return self._tensor


@register_norm("rmsnorm")
class RMSNorm(Norm):
    graph_safe = True

    def __init__(self, spec):
        super().__init__(spec)
        self.size = int(spec["size"])
        self.eps = float(spec["eps"])
        self.one_centered = bool(spec.get("one_centered", False))

    @property
    def tensor_name(self) -> str:
        """``prefix`` + "weight", unless the layout names the tensor itself (``tensor``)."""
        return self.spec.get("tensor") or self.prefix + "weight"

    def tensors(self) -> Dict[str, TensorDecl]:
        # a weight stored around zero (used as 1 + w) starts around zero
        return {self.tensor_name: TensorDecl((self.size,), role="vector", init="bias" if self.one_centered else "norm")}

    def bind(self, tensors, dtype, device) -> None:
        super().bind(tensors, dtype, device)
        self.weight = tensors[self.tensor_name]

    def rms_parameters(self):
        return self.weight, self.eps, self.one_centered

    def row_norm(self):
        """The norm for a kernel that applies it beside other work on the row, or None where the norm is
        not of that plain form."""
        return None if self.one_centered else RowNorm(self.weight, self.eps, False)

    def forward(self, x: torch.Tensor, ctx, row_index: Optional[torch.Tensor] = None) -> torch.Tensor:
        return ops.rmsnorm_rows(x, self.weight, self.eps, self.dtype, row_index=row_index,
                                one_centered=self.one_centered)


@register_norm("layernorm")
class LayerNorm(Norm):
    """(x - mean) / sqrt(variance + eps) * w, the variance the mean of the squared deviations; with ``bias`` + b, the
    tensor of the weight's name with ".b" behind it."""
    graph_safe = True

    def __init__(self, spec):
        super().__init__(spec)
        self.size = int(spec["size"])
        self.eps = float(spec["eps"])
        self.has_bias = bool(spec.get("bias", False))

    @property
    def tensor_name(self) -> str:
        return self.spec.get("tensor") or self.prefix + "weight"

    def tensors(self) -> Dict[str, TensorDecl]:
        declared = {self.tensor_name: TensorDecl((self.size,), role="vector", init="norm")}
        if self.has_bias:
            declared[self.tensor_name + ".b"] = TensorDecl((self.size,), role="vector", init="bias")
        return declared

    def bind(self, tensors, dtype, device) -> None:
        super().bind(tensors, dtype, device)
        self.weight = tensors[self.tensor_name]
        self.bias = tensors[self.tensor_name + ".b"] if self.has_bias else None

    def row_norm(self):
        return RowNorm(self.weight, self.eps, True, self.bias)

    def forward(self, x: torch.Tensor, ctx, row_index: Optional[torch.Tensor] = None) -> torch.Tensor:
        return ops.layernorm_rows(x, self.weight, self.eps, self.dtype, row_index=row_index, bias=self.bias)


@register_norm("tanh")
class TanhNorm(Norm):
    """tanh(alpha x) * w + b per channel (Dynamic Tanh: Zhu, Chen, He, LeCun and Liu, "Transformers without Normalization"). The
    scalar and the bias are the tensors of the weight's name with ".alpha" and ".b" behind it. A kernel that works on some
    channels of a row alone can apply it (``tanh_parameters``)."""
    graph_safe = True

    def __init__(self, spec):
        super().__init__(spec)
        self.size = int(spec["size"])

    @property
    def tensor_name(self) -> str:
        return self.spec.get("tensor") or self.prefix + "weight"

    def tensors(self) -> Dict[str, TensorDecl]:
        return {self.tensor_name: TensorDecl((self.size,), role="vector", init="norm"),
                self.tensor_name + ".b": TensorDecl((self.size,), role="vector", init="bias"),
                self.tensor_name + ".alpha": TensorDecl((), role="vector", init="norm")}

    def bind(self, tensors, dtype, device) -> None:
        super().bind(tensors, dtype, device)
        self.weight = tensors[self.tensor_name]
        self.bias = tensors[self.tensor_name + ".b"]
        self.alpha = tensors[self.tensor_name + ".alpha"]

    def tanh_parameters(self):
        return self.weight, self.bias, self.alpha

    def forward(self, x: torch.Tensor, ctx, row_index: Optional[torch.Tensor] = None) -> torch.Tensor:
        return ops.stream_read(x.unsqueeze(1), None, self.dtype, kind=ops.NEXT_TANH, weight=self.weight, bias=self.bias, alpha=self.alpha,
                               row_index=row_index)
