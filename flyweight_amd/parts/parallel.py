"""Mixers side by side: every branch reads the same input and the outputs are mixed with fixed
weights, out = sum_i scale_i * branch_i(h). A branch is any registered mixer that can give its
output as rows of its own (``output(h, ctx, cache)``); each keeps its own cache entry, so the
whole asks the cache manager for a mapping branch name -> that branch's need. A branch may have an RMS norm
of its own that its output passes first, out = sum_i scale_i * norm_i(branch_i(h)).
"""

from __future__ import annotations

from typing import Dict, List, Tuple

import torch

from ..config.spec import ConfigError
from ..kernels import ops
from ..weights.loader import TensorDecl
from .base import Mixer, SublayerOutput, build_part, register_mixer


@register_mixer("parallel_branches")
class ParallelBranches(Mixer):
    """``branches``: a sequence of (name, PartSpec of a mixer, scale). ``norms``: branch name -> PartSpec of the RMS norm (plain
    weight) on its output; either every branch has one or none."""

    def __init__(self, spec):
        super().__init__(spec)
        self.branches: List[Tuple[str, Mixer, float]] = []
        for name, part, scale in spec["branches"]:
            mixer = build_part("mixer", part)
            if not hasattr(mixer, "output"):
                raise ConfigError(f"mixer '{part.kind}' cannot stand in a parallel arrangement: it has no output()")
            self.branches.append((str(name), mixer, float(scale)))
        if not self.branches:
            raise ConfigError("a parallel arrangement needs at least one branch")
        if len({name for name, _, _ in self.branches}) != len(self.branches):
            raise ConfigError("the branches of a parallel arrangement need different names")
        self.norms = {str(name): build_part("norm", part) for name, part in dict(spec.get("norms") or {}).items()}
        if self.norms and set(self.norms) != {name for name, _, _ in self.branches}:
            raise ConfigError("either every branch of a parallel arrangement has a norm on its output, or none")
        if any(not hasattr(norm, "rms_parameters") or norm.one_centered for norm in self.norms.values()):
            raise ConfigError("the norms on the branches of a parallel arrangement are RMS norms with a plain weight")

    @property
    def graph_safe(self) -> bool:
        return all(mixer.graph_safe and getattr(getattr(mixer, "position", None), "graph_safe", True)
                   for _, mixer, _ in self.branches)

    def tensors(self) -> Dict[str, TensorDecl]:
        declared: Dict[str, TensorDecl] = {}
        for _, mixer, _ in self.branches:
            declared.update(mixer.tensors())
        for norm in self.norms.values():
            declared.update(norm.tensors())
        return declared

    def bind(self, tensors, dtype, device) -> None:
        super().bind(tensors, dtype, device)
        for _, mixer, _ in self.branches:
            mixer.bind(tensors, dtype, device)
        for norm in self.norms.values():
            norm.bind(tensors, dtype, device)

    def cache_need(self):
        return {name: mixer.cache_need() for name, mixer, _ in self.branches}

    # a branch's index arrays travel with the step as any part's do
    def sub_parts(self):
        return [mixer for _, mixer, _ in self.branches]

    def output_terms(self, h, ctx, cache) -> List[Tuple[torch.Tensor, float]]:
        """[(float32 rows, scale)]: the mixer's output is their weighted sum, which the caller forms
        where it reads them."""
        terms = [(mixer.output(h, ctx, cache[name]), scale) for name, mixer, scale in self.branches]
        if self.norms:
            norms = [self.norms[name].rms_parameters() for name, _, _ in self.branches]
            terms = [(ops.rmsnorm_rows(rows, weight, eps, torch.float32), scale) for (rows, scale), (weight, eps, _) in zip(terms, norms)]
        return terms

    def joined_output(self, h, ctx, cache) -> SublayerOutput:
        """The same for a kernel that joins it to the residual stream: two branches with norms are left to that kernel."""
        if len(self.branches) == 2 and self.norms:
            (a, _, scale_a), (b, _, scale_b) = self.branches
            (weight_a, eps_a, _), (weight_b, eps_b, _) = (self.norms[name].rms_parameters() for name in (a, b))
            if eps_a == eps_b:
                rows_a, rows_b = (mixer.output(h, ctx, cache[name]) for name, mixer, _ in self.branches)
                return SublayerOutput(rows_a, branches=(rows_b, weight_a, weight_b, scale_a, scale_b, eps_a))
        terms = self.output_terms(h, ctx, cache)
        total = terms[0][0] * terms[0][1]
        for rows, scale in terms[1:]:
            total.add_(rows, alpha=scale)
        return SublayerOutput(total)

    def forward(self, h, residual, ctx, cache):
        for rows, scale in self.output_terms(h, ctx, cache):
            residual.add_(rows, alpha=scale)
        return None
