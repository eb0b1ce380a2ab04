"""Normalisation parts: RMS norm, and layer norm with weight and bias.

Formula (include/photon/ops/kernels/rmsnorm_kernel.hpp:55-87): mean of squares over
the row, ``rms = sqrt(mean + eps)`` with eps inside the root, ``y = w * (x / rms)``;
no mean-centring, no bias.  A model that stores its weights around zero uses ``offset + w``.  Sum, root and scaling run in float32; the result is
rounded once to the compute dtype.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional

import torch

from .. import ops
from ..weights.loader import TensorSpec
from .base import NORMS, Norm


# Key in a step's ``scratch``: (streams, a sublayer's result, the numbers it joins them by) - an update of streams that run
# side by side, left to whoever reads them next.
LEFT_UPDATE = "update of the streams left to their next reader"

# Key in a step's ``scratch``: a ``LeftJoin``, a sublayer's result that joins the stream through a norm of its own and has been left
# to the stream's next reader, which makes its own norm in the same pass.
LEFT_JOIN = "result left to the stream's next reader"


@dataclass
class LeftJoin:
    x: torch.Tensor                  # the stream
    y: torch.Tensor                  # the result (its product may still be in pieces in the workspace)
    weight: torch.Tensor             # the norm it goes through, float32
    eps: float
    choices: Optional[object] = None  # ops.LeftChoices: the result is still a sum over experts' rows

    def apply(self, ws, nxt=None, next_eps: float = 0.0, dtype=None, rows=None):
        return ops.rms_join(self.x, self.y, self.weight, self.eps, nxt, next_eps, dtype, rows, ws, self.choices)


def take_left_join(x: torch.Tensor, ctx) -> Optional[LeftJoin]:
    left = ctx.scratch.get(LEFT_JOIN) if ctx is not None else None
    if left is None or left.x is not x:
        return None
    return ctx.scratch.pop(LEFT_JOIN)


def settle_left_join(x: torch.Tensor, ctx) -> None:
    """Apply a result that was left for ``x``, if there is one (before a reader that knows nothing of it)."""
    left = take_left_join(x, ctx)
    if left is not None:
        left.apply(ctx.workspace)


class RMSNorm(Norm):
    consumes_deferred = True   # reads the stream through ops.rmsnorm, which adds a pending update
    takes_left_join = True     # and a result that a sandwich block has left
    graph_safe = True

    def __init__(self, dim: int, eps: float, offset: float = 0.0, tensor_name: str = "weight", mult: float = 1.0):
        """``offset``: what is added to the stored weight (1.0 for weights stored around zero, used
        as 1 + w); the sum is made and kept in float32.  ``mult``: a factor on the normalised row, made part of
        the float32 weight (for a head whose logits carry a factor).  ``tensor_name``: the weight's name
        after the part's prefix (may be empty: the prefix is the name)."""
        self.dim = int(dim)
        self.eps = float(eps)
        self.offset, self.mult = float(offset), float(mult)
        self.tensor_name = tensor_name
        self.weight: Optional[torch.Tensor] = None

    def tensor_specs(self) -> List[TensorSpec]:
        return [TensorSpec(self.tensor_name, (self.dim,), "norm_zero" if self.offset else "norm")]

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        self.weight = tensors[self.tensor_name]
        if self.offset or self.mult != 1.0:
            self.weight = ((self.weight.to(torch.float32) + self.offset) * self.mult).contiguous()

    def weight_f32(self) -> torch.Tensor:
        """The weight as the kernels that want float32 weights take it (made once)."""
        if getattr(self, "_w32", None) is None:
            self._w32 = self.weight.to(torch.float32).contiguous()
        return self._w32

    def forward(self, x: torch.Tensor, ctx=None, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        left = take_left_join(x, ctx)
        if left is not None:
            return left.apply(ctx.workspace, self.weight_f32(), self.eps, self.dtype, rows)
        m = x.shape[0] if rows is None else rows.shape[0]
        out = torch.empty((m, self.dim), dtype=self.dtype, device=x.device)
        ops.rmsnorm(out, x, self.weight, self.eps, rows, ws=ctx.workspace if ctx is not None else None)
        return out


NORMS.register("rmsnorm", RMSNorm)


class StreamSumRMSNorm(RMSNorm):
    """The RMS norm of the sum of several streams that run side by side (``x`` is [T, streams, D]), read from them in the
    norm's own pass.  An update that a block of such streams has left to the next reader (``HyperConnectionBlock``) is
    applied on the way."""

    consumes_deferred = takes_left_join = False

    def __init__(self, dim: int, eps: float, streams: int, offset: float = 0.0, tensor_name: str = "weight"):
        super().__init__(dim, eps, offset, tensor_name)
        self.streams = int(streams)

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        self.ones = torch.ones(self.streams, dtype=torch.float32, device=device)

    def forward(self, x: torch.Tensor, ctx=None, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        left = ctx.scratch.pop(LEFT_UPDATE, None) if ctx is not None else None
        y, post = (left[1], left[2]) if left is not None and left[0] is x else (None, None)
        return ops.hyper_streams(x, y=y, post=post, h_dtype=self.dtype, read=self.ones, norm=self.weight_f32(), eps=self.eps, rows=rows,
                                 ws=ctx.workspace if ctx is not None else None)


NORMS.register("stream_sum_rmsnorm", StreamSumRMSNorm)


class LayerNorm(Norm):
    """Layer norm with weight and bias: ``(x - mean) / sqrt(variance + eps) * w + b``, the variance the mean of the
    squared deviations; mean, variance and scaling in float32, rounded once to the compute dtype.
    ``tensor_name``: the weight's name after the part's prefix (may be empty: the prefix is the name); the bias is
    that name plus ``bias_suffix``."""

    graph_safe = True

    def __init__(self, dim: int, eps: float, tensor_name: str = "weight", bias_suffix: str = ".b"):
        self.dim, self.eps = int(dim), float(eps)
        self.tensor_name, self.bias_name = tensor_name, tensor_name + bias_suffix
        self.weight: Optional[torch.Tensor] = None
        self.bias: Optional[torch.Tensor] = None

    def tensor_specs(self) -> List[TensorSpec]:
        return [TensorSpec(self.tensor_name, (self.dim,), "norm"), TensorSpec(self.bias_name, (self.dim,), "small_bias")]

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        self.weight = tensors[self.tensor_name].to(torch.float32).contiguous()
        self.bias = tensors[self.bias_name].to(torch.float32).contiguous()

    def weight_bias_f32(self):
        """(weight, bias) as the kernels that fold this norm into another pass take them."""
        return self.weight, self.bias

    def forward(self, x: torch.Tensor, ctx=None, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        m = x.shape[0] if rows is None else rows.shape[0]
        out = torch.empty((m, self.dim), dtype=self.dtype, device=x.device)
        ops.layer_norm(out, x, self.weight, self.bias, self.eps, rows)
        return out


NORMS.register("layernorm", LayerNorm)
