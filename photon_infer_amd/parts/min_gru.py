"""minGRU: a recurrence of one number per feature whose gate and candidate do not look at the state
(Feng et al., "Were RNNs All We Needed?").

With input h: ``z = sigmoid(Wz h + bz)``, ``u = Wx h + bx``; the candidate is ``c = u + 1/2`` where u >= 0 and
``sigmoid(u)`` below; per feature ``S <- (1 - z) S + z c``; the result is ``Wo (S * silu(Wg h))``.

Everything between the projections and the one rounding of ``S * silu(Wg h)`` is float32 in both compute modes.  A
request's state row holds S, is cleared when the request is admitted and carried from step to step, so a prompt may be
cut anywhere.
"""
from __future__ import annotations

from typing import Dict, List

import torch

from .. import ops
from ..weights.loader import TensorSpec
from .base import MIXERS, LayerCache, Mixer, StateSpec, StepContext


class MinGRU(Mixer):
    graph_safe = True        # slots and request boundaries are read on the device

    def __init__(self, hidden_size: int, width: int, bias_suffix: str = ".b", accumulate: bool = True):
        self.hidden_size, self.width = int(hidden_size), int(width)
        self.bias_suffix, self.accumulate = bias_suffix, bool(accumulate)

    def tensor_specs(self) -> List[TensorSpec]:
        D, W, b = self.hidden_size, self.width, self.bias_suffix
        return [TensorSpec("z", (W, D)), TensorSpec("z" + b, (W,), "bias"), TensorSpec("x", (W, D)), TensorSpec("x" + b, (W,), "small_bias"),
                TensorSpec("g", (W, D)), TensorSpec("o", (D, W))]

    def cache_spec(self):
        return StateSpec((self.width,), torch.float32)

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        mats = [tensors[n] for n in ("z", "x", "g")]
        common = torch.float32 if any(m.dtype == torch.float32 for m in mats) else mats[0].dtype
        self.w_in = torch.cat([m.to(common) for m in mats], dim=0).contiguous()      # one projection, rows [z | x | g]
        self.bias = torch.cat([tensors[n + self.bias_suffix].to(torch.float32) for n in ("z", "x")]).contiguous()
        self.w_o = tensors["o"]

    def streamed_weights(self) -> List[torch.Tensor]:
        return [self.w_in, self.w_o]

    def forward(self, h: torch.Tensor, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> None:
        # float32 results: a tensor, or - where the product was split over k - its pieces, which the next kernel adds
        proj = ops.qkv_projection(h, self.w_in, torch.float32, ctx.workspace)
        act = torch.empty((h.shape[0], self.width), dtype=self.dtype, device=h.device)
        ops.min_gru(act, proj, self.bias, ctx, cache.state, self.width)
        ops.gemm(x, act, self.w_o, accumulate=self.accumulate, may_defer=getattr(ctx, "may_defer", False), ws=ctx.workspace)


MIXERS.register("min_gru", MinGRU)
