"""Retention, a linear attention whose state decays by a constant (Sun et al., "Retentive Network: A Successor to Transformer for
Large Language Models").

With input h, ``heads`` heads with keys of ``key_dim`` and values of ``value_dim``:

* ``q, k, v = W_q h, W_k h, W_v h``; q and k rotated by the token's position (``position``, a rotation over
  any leading part of a head; None: none), then ``k <- k * key_dim^-1/2``;
* per head, state S [key_dim, value_dim]: ``S <- decay S + k v^T``, ``o = S^T q``, with ``decays[head]`` a constant;
* ``y = W_o (silu(W_g h) * concat_n(o_n / rms(o_n)))``, the root mean square per head, no weight.

The state, the powers of the decay, the rotation and the norm are float32 in both compute modes; q, k, v and the gate
enter as the float32 results of their projection.  A request's state row holds S, is cleared when the request is admitted
and carried from step to step, so a prompt may be cut anywhere.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence

import torch

from .. import ops
from ..errors import UnsupportedModelError
from ..weights.loader import TensorSpec
from .base import MIXERS, LayerCache, Mixer, PositionEncoding, StateSpec, StepContext


class Retention(Mixer):
    graph_safe = True        # slots and request boundaries are read on the device

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, decays: Sequence[float], eps: float,
                 position: Optional[PositionEncoding] = None, accumulate: bool = True, names=("q", "k", "v", "g", "o")):
        self.hidden_size, self.num_heads = int(hidden_size), int(num_heads)
        self.key_dim, self.value_dim = int(key_dim), int(value_dim)
        self.decays = tuple(float(d) for d in decays)
        self.eps, self.accumulate, self.position, self.names = float(eps), bool(accumulate), position, tuple(names)
        if len(self.decays) != self.num_heads or any(not 0.0 <= d <= 1.0 for d in self.decays):
            raise UnsupportedModelError(f"retention: {self.num_heads} heads need as many decays between 0 and 1, got {list(self.decays)}")
        if position is not None and (position.rotary_params() is None or getattr(position, "rotary_dim", self.key_dim) > self.key_dim):
            raise UnsupportedModelError("retention: positions enter by a rotation of queries and keys, or not at all")
        self.qk_size, self.v_size = self.num_heads * self.key_dim, self.num_heads * self.value_dim

    def tensor_specs(self) -> List[TensorSpec]:
        D, (q, k, v, g, o) = self.hidden_size, self.names
        return [TensorSpec(q, (self.qk_size, D)), TensorSpec(k, (self.qk_size, D)), TensorSpec(v, (self.v_size, D)),
                TensorSpec(g, (self.v_size, D)), TensorSpec(o, (D, self.v_size))]

    def cache_spec(self):
        return StateSpec((self.num_heads * self.key_dim * self.value_dim,), torch.float32)

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        # one projection with float32 results, rows [q | k | v | gate]
        self.w_in = torch.cat([tensors[n] for n in self.names[:4]], dim=0).contiguous()
        self.w_o = tensors[self.names[4]]
        self.decay = ops.decay_table(self.decays, device)
        if self.position is not None:
            self.position.load({}, dtype, device)

    def streamed_weights(self) -> List[torch.Tensor]:
        return [self.w_in, self.w_o]

    def forward(self, h: torch.Tensor, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> None:
        T, ws = h.shape[0], ctx.workspace
        rotary = self.position.rotary_params(ctx) if self.position is not None else None
        if ctx.all_decode:       # a tensor, or the pieces of a product split over k, which the one kernel of such a step adds
            proj = ops.qkv_projection(h, self.w_in, torch.float32, ws)
        else:
            proj = torch.empty((T, self.w_in.shape[0]), dtype=torch.float32, device=h.device)
            ops.gemm(proj, h, self.w_in, ws=ws)
        y = torch.empty((T, self.v_size), dtype=self.dtype, device=h.device)
        ops.retention(y, proj, rotary, self.decay, self.key_dim ** -0.5, self.eps, ctx, cache.state, self.num_heads, self.key_dim, self.value_dim)
        ops.gemm(x, y, self.w_o, accumulate=self.accumulate, may_defer=getattr(ctx, "may_defer", False), ws=ws)


MIXERS.register("retention", Retention)
