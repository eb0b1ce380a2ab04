"""Token shift: what a sublayer reads is moved, per feature, towards what the token before read:

    h <- h + (h_before - h) * share

h_before is the unshifted h of the neighbour on the left; a sequence starts with a neighbour of zeros.  A
request's state row holds the unshifted h of its last token in float32, so a prompt may be cut anywhere.

The arrangement that uses it makes h, the shift and the state update in one kernel (``ops.hyper_streams``); this part
holds the weights and declares the state.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..weights.loader import TensorSpec
from .base import Part, StateSpec


class TokenShift(Part):
    graph_safe = True        # slots and request boundaries are read on the device

    def __init__(self, hidden_size: int, tensor_name: str = "shift"):
        self.hidden_size, self.tensor_name = int(hidden_size), tensor_name
        self.share: Optional[torch.Tensor] = None

    def tensor_specs(self) -> List[TensorSpec]:
        return [TensorSpec(self.tensor_name, (self.hidden_size,), "share")]

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        self.share = tensors[self.tensor_name].to(torch.float32).contiguous()

    # what the cache planner asks of whoever keeps something per request
    def cache_spec(self):
        return StateSpec((self.hidden_size,), torch.float32)

    def step_planner(self, page_size: int):
        return None
