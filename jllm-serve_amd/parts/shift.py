"""Token shift: what a sublayer reads, h_t, is replaced by h_t + shift (h_(t-1) - h_t), element by element with a learned
vector, h_(t-1) being the same request's row before (as it was before its own replacement; zeros before the first token).
The last row of a request is its state, fp32 [width], in the cache manager's state slots.

In a step whose requests bring one row each (decoding) the shift rides on the launch that writes the rows
(``ops.rms_seam``); otherwise it is a launch of its own, and one more that moves the states on."""
from __future__ import annotations

import torch

from ..cache.manager import StateSpec
from ..kernels import ops
from ..weights.loader import WeightSpec
from .base import BuildContext, Part


class TokenShift(Part):
    def __init__(self, name: str, build: BuildContext):
        self.name = name
        self.width = build.hidden
        self.out_dtype = build.dtype
        self.shift = None

    def weight_specs(self):
        return [WeightSpec(self.name, (self.width,), init="bias")]

    def load(self, get):
        self.shift = get(self.name).float().contiguous()

    def state_spec(self):
        return StateSpec((self.width,), torch.float32)

    @staticmethod
    def rides(step) -> bool:
        """Whether every request of the step brings one row: the launch that writes the rows can shift them."""
        return step.n_tokens == step.n_requests

    def forward(self, h, step, state):
        return ops.token_shift(h, self.shift, state, step.row_req, step.state_slots, step.n_requests, self.out_dtype)
