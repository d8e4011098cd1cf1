"""Token shift: what a sublayer reads is mixed, element by element, with the same of the token before:
    h_t = x_t + (x_{t-1} - x_t) * mu        x_{-1} = 0; the rows mixed in are the stream's, not their mixtures
The last x of every sequence is a state of `dim` float32 values, kept in a row of the cache's state area.  Shared by
blocks; not a registered part by itself."""
from __future__ import annotations

import torch

from .base import ParamSpec, Part
from .linear import upload


class TokenShift(Part):
    prompt_capturable = True    # a prompt step is read from the context's device tensors alone

    def __init__(self, dim: int):
        self.dim, self.mu = int(dim), None

    def tensors(self):
        return {"mu": ParamSpec((self.dim,), "normal")}

    def load(self, tensors, device, dtype):
        self.mu = upload(tensors["mu"], device, torch.float32)

    @property
    def state_floats(self) -> int:
        return self.dim

    def apply(self, stream, state, ctx):
        """state: [slots + 1, >= dim] float32, this shift's columns of the state rows."""
        return stream.mixed_with_previous(self.mu, state, ctx)
