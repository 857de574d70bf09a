"""Per-sequence state that is not a growing cache: a slot of a pool per live sequence.  The runner allocates and binds the pools of every
module that offers `states` and `state_shape` (engine/model_runner.py), the step's Context names each sequence's slot."""
from __future__ import annotations

import torch
from torch import nn

from ..utils.context import get_context


class StatePool(nn.Module):
    """A per-sequence fp32 state of fixed shape, one pool [slots, *shape] per pass (`states[run]`, bound by the runner)."""

    def __init__(self, shape: tuple, state_runs: int = 1):
        super().__init__()
        self._shape = tuple(int(n) for n in shape)
        self.state_runs = state_runs
        self.states: list = [None] * state_runs

    def state_shape(self) -> tuple:
        return self._shape

    def pool(self, run: int) -> torch.Tensor:
        ctx = get_context()
        if self.states[run] is None or ctx.state_slots is None:
            raise RuntimeError("a recurrent layer needs a bound state pool and a state slot per sequence")
        return self.states[run]


class LastToken(StatePool):
    """The last token id of every sequence (for layers that read a token together with the one before it): one 32-bit integer per slot,
    in the same fp32 pool memory as the other states."""

    def __init__(self, state_runs: int = 1):
        super().__init__((1,), state_runs)

    def ids(self, run: int = 0) -> torch.Tensor:
        return self.pool(run).view(torch.int32)
