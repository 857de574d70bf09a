"""Hyper-connections ("Hyper-Connections", Zhu et al.; the static form): the residual stream is kept in several fp32 copies x_1 .. x_S, all
equal to the embedding at the start.  A sublayer reads one weighted sum of them and its result is handed back to all,

    u = sum_s in[s] x_s,      y = sublayer(norm(u)),      x_t <- sum_s mix[s, t] x_s + out[t] y      (all t at once)

and the model's last norm reads the plain sum of the copies.  HyperConnection holds a sublayer's numbers; `open` gives the first sublayer its
input, `close` finishes a sublayer and gives the next one its input in one launch (ops.hyper_norm)."""
from __future__ import annotations

import torch
from torch import nn

from .. import ops
from .layernorm import StreamNorm


class HyperConnection(nn.Module):
    def __init__(self, streams: int):
        super().__init__()
        # (operands of the fp32 stream, whatever the activation type)
        self.in_weights = nn.Parameter(torch.ones(streams, dtype=torch.float32), requires_grad=False)
        self.out_weights = nn.Parameter(torch.ones(streams, dtype=torch.float32), requires_grad=False)
        self.mix = nn.Parameter(torch.eye(streams, dtype=torch.float32), requires_grad=False)

    def open(self, x: torch.Tensor, norm: StreamNorm) -> torch.Tensor:
        """x [T, S, width] (only read) -> norm(u) in the activation type."""
        return ops.hyper_norm(x, in_weights=self.in_weights.data, **norm.spec())

    def close(self, x: torch.Tensor, terms: dict, opening: "tuple[HyperConnection, StreamNorm] | None" = None) -> torch.Tensor | None:
        """This sublayer's result (`terms`: the sum's terms as ops.hyper_norm takes them) into x in place; returns norm(u) for the next
        sublayer, `opening` = (its connection, its norm)."""
        nxt = {} if opening is None else dict(in_weights=opening[0].in_weights.data, **opening[1].spec())
        return ops.hyper_norm(x, self.mix.data, self.out_weights.data, **terms, **nxt)
