"""What begins every pass of a stretch of layers that runs several times: the stream becomes a projection of itself joined
with the embedding, plus a vector of the pass's own,

    x <- W [x ; x0] + step[t],        t = 0, 1, ... the number of the pass.

W [d, 2 d] is bound as its two halves: W_0 x0 is the same in every pass and computed once a step; a pass multiplies W_x with
x and one kernel adds the three and norms the sum for the pass's first sublayer.
"""
from __future__ import annotations

import torch

from ..csrc import ops
from .base import Part, Runtime, WeightDecl
from .linear import Linear


class PassEntry(Part):
    graph_safe = True
    records_portions = True

    def __init__(self, hidden_size: int, times: int, *, names: dict[str, str]):
        """names: checkpoint names of 'in' [d, 2 d] (the stream's columns first) and 'step' [times, d]."""
        self.d, self.times, self.names = int(hidden_size), int(times), dict(names)
        self.of_x = Linear(names["in"] + "/x", self.d, self.d)
        self.of_x0 = Linear(names["in"] + "/x0", self.d, self.d)

    def weight_decls(self):
        return [WeightDecl(self.names["in"], (self.d, 2 * self.d), "normal", role="projection"),
                WeightDecl(self.names["step"], (self.times, self.d), "normal")]

    def kernel_modules(self):
        return ["postnorm", "elementwise"]

    def bind(self, weights, rt: Runtime):
        self.rt = rt
        w = weights[self.names["in"]]
        self.of_x.bind({self.of_x.names[0]: w[:, :self.d].contiguous()}, rt)
        self.of_x0.bind({self.of_x0.names[0]: w[:, self.d:].contiguous()}, rt)
        self.step = weights[self.names["step"]].float().contiguous()

    def embedding_part(self, x0_rows) -> torch.Tensor:
        """float32 [T, d]: W_0 x0, once a step.  x0_rows: the embedding in the compute type."""
        return self.of_x0.forward(x0_rows, out_dtype=torch.float32)

    def forward(self, rows, z0, t: int, read):
        """rows [T, d]: the stream in the compute type; z0: embedding_part().  Returns the new stream, float32 [T, d], and what
        the pass's first sublayer reads of it: read = (norm weight, eps)."""
        x = self.of_x.forward(rows, out_dtype=torch.float32)
        h = self.rt.empty(*x.shape)
        ops.post_norm_add(x, extra=z0, row=self.step[t], next_w=read[0], next_eps=read[1], h_out=h)
        return x, h
