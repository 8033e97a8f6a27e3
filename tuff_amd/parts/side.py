"""A narrow input of a layer's own for every token: a vector looked up by the token's id, gated by the stream.

    e = table[token, columns of the layer]          [dim]
    g = act(W_gate x) * e                           (x: the residual stream itself, no norm before it)
    x <- x + n / sqrt(mean(n^2) + eps) * w,   n = W_proj g

The table holds every layer's columns side by side and is one tensor of the model (Part.shared_decls).  The norm of the
result and the sum run in the kernel of the block that owns the part.
"""
from __future__ import annotations

import torch

from ..csrc import ops
from .base import Part, Runtime, WeightDecl
from .linear import Linear
from .norm import RMSNorm


class TokenSide(Part):
    graph_safe = True
    records_portions = True

    def __init__(self, hidden_size: int, dim: int, vocab_size: int, table_width: int, col0: int, eps: float, *, names: dict[str, str],
                 activation: str = "gelu_tanh"):
        """names: checkpoint names of 'table' [vocab, table_width] (this layer's columns are col0 .. col0 + dim - 1), 'gate'
        [dim, d], 'proj' [d, dim] and 'norm' [d] (a plain weight)."""
        self.d, self.dim, self.col0 = int(hidden_size), int(dim), int(col0)
        if not 0 <= self.col0 <= int(table_width) - self.dim:
            raise ValueError(f"columns {col0} .. {col0 + dim - 1} of a table of {table_width}")
        if activation not in ops.ACTIVATIONS:
            raise ValueError(f"unknown activation '{activation}'")
        self.table_decl = WeightDecl(names["table"], (int(vocab_size), int(table_width)), "normal")
        self.activation = activation
        self.gate = Linear(names["gate"], self.d, self.dim)
        self.proj = Linear(names["proj"], self.dim, self.d)
        self.norm = RMSNorm(self.d, eps, names["norm"])

    def weight_decls(self):
        return self.gate.weight_decls() + self.proj.weight_decls() + self.norm.weight_decls()

    def shared_decls(self):
        return [self.table_decl]

    def kernel_modules(self):
        return ["elementwise", "postnorm"]

    def bind(self, weights, rt: Runtime):
        self.rt = rt
        self.table = weights[self.table_decl.name].contiguous()
        for p in (self.gate, self.proj, self.norm):
            p.bind(weights, rt)

    def forward(self, rows, ctx, y) -> None:
        """rows [T, d]: the stream in the compute type.  Adds n into y (float32 [T, d])."""
        u = self.gate.forward(rows, out_dtype=torch.float32)          # the activation reads the sums as they are
        g = self.rt.empty(u.shape[0], self.proj.k_padded)             # (as wide as the next product reads its rows)
        ops.act_lookup(u, self.table, ctx.tokens, g, self.activation, self.col0)
        self.proj.forward(g, accumulate_into=y)
