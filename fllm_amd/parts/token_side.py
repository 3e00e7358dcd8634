"""What a token itself brings to a layer, beside the stream.

A table holds `layers * dim` numbers a token; layer i takes the part e = table[token][i * dim : (i + 1) * dim].  The stream
chooses among them, g = gelu_tanh(W_g x) * e, and y = W_p g joins it behind an RMS norm: x += y / rms(y) * w.  A part of role
`stream` that an arrangement runs at a layer's end.
"""
from __future__ import annotations

import torch

from ..registry import register_part
from .base import INIT_MATRIX, INIT_NORM, Part


class TokenSide(Part):
    role = "stream"
    graph_safe = True

    @classmethod
    def tensor_shapes(cls, spec):
        size, dim = spec["size"], spec["dim"]
        return {"table": ((spec["vocab_size"], spec["layers"] * dim), INIT_MATRIX), "gate": ((dim, size), INIT_MATRIX),
                "proj": ((size, dim), INIT_MATRIX), "norm": ((size,), INIT_NORM)}

    def __init__(self, spec, weights, rt):
        super().__init__(spec, weights, rt)
        self.size, self.dim = int(spec["size"]), int(spec["dim"])
        self.eps = float(spec["eps"])
        layer, layers = int(spec["layer"]), int(spec["layers"])
        if not 0 <= layer < layers:
            raise ValueError(f"layer {layer} of {layers}")
        self.offset = layer * self.dim
        self.table = rt.matrix(weights["table"])
        self.w_gate = rt.matrix(weights["gate"])
        self.w_proj = rt.matrix(weights["proj"])
        self.weight = rt.vector(weights["norm"])

    def forward(self, ctx, x, embedding=None) -> None:
        rt, ops = self.rt, self.rt.ops
        rows = x.shape[0]
        g = rt.empty((rows, self.dim))
        gate = getattr(ops, "side_gate", None)          # steps of few rows: one kernel up to the gated numbers
        if gate is None or not gate(x, self.w_gate, ctx.ids, self.table, self.offset, g):
            h = rt.empty((rows, self.size))
            ops.cast_rows(x, h)
            z = rt.empty((rows, self.dim))
            ops.linear(h, self.w_gate, z)
            ops.gelu_side(z, ctx.ids, self.table, self.offset, g)
        y = rt.empty((rows, self.size), torch.float32)
        ops.linear(g, self.w_proj, y)
        ops.postnorm_add(x, y, self.weight, self.eps)


register_part("stream", "token_side", TokenSide)
