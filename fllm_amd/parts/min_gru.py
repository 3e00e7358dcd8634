"""A gated recurrence lane by lane whose gates read the current token alone (minGRU).

z = sigmoid(W_z h + b_z) and u = W_x h + b_x, both of `size` lanes; the candidate is c = u + 1/2 where u >= 0 and sigmoid(u)
where u < 0; S_t = (1 - z) S_(t-1) + z c lane by lane; the output is W_o (S_t * silu(W_g h)).  S starts at zero, is float32
[size] for every live request, and is all this mixer keeps: it has no pages, and a prompt may be cut anywhere.  z, u and the
gate are one product with the concatenated matrix; the biases, the gates and the recurrence are float32 behind it.
"""
from __future__ import annotations

import torch

from ..registry import register_part
from .base import INIT_BIAS, INIT_MATRIX, Mixer, StateNeed, add_and_prepare


class MinGRU(Mixer):
    graph_safe = True
    stores_branch = True

    @classmethod
    def tensor_shapes(cls, spec):
        h, n = spec["hidden_size"], spec["size"]
        shapes = {name: ((n, h), INIT_MATRIX) for name in ("z", "x", "g")}
        shapes.update(o=((h, n), INIT_MATRIX), z_bias=((n,), INIT_BIAS), x_bias=((n,), INIT_BIAS))
        return shapes

    def __init__(self, spec, weights, rt):
        super().__init__(spec, weights, rt)
        self.hidden, self.size = int(spec["hidden_size"]), int(spec["size"])
        self.w_zxg = torch.cat([rt.matrix(weights[n]) for n in ("z", "x", "g")], dim=0).contiguous()
        self.bias = torch.cat([rt.vector(weights[n]) for n in ("z_bias", "x_bias")]).contiguous()
        self.w_o = rt.matrix(weights["o"])
        rt.tile_for_decode(self.w_o)
        rt.tile_for_decode(self.w_zxg, priority=1)

    def state_need(self):
        return StateNeed((self.size,), torch.float32)

    def forward(self, ctx, h, residual, binding, branch=None) -> None:
        rt, ops = self.rt, self.rt.ops
        zxg = rt.empty((h.shape[0], 3 * self.size))
        ops.linear(h, self.w_zxg, zxg)
        out = rt.empty((h.shape[0], self.size))
        ops.min_recurrence(zxg, self.bias, binding.state, ctx.row_seg, ctx.seg_start, ctx.slots, out)
        if branch is not None:
            ops.linear(out, self.w_o, branch)
        elif not add_and_prepare(ctx, ops, out, self.w_o, residual, None):
            ops.linear(out, self.w_o, residual, accumulate=True)


register_part("mixer", "min_gru", MinGRU)
