"""Linear attention with a decay a key channel that every token chooses (gated linear attention).

q = W_q h * query_scale and k = W_k h (heads x dim), v = W_v h (heads x vdim); alpha = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau),
heads x dim numbers in (0, 1).  Per head S_t = diag(alpha_t) S_(t-1) + k_t v_t^T and o_t = S_t^T q_t.  Every head's o is
RMS-normed over its vdim lanes (one weight vector of that size for all heads), multiplied lane by lane with silu(W_g h), and
the heads side by side are projected by W_o.  S starts at zero, is float32 [heads, dim, vdim] for every live request, and is
all this mixer keeps: it has no pages, and a prompt may be cut anywhere.  q, k, v, the gate and W_a1 h are one product with the
concatenated matrix; W_a2's product leaves float32, and everything behind the projections that enters the recurrence (bias,
logarithm of the decay, scale) is float32.  The rank of the decay's projection is whatever the checkpoint's W_a1 has.
"""
from __future__ import annotations

import torch

from ..registry import register_part
from .base import INIT_BIAS, INIT_MATRIX, INIT_NORM, Mixer, SizeFromFile, StateNeed, add_and_prepare

DEFAULT_RANK = 16      # of random weights


class GatedLinearAttention(Mixer):
    graph_safe = True
    stores_branch = True

    @classmethod
    def tensor_shapes(cls, spec):
        h, nh, d, dv = spec["hidden_size"], spec["num_heads"], spec["head_dim"], spec["value_head_dim"]
        rank = SizeFromFile(spec.get("rank", DEFAULT_RANK))
        return {"q": ((nh * d, h), INIT_MATRIX), "k": ((nh * d, h), INIT_MATRIX), "v": ((nh * dv, h), INIT_MATRIX),
                "g": ((nh * dv, h), INIT_MATRIX), "o": ((h, nh * dv), INIT_MATRIX), "norm": ((dv,), INIT_NORM),
                "a1": ((rank, h), INIT_MATRIX), "a2": ((nh * d, rank), INIT_MATRIX), "a2_bias": ((nh * d,), INIT_BIAS)}

    def __init__(self, spec, weights, rt):
        super().__init__(spec, weights, rt)
        self.hidden = int(spec["hidden_size"])
        self.heads = int(spec["num_heads"])
        self.dim = int(spec["head_dim"])
        self.v_dim = int(spec["value_head_dim"])
        self.eps = float(spec["eps"])
        self.tau = float(spec["tau"])
        self.query_scale = float(spec.get("query_scale", 1.0))
        if not self.tau > 0.0:
            raise ValueError("tau must be positive")
        a1, a2 = rt.matrix(weights["a1"]), rt.matrix(weights["a2"])
        self.rank = int(a1.shape[0])
        if a2.shape[1] != self.rank:
            raise ValueError(f"the decay's two matrices do not meet: {tuple(a1.shape)} and {tuple(a2.shape)}")
        pieces = [rt.matrix(weights[n]) for n in ("q", "k", "v", "g")]
        used = sum(p.shape[0] for p in pieces)
        # zero rows before and behind W_a1, so that its columns of the product begin on 16 bytes, and so does every row; zero
        # columns of W_a2 likewise bring the rank to a multiple of 8
        zeros = lambda n: torch.zeros((n, self.hidden), dtype=a1.dtype, device=rt.device)
        self.a_at = used + (-used) % 8
        self.rank_wide = self.rank + (-self.rank) % 8
        if self.a_at != used:
            pieces.append(zeros(self.a_at - used))
        pieces.append(a1)
        if self.rank_wide != self.rank:
            pieces.append(zeros(self.rank_wide - self.rank))
            a2 = torch.cat([a2, torch.zeros((a2.shape[0], self.rank_wide - self.rank), dtype=a2.dtype, device=rt.device)], dim=1)
        self.w_joint = torch.cat(pieces, dim=0).contiguous()
        self.w_a2 = a2.contiguous()
        self.a2_bias = rt.vector(weights["a2_bias"])
        self.norm_weight = rt.vector(weights["norm"])
        self.w_o = rt.matrix(weights["o"])
        rt.tile_for_decode(self.w_o)
        rt.tile_for_decode(self.w_joint, priority=1)

    def state_need(self):
        return StateNeed((self.heads, self.dim, self.v_dim), torch.float32)

    def forward(self, ctx, h, residual, binding, branch=None) -> None:
        rt, ops = self.rt, self.rt.ops
        rows = h.shape[0]
        nq, nv = self.heads * self.dim, self.heads * self.v_dim
        joint = rt.empty((rows, self.w_joint.shape[0]))
        ops.linear(h, self.w_joint, joint)
        z = rt.empty((rows, nq), torch.float32)
        ops.linear(joint[:, self.a_at:self.a_at + self.rank_wide], self.w_a2, z)
        o = rt.empty((rows, nv), torch.float32)
        ops.gated_linear_attention(joint, z, self.a2_bias, self.tau, self.query_scale, binding.state, ctx.row_seg, ctx.seg_start, ctx.slots, o,
                                   self.heads, self.dim, self.v_dim)
        gated = rt.empty((rows, nv))
        ops.group_norm_gate(o, self.eps, self.v_dim, joint[:, 2 * nq + nv:2 * (nq + nv)], gated, activation="silu", weight=self.norm_weight)
        if branch is not None:
            ops.linear(gated, self.w_o, branch)
        elif not add_and_prepare(ctx, ops, gated, self.w_o, residual, None):
            ops.linear(gated, self.w_o, residual, accumulate=True)


register_part("mixer", "gated_linear", GatedLinearAttention)
