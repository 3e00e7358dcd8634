"""Attention whose queries, keys and values pass a short convolution over time behind their projections, over the paged cache.

q, k, v (and the gate) are one product with the concatenated matrix; biases are added, then every channel of q, k and v becomes
y_t = sum_j w[:, j] u_(t - taps + 1 + j) (u: the projected value with its bias; zeros before the sequence's start).  The last
taps - 1 products of every live request are this mixer's state (without the biases, which the kernel adds where a product
exists).  Then, as the design asks: an RMS norm of every head of q and of k with one weight vector (`qk_norm_eps`), rotary on
the first lanes of every head (`position`, either pairing).  Keys and values go into the pages as they are then.

What a row sees: `chunk`: the keys of its own chunk of that many positions up to itself (chunks counted from position 0);
`window` and `keep_first`: its last `window` positions, itself included, and the first `keep_first` positions of the sequence.
Scores are q . k * scale, with `softcap` cap * tanh(score / cap); `sink` "zero" puts one more term exp(0), which has no value,
into the softmax's denominator.  `mix_weights`: head h applies sum_g talk[h, g] * (weights of head g) to the values of its own
key/value head.  That sum is taken behind the values: every head's weights meet the values of ALL key/value heads, and the
head's output is sum_g talk[h, g] * (head g's weights times h's values), in float32.  `output_gate`: the heads' outputs times
sigmoid(W_g h) before the output projection.

`own_keys` False: the layer has queries alone and reads the pages of the run entry that the run order names.
"""
from __future__ import annotations

import torch

from ..config.spec import PartSpec
from ..registry import part_class, register_part
from .base import INIT_BIAS, INIT_MATRIX, INIT_NORM, KVNeed, Mixer, StateNeed, add_and_prepare


class ConvAttention(Mixer):
    graph_safe = True      # forward launches kernels only: no per-step decision on the host
    stores_branch = True
    KEY_CHUNK = 8

    @classmethod
    def tensor_shapes(cls, spec):
        h, nh, nkv, d = spec["hidden_size"], spec["num_heads"], spec["num_kv_heads"], spec["head_dim"]
        dv, taps = spec.get("value_head_dim") or d, spec["taps"]
        sizes = {"q": nh * d, "k": nkv * d, "v": nkv * dv}
        shapes = {"o": ((h, nh * dv), INIT_MATRIX), "g": ((nh * dv, h), INIT_MATRIX), "q_norm": ((d,), INIT_NORM), "k_norm": ((d,), INIT_NORM),
                  "talk": ((nh, nh), INIT_MATRIX)}
        for name, n in sizes.items():
            shapes.update({name: ((n, h), INIT_MATRIX), f"{name}_bias": ((n,), INIT_BIAS), f"{name}_conv": ((n, taps), INIT_NORM)})
        return shapes

    def __init__(self, spec, weights, rt):
        super().__init__(spec, weights, rt)
        self.hidden = int(spec["hidden_size"])
        self.heads = int(spec["num_heads"])
        self.kv_heads = int(spec["num_kv_heads"])
        self.head_dim = int(spec["head_dim"])
        self.v_dim = int(spec.get("value_head_dim") or self.head_dim)
        self.scale = float(spec["scale"])
        self.taps = int(spec["taps"])
        self.own_keys = bool(spec.get("own_keys", True))
        if self.heads % self.kv_heads != 0:
            raise ValueError(f"head count {self.heads} is not a multiple of key/value head count {self.kv_heads}")
        if not 1 <= self.taps <= 16:
            raise ValueError(f"a convolution of {self.taps} taps is outside 1..16")
        self.chunk, self.window = int(spec.get("chunk") or 0), int(spec.get("window") or 0)
        self.keep_first = int(spec.get("keep_first") or 0)
        if self.chunk < 0 or self.window < 0 or self.keep_first < 0 or (self.chunk and self.window) or (self.keep_first and not self.window):
            raise ValueError("a row sees its chunk, or a window with first tokens kept")
        self.softcap = float(spec.get("softcap") or 0.0)          # 0: scores as they are
        sink = spec.get("sink")
        if sink not in (None, "zero"):
            raise ValueError(f"sink {sink!r}: 'zero' or None")
        self.zero_sink = sink == "zero"
        self.eps = float(spec.get("qk_norm_eps") or 0.0)
        self.q_weight = self.k_weight = None
        if self.eps > 0.0:
            self.q_weight = rt.vector(weights["q_norm"])
            self.k_weight = rt.vector(weights["k_norm"]) if self.own_keys else None
        self.gated = bool(spec.get("output_gate", False))
        self.talk = rt.vector(weights["talk"]) if spec.get("mix_weights", False) else None
        self.key_chunk = self.KEY_CHUNK if self.head_dim % self.KEY_CHUNK == 0 else 1
        position = spec.get("position")
        self.position = None
        if position is not None:
            position = dict(position)
            kind = position.pop("kind")
            self.position = part_class("position", kind)(PartSpec(kind, position), {}, rt)
            if self.position.dims > self.head_dim:
                raise ValueError(f"{self.position.dims} rotated lanes in heads of {self.head_dim}")
        names = ("q", "k", "v") if self.own_keys else ("q",)
        pieces = [rt.matrix(weights[n]) for n in names]
        self.channels = sum(p.shape[0] for p in pieces)           # what passes the convolution; the gate stands behind
        self.gate_at = self.channels
        if self.gated:
            pieces.append(rt.matrix(weights["g"]))
        self.w_joint = torch.cat(pieces, dim=0).contiguous()
        self.w_o = rt.matrix(weights["o"])
        rt.tile_for_decode(self.w_o)
        rt.tile_for_decode(self.w_joint, priority=1)
        self.w_conv = torch.cat([rt.vector(weights[f"{n}_conv"]) for n in names], dim=0).contiguous()      # float32 [channels, taps]
        self.bias = None
        if any(weights.get(f"{n}_bias") is not None for n in names):
            self.bias = torch.cat([rt.vector(weights[f"{n}_bias"]) if weights.get(f"{n}_bias") is not None
                                   else torch.zeros(p.shape[0], dtype=torch.float32, device=rt.device)
                                   for n, p in zip(names, pieces)]).contiguous()

    def cache_need(self):
        # every key is kept: a chunk is a mask, and a window's first tokens never leave it
        return KVNeed(self.kv_heads, self.head_dim, self.v_dim, None, key_chunk=self.key_chunk)

    def state_need(self):
        return StateNeed((self.taps - 1, self.channels), self.rt.dtype) if self.taps > 1 else None

    def forward(self, ctx, h, residual, binding, branch=None) -> None:
        rt, ops = self.rt, self.rt.ops
        rows = h.shape[0]
        nh, nkv, d, dv = self.heads, self.kv_heads, self.head_dim, self.v_dim
        if binding.writes != self.own_keys:
            raise ValueError("a layer without keys of its own reads another run entry's pages, any other writes its own")
        joint = rt.empty((rows, self.w_joint.shape[0]))
        ops.linear(h, self.w_joint, joint)
        tables = ctx.tables[binding.group]
        if self.position is not None:
            cos, sin, dims, pairing = self.position.cos, self.position.sin, self.position.dims, self.position.pairing
        else:
            cos, sin, dims, pairing = ctx.no_rotation(rt)
        q = rt.empty((rows, nh * d))
        ops.conv_qkv_store(joint, self.w_conv, self.bias, binding.state if self.taps > 1 else None, self.q_weight, self.k_weight, self.eps,
                           q, ctx.row_pos, ctx.row_seg, ctx.seg_start, ctx.slots, tables, cos, sin, binding.k_pages if self.own_keys else None,
                           binding.v_pages if self.own_keys else None, nh, nkv, d, dv, dims, pairing, binding.page_size, self.key_chunk,
                           single_rows=bool(ctx.uniform_rows))
        out = rt.empty((rows, nh * dv))
        mask = dict(chunk=self.chunk, window=self.window, keep_first=self.keep_first, softcap=self.softcap, zero_sink=self.zero_sink,
                    talk=self.talk, max_context=ctx.max_context)
        ops.masked_attention(q, binding.k_pages, binding.v_pages, tables, ctx.row_pos, ctx.row_seg, ctx.seg_start, out, nh, nkv, d, dv,
                             binding.page_size, self.scale, self.key_chunk, **mask)
        if self.gated:
            gated = rt.empty((rows, nh * dv))
            out = ops.gated_norm(out, None, 0.0, joint[:, self.gate_at:], gated)
        if branch is not None:
            ops.linear(out, self.w_o, branch)
        elif not add_and_prepare(ctx, ops, out, self.w_o, residual, None):
            ops.linear(out, self.w_o, residual, accumulate=True)


register_part("mixer", "conv_attention", ConvAttention)
