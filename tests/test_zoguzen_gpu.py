"""Zoguzen on the MI355X: each of its kernels alone against tests/reference_ops.py (float64), then the engine's steps however a
request is cut and batched, captured decode steps and greedy generation against tests/plain_zoguzen.py."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_zoguzen as pz
import trace_tools as tt
import zoguzen_configs as zc
from reference_ops import ReferenceOps

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
BF16_EPS = 2.0 ** -8
F32, BF16, F64 = torch.float32, torch.bfloat16, torch.float64


@pytest.fixture(scope="module")
def ops():
    from fllm_amd.kernels import Ops
    return Ops()


@pytest.fixture(scope="module")
def ref():
    return ReferenceOps()


def gen(seed):
    g = torch.Generator()
    g.manual_seed(seed)
    return g


def close(got, want, rtol, atol, what=""):
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    err = (got - want).abs()
    assert torch.isfinite(got).all(), f"{what}: not finite"
    worst = (err - (atol + rtol * want.abs())).max().item()
    assert worst <= 0, f"{what}: max err {err.max().item():.3e} (|want| max {want.abs().max().item():.3e}), over by {worst:.3e}"


class Batch:
    """Requests that hold `held` tokens in shuffled pages and bring `new` rows each, in state slots out of order; CPU tensors."""

    def __init__(self, segments, page, seed):
        g = gen(seed)
        self.segments, self.page = segments, page
        each = [-(-(held + new) // page) for held, new in segments]
        self.num_pages = sum(each) + 3
        order = torch.randperm(self.num_pages - 1, generator=g) + 1            # page 0 stays unused: a wrong lookup shows
        self.tables = torch.full((len(segments), max(each)), -1, dtype=torch.int32)
        at = 0
        for s, n in enumerate(each):
            self.tables[s, :n] = order[at:at + n].to(torch.int32)
            at += n
        pos, seg, start = [], [], [0]
        for s, (held, new) in enumerate(segments):
            pos += list(range(held, held + new))
            seg += [s] * new
            start.append(start[-1] + new)
        i32 = lambda v: torch.tensor(v, dtype=torch.int32)
        self.row_pos, self.row_seg, self.seg_start = i32(pos), i32(seg), i32(start)
        self.slots = torch.randperm(len(segments) + 2, generator=g)[:len(segments)].to(torch.int32)
        self.num_slots = len(segments) + 2
        self.rows = len(pos)
        self.max_pos = max(h + n for h, n in segments)
        self.single = all(n == 1 for _, n in segments)

    def on(self, device):
        return [t.to(device) for t in (self.row_pos, self.row_seg, self.seg_start, self.slots, self.tables)]


MIXED = [(0, 9), (37, 1), (100, 30), (61, 3), (250, 1), (300, 70), (0, 2)]
SINGLES = [(0, 1), (37, 1), (100, 1), (63, 1), (250, 1), (64, 1), (700, 1)]


# ---------------------------------------------------------------------------------------------
# norms and small passes
# ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("rows,width", [(1, 48), (7, 52), (33, 1024), (5, 1536), (3, 5000), (2, 9000)])
def test_layer_norms_of_rows_with_an_offset(ops, ref, rows, width, dtype):
    g = gen(width)
    x = torch.randn(rows, width, generator=g) * 2 + 30.0            # a mean far from zero: it has to be taken off first
    w1, w2 = 1 + torch.rand(width, generator=g), torch.randn(width, generator=g)
    want1, want2 = torch.empty(rows, width, dtype=F64), torch.empty(rows, width, dtype=F64)
    ref.layernorm_pair(x, w1, 1e-5, want1, w2, 1e-2, want2)
    got1, got2 = torch.empty(rows, width, dtype=dtype, device=DEV), torch.empty(rows, width, dtype=dtype, device=DEV)
    ops.layernorm_pair(x.to(DEV), w1.to(DEV), 1e-5, got1, w2.to(DEV), 1e-2, got2)
    tol = (1e-5, 2e-5) if dtype == F32 else (BF16_EPS, 1e-3)
    close(got1, want1, *tol)
    close(got2, want2, *tol)
    pick = torch.tensor([rows - 1, 0], dtype=torch.int32)
    one = torch.empty(2, width, dtype=dtype, device=DEV)
    ops.layernorm(x.to(DEV), w1.to(DEV), 1e-5, one, rows=pick.to(DEV))
    assert torch.equal(one, got1[[rows - 1, 0]])


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("two", [True, False])
@pytest.mark.parametrize("width,taps", [(48, 2), (52, 1), (1024, 2), (1536, 4), (5000, 2)])
def test_norms_and_convolution_in_one_kernel(ops, width, taps, two, dtype):
    """Steps of single rows: the bits of layer norm and convolution one after the other, the state moved on likewise; a padding
    row gives zeros and leaves the state alone."""
    g = gen(width + taps)
    rows = 5
    x = (torch.randn(rows, width, generator=g) * 2 + 10.0).to(DEV)
    w1, w2 = (1 + torch.rand(width, generator=g)).to(DEV), torch.randn(width, generator=g).to(DEV)
    conv = torch.randn(width, taps, generator=g).to(DEV)
    state = torch.randn(7, taps - 1, width, generator=g).to(dtype).to(DEV) if taps > 1 else None
    slots, row_seg = torch.tensor([6, 0, 3, 1, 0], dtype=torch.int32, device=DEV), torch.tensor([0, 1, 2, 3, -1], dtype=torch.int32, device=DEV)
    seg_start = torch.arange(rows + 1, dtype=torch.int32, device=DEV)
    h, other, want = (torch.empty(rows, width, dtype=dtype, device=DEV) for _ in range(3))
    ops.layernorm_pair(x, w1, 1e-5, h, w2, 1e-3, other)
    st = None if state is None else state.clone()
    ops.short_conv(h, conv, st, row_seg, seg_start, slots, want)
    got, second = (torch.full((rows, width), float("nan"), dtype=dtype, device=DEV) for _ in range(2))
    st2 = None if state is None else state.clone()
    assert ops.layernorm_conv(x, w1, 1e-5, conv, st2, row_seg, slots, got, *((w2, 1e-3, second) if two else ()))
    assert torch.equal(got[:4], want[:4]) and not got[4].any()
    if two:
        assert torch.equal(second[:4], other[:4]) and not second[4].any()
    if state is not None:
        assert torch.equal(st, st2) and not torch.equal(st2[6], state[6])
    assert not ops.layernorm_conv(torch.zeros(1, 8193, device=DEV), w1, 1e-5, torch.zeros(8193, taps, device=DEV), st2, row_seg, slots, got)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("rows,width,dim", [(1, 48, 5), (2, 1536, 192), (3, 520, 1), (8, 1024, 64)])
def test_the_side_inputs_gate_in_one_kernel(ops, ref, rows, width, dim, dtype):
    g = gen(rows)
    x, w = torch.randn(rows, width, generator=g) * 3, (torch.randn(dim, width, generator=g) * width ** -0.5).to(dtype)
    table = torch.randn(31, 3 * dim, generator=g).to(dtype)
    ids = torch.randint(0, 31, (rows,), generator=g, dtype=torch.int32)
    want, got = torch.empty(rows, dim, dtype=F64), torch.full((rows, dim), float("nan"), dtype=dtype, device=DEV)
    ref.gelu_side(x.to(dtype).double() @ w.double().T, ids, table.double(), 2 * dim, want)
    assert ops.side_gate(x.to(DEV), w.to(DEV), ids.to(DEV), table.to(DEV), 2 * dim, got)
    close(got, want, *((1e-5, 1e-5) if dtype == F32 else (BF16_EPS, 1e-3)))
    nine = torch.zeros(9, width, device=DEV)
    assert not ops.side_gate(nine, w.to(DEV), torch.zeros(9, dtype=torch.int32, device=DEV), table.to(DEV), 0, torch.empty(9, dim, dtype=dtype, device=DEV))
    odd = torch.zeros(1, 52, device=DEV)
    assert not ops.side_gate(odd, torch.zeros(dim, 52, dtype=dtype, device=DEV), ids[:1].to(DEV), table.to(DEV), 0, got[:1])


@pytest.mark.parametrize("rows,experts,top", [(9, 4, 2), (40, 8, 3), (700, 5, 2)])
def test_grouped_experts_read_the_rows_as_they_are(ops, rows, experts, top):
    """Without weights: the bits of weights that are all 1, also where the rows lie apart from each other."""
    g = gen(rows)
    wide = torch.randn(rows, 200, generator=g).to(BF16).to(DEV)
    h = wide[:, :136]
    w_gate_up = (torch.randn(experts, 2 * 48, 136, generator=g) * 136 ** -0.5).to(BF16).to(DEV)
    w_down = (torch.randn(experts, 136, 48, generator=g) * 48 ** -0.5).to(BF16).to(DEV)
    ids = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(rows)]).to(torch.int32).to(DEV)
    want, got = (torch.full((rows * top, 136), float("nan"), device=DEV) for _ in range(2))
    assert ops.experts_grouped(h, ids, torch.ones(rows, top, device=DEV), w_gate_up, w_down, want)
    assert ops.experts_grouped(h, ids, None, w_gate_up, w_down, got)
    assert torch.equal(got, want)


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_the_small_passes(ops, ref, dtype):
    g = gen(2)
    rows, width, dim, vocab = 13, 200, 24, 50
    x, y, out = (torch.randn(rows, width, generator=g) * s for s in (3.0, 0.2, 1.0))
    wx, wy = torch.randn(width, generator=g), torch.randn(width, generator=g)
    for accumulate in (True, False):
        want, got = out.double(), out.to(DEV)
        ref.normed_pair_sum(want, x, wx, 0.5, y, wy, 0.7, 1e-5, accumulate=accumulate)
        ops.normed_pair_sum(got, x.to(DEV), wx.to(DEV), 0.5, y.to(DEV), wy.to(DEV), 0.7, 1e-5, accumulate=accumulate)
        close(got, want, 1e-5, 1e-5, "normed pair")
    cast = torch.empty(rows, width, dtype=dtype, device=DEV)
    ops.cast_rows(x.to(DEV), cast)
    assert torch.equal(cast.cpu(), x.to(dtype))
    capped = (x * 20).to(DEV)
    ops.softcap_(capped, 25.0)
    close(capped, 25.0 * torch.tanh(x.double() * 20 / 25.0), 1e-5, 1e-5, "cap")
    z, table = (torch.randn(rows, dim, generator=g) * 2).to(dtype), torch.randn(vocab, 3 * dim, generator=g).to(dtype)
    ids = torch.randint(0, vocab, (rows,), generator=g, dtype=torch.int32)
    want, got = torch.empty(rows, dim, dtype=F64), torch.empty(rows, dim, dtype=dtype, device=DEV)
    ref.gelu_side(z.double(), ids, table.double(), dim, want)
    ops.gelu_side(z.to(DEV), ids.to(DEV), table.to(DEV), dim, got)
    close(got, want, *((1e-5, 1e-5) if dtype == F32 else (BF16_EPS, 1e-3)), "side input")
    o, gate, w = torch.randn(rows, 48, generator=g), torch.randn(rows, 48, generator=g).to(dtype), torch.randn(24, generator=g)
    want, got = torch.empty(rows, 48, dtype=F64), torch.empty(rows, 48, dtype=dtype, device=DEV)
    ref.group_norm_gate(o.double(), 1e-5, 24, gate.double(), want, weight=w)
    ops.group_norm_gate(o.to(DEV), 1e-5, 24, gate.to(DEV), got, weight=w.to(DEV))
    close(got, want, *((1e-5, 1e-5) if dtype == F32 else (BF16_EPS, 1e-3)), "heads normed with a weight")


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_the_shift_is_a_convolution_of_two_taps(ops, dtype):
    b = Batch([(0, 5), (4, 1), (9, 3)], 8, 1)
    g = gen(4)
    h, amount = torch.randn(b.rows, 40, generator=g).to(dtype), torch.rand(40, generator=g)
    state = torch.randn(b.num_slots, 1, 40, generator=g).to(dtype)
    state[b.slots[0].item()] = 0
    _, row_seg, seg_start, slots, _ = b.on(DEV)
    got, st = torch.empty_like(h, device=DEV), state.to(DEV)
    ops.short_conv(h.to(DEV), torch.stack([amount, -amount], dim=1).to(DEV), st, row_seg, seg_start, slots, got)
    for s in range(3):
        r0, r1 = int(b.seg_start[s]), int(b.seg_start[s + 1])
        before = torch.cat([state[int(b.slots[s])].double(), h[r0:r1 - 1].double()])
        close(got[r0:r1], h[r0:r1].double() + (before - h[r0:r1].double()) * amount.double(), *((1e-6, 1e-6) if dtype == F32 else (BF16_EPS, 1e-6)))
        assert torch.equal(st[int(b.slots[s]), 0].cpu(), h[r1 - 1])


# ---------------------------------------------------------------------------------------------
# projections behind a convolution
# ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("segments", [MIXED, SINGLES, [(0, 1), (1, 1), (2, 1), (3, 2), (2, 7)]])
@pytest.mark.parametrize("H,G,d,dv,rope,pairing,taps,norm,bias,keys", [
    (4, 2, 32, 16, 16, 1, 4, False, False, True), (3, 1, 10, 6, 6, 1, 3, True, True, True), (8, 4, 64, 64, 64, 0, 2, True, True, True),
    (2, 2, 24, 24, 0, 0, 4, True, True, False), (2, 1, 128, 300, 128, 1, 16, False, True, True), (3, 3, 8, 8, 0, 0, 1, True, False, True)])
def test_convolved_queries_keys_and_values(ops, ref, H, G, d, dv, rope, pairing, taps, norm, bias, keys, segments, dtype):
    b = Batch(segments, 16, H * 10 + d)
    g = gen(5)
    channels = H * d + (G * (d + dv) if keys else 0)
    kc = 8 if d % 8 == 0 else 1
    joint = torch.randn(b.rows, channels + 8, generator=g).to(dtype)
    conv, bs = torch.randn(channels, taps, generator=g), torch.randn(channels, generator=g) if bias else None
    qw, kw = (1 + 0.4 * torch.rand(d, generator=g) for _ in range(2)) if norm else (None, None)
    state = torch.randn(b.num_slots, taps - 1, channels, generator=g).to(dtype) if taps > 1 else None
    if taps > 1:                      # entries before a sequence's first token are zeros
        for s, (held, _) in enumerate(segments):
            state[int(b.slots[s]), :max(0, taps - 1 - held)] = 0
    cos, sin = torch.rand(800, rope // 2, generator=g) * 2 - 1, torch.rand(800, rope // 2, generator=g) * 2 - 1
    kp, vp = torch.randn(b.num_pages, G, d // kc, 16, kc, generator=g).to(dtype), torch.randn(b.num_pages, G, dv, 16, generator=g).to(dtype)
    results = []
    for o, dev, kind in ((ref, "cpu", F64), (ops, DEV, dtype)):
        on = lambda t: None if t is None else t.to(dev).contiguous()
        as_kind = lambda t: None if t is None else t.to(device=dev, dtype=kind).contiguous()
        row_pos, row_seg, seg_start, slots, tables = b.on(dev)
        q, st, k, v = torch.zeros(b.rows, H * d, dtype=kind, device=dev), as_kind(state), as_kind(kp), as_kind(vp)
        o.conv_qkv_store(as_kind(joint), on(conv), on(bs), st, on(qw), on(kw), 1e-5 if norm else 0.0, q, row_pos, row_seg, seg_start, slots, tables,
                         on(cos), on(sin), k if keys else None, v if keys else None, H, G, d, dv, rope, pairing, 16, kc, single_rows=b.single)
        results.append((q, k, v, st))
    tol = (2e-5, 2e-5) if dtype == F32 else (BF16_EPS, 2e-3)
    for name, want, got in zip(("queries", "keys", "values"), results[0], results[1]):
        close(got, want, *tol, name)
    if taps > 1:
        assert torch.equal(results[1][3].double().cpu(), results[0][3]), "the last products of every sequence"


# ---------------------------------------------------------------------------------------------
# masked attention
# ---------------------------------------------------------------------------------------------
SHAPES = [(4, 2, 32, 32, 8), (3, 3, 12, 10, 16), (8, 2, 64, 64, 16), (6, 3, 96, 64, 32), (12, 2, 128, 128, 16), (4, 1, 64, 128, 64), (20, 1, 32, 96, 16),
          (2, 1, 128, 300, 32), (8, 8, 32, 64, 16), (9, 3, 40, 32, 16)]
MASKS = [dict(chunk=50, softcap=3.0, zero_sink=True, talk=True), dict(chunk=7, zero_sink=True, talk=True), dict(window=40, keep_first=20),
         dict(window=5, keep_first=100, softcap=2.0), dict(window=130, keep_first=1), dict(window=1), dict(softcap=20.0, talk=True)]


def attend(o, q, pages, index, kind, dev, b, H, G, d, dv, kc, mask, talk):
    row_pos, row_seg, seg_start, _, tables = index
    out = torch.full((b.rows, H * dv), float("nan"), dtype=kind, device=dev)
    args = dict(mask, talk=talk if mask.get("talk") else None)
    o.masked_attention(q, pages[0], pages[1], tables, row_pos, row_seg, seg_start, out, H, G, d, dv, b.page, 0.25, kc, max_context=b.max_pos, **args)
    return out


@pytest.mark.parametrize("segments", [MIXED, SINGLES])
@pytest.mark.parametrize("dtype,fast", [(F32, True), (BF16, True), (BF16, False)])
@pytest.mark.parametrize("mask", MASKS, ids=lambda m: "-".join(f"{k}{int(v)}" for k, v in m.items()))
@pytest.mark.parametrize("H,G,d,dv,page", SHAPES)
def test_masked_attention_over_pages(ops, ref, H, G, d, dv, page, mask, dtype, fast, segments):
    """`fast` False: the plain kernels also where the matrix-core kernels would serve."""
    b = Batch(segments, page, d + G)
    g = gen(3)
    kc = 8 if d % 8 == 0 else 1
    kp, vp = torch.randn(b.num_pages, G, d // kc, page, kc, generator=g).to(dtype), torch.randn(b.num_pages, G, dv, page, generator=g).to(dtype)
    q, talk = torch.randn(b.rows, H * d, generator=g).to(dtype), torch.randn(H, H, generator=g)
    want = attend(ref, q.double(), (kp.double(), vp.double()), b.on("cpu"), F64, "cpu", b, H, G, d, dv, kc, mask, talk)
    ops.set_fast_kernels(fast)
    try:
        got = attend(ops, q.to(DEV), (kp.to(DEV), vp.to(DEV)), b.on(DEV), dtype, DEV, b, H, G, d, dv, kc, mask, talk.to(DEV))
        torch.cuda.synchronize()
    finally:
        ops.set_fast_kernels(True)
    scale = want.abs().max().item()
    close(got, want, *((3e-5, 3e-5 * scale) if dtype == F32 else (2 * BF16_EPS, 2e-3 * scale)), "attention")


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("rows", [1, 20])
@pytest.mark.parametrize("mask,at,seen", [
    (dict(window=24, keep_first=5), 477, True), (dict(window=24, keep_first=5), 476, False), (dict(window=24, keep_first=5), 4, True),
    (dict(window=24, keep_first=5), 5, False), (dict(window=24, keep_first=5), 0, True), (dict(window=24, keep_first=5), 500, True),
    (dict(chunk=100), 500, True), (dict(chunk=100), 499, False), (dict(chunk=100), 0, False), (dict(chunk=501), 0, True), (dict(), 3, True)])
def test_one_key_that_stands_out_at_an_edge(ops, mask, at, seen, rows, dtype):
    """The last query sits at position 500; one position's key points along it and its value is marked: inside what the query sees it
    takes nearly all the weight, outside none of it arrives, whether the query comes alone or ends a portion."""
    H, G, d, dv, page = 4, 2, 32, 32, 16
    b = Batch([(501 - rows, rows)], page, 7)
    g = gen(at)
    kp, vp = 0.05 * torch.randn(b.num_pages, G, d // 8, page, 8, generator=g), torch.randn(b.num_pages, G, dv, page, generator=g)
    p, off = int(b.tables[0, at // page]), at % page
    kp[p, :, :, off, :], vp[p, :, :, off] = 3.0, 1000.0
    q = torch.ones(b.rows, H * d)
    got = attend(ops, q.to(DEV, dtype), (kp.to(DEV, dtype), vp.to(DEV, dtype)), b.on(DEV), dtype, DEV, b, H, G, d, dv, 8, mask, None)[-1].float().cpu()
    assert ((got > 990).all() if seen else (got.abs() < 10).all()), got[:4]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("rows", [1, 3])
def test_a_sink_by_hand_and_heads_mixed_behind_the_softmax(ops, rows, dtype):
    """Keys of score 0 (queries are zeros): n of them and the sink share the weight, n / (n + 1); head h gives the sum of its row of
    the mixing matrix times that."""
    H, G, d, dv, page = 4, 2, 64, 64, 16
    b = Batch([(41, rows)], page, 2)
    vp = torch.zeros(b.num_pages, G, dv, page)
    vp[:, 0], vp[:, 1] = 1.0, 10.0
    kp = torch.randn(b.num_pages, G, d // 8, page, 8, generator=gen(1))
    talk = torch.tensor([[1.0, 0, 0, 0], [0.5, 0.5, 1.0, -3.0], [0, 0, 0, 2.0], [0, 0, 0, 0]])
    got = attend(ops, torch.zeros(rows, H * d, device=DEV, dtype=dtype), (kp.to(DEV, dtype), vp.to(DEV, dtype)), b.on(DEV), dtype, DEV, b, H, G, d, dv,
                 8, dict(chunk=20, zero_sink=True, softcap=4.0, talk=True), talk.to(DEV)).float().cpu().view(rows, H, dv)
    for r in range(rows):
        n = (41 + r) % 20 + 1
        want = n / (n + 1) * torch.tensor([1.0, -1.0, 20.0, 0.0])
        assert torch.allclose(got[r], want[:, None].expand(H, dv), atol=0.08 if dtype == BF16 else 1e-4)


# ---------------------------------------------------------------------------------------------
# recurrences whose gates the token chooses
# ---------------------------------------------------------------------------------------------
LONG = [(0, 1), (5, 2), (0, 15), (9, 16), (0, 17), (3, 33), (0, 255), (40, 256), (0, 257), (7, 600)]


def run_gated(o, dev, kind, b, joint, z, bias, tau, state, heads, dim, vdim, **kw):
    _, row_seg, seg_start, slots, _ = b.on(dev)
    st, out = state.to(dev), torch.full((b.rows, heads * vdim), float("nan"), dtype=F64 if kind == F64 else F32, device=dev)
    if kind == F64:
        st = st.double()
    o.gated_linear_attention(joint.to(dev, kind), z.to(dev), bias.to(dev), tau, 0.3, st, row_seg, seg_start, slots, out, heads, dim, vdim, **kw)
    return out, st


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("form", ["tokens", "auto"])
@pytest.mark.parametrize("speed", ["slow", "fast", "extreme"])
@pytest.mark.parametrize("heads,dim,vdim", [(2, 64, 64), (1, 128, 48), (3, 16, 16), (2, 96, 32), (3, 9, 7), (1, 200, 12)])
def test_gated_linear_attention_in_all_forms(ops, ref, heads, dim, vdim, speed, form, dtype):
    """"fast": decays of e^-3 a token and channel here and there (a chunk's product under e^-40: its scores are summed term by term);
    "extreme": e^-60 and more, whose products underflow and whose reciprocals would not be numbers."""
    segments = LONG if dim in (64, 96, 9) else [(0, 3), (4, 1), (0, 40), (8, 300)]
    b = Batch(segments, 16, dim)
    g = gen(heads + dim)
    joint = torch.randn(b.rows, heads * (2 * dim + vdim) + 8, generator=g).to(dtype)
    z = torch.randn(b.rows, heads * dim, generator=g) * 2
    if speed != "slow":
        hit = torch.rand(b.rows, heads * dim, generator=g) < 0.2
        z = torch.where(hit, torch.full_like(z, -12.0 if speed == "fast" else -250.0), z)
    bias = torch.randn(heads * dim, generator=g)
    state = torch.randn(b.num_slots, heads, dim, vdim, generator=g)
    want, want_state = run_gated(ref, "cpu", F64, b, joint, z, bias, 4.0, state, heads, dim, vdim)
    got, got_state = run_gated(ops, DEV, dtype, b, joint, z, bias, 4.0, state, heads, dim, vdim, form=form)
    tol = 3e-5 if dtype == F32 else 2e-4          # bfloat16: operands are exact in it, only the hardware's exponentials differ
    close(got, want, tol, tol * want.abs().max().item(), "outputs")
    close(got_state, want_state, tol, tol * want_state.abs().max().item(), "states")
    unused = sorted(set(range(b.num_slots)) - set(b.slots.tolist()))
    assert torch.equal(got_state[unused].cpu(), state[unused]), "slots of no request were touched"


@pytest.mark.parametrize("far", [0, 15, 16, 255, 256, 511, 598])
@pytest.mark.parametrize("decoded", [False, True])
def test_one_far_key_arrives_through_the_product_of_its_channels_decays(ops, far, decoded):
    """600 tokens, key and value of one alone are not zero: what the last token reads of it is the product of its channel's decays
    since, across chunks and parts of the kernel, or token after token."""
    dim, vdim, T = 32, 16, 600
    g = gen(far)
    joint = torch.zeros(T, 2 * dim + vdim)
    joint[far, dim:2 * dim] = torch.arange(1, dim + 1, dtype=F32) / dim
    joint[far, 2 * dim:] = 2.0
    joint[-1, 5] = 1.0                                       # the last query reads channel 5
    z = torch.rand(T, dim, generator=g) + 3.0
    bias, state = torch.zeros(dim), torch.zeros(1, 1, dim, vdim)
    st = state.to(DEV)
    out = torch.empty(T, vdim, device=DEV)
    cuts = [T] if not decoded else [590] + [1] * 10
    at = 0
    for n in cuts:
        i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)
        ops.gated_linear_attention(joint[at:at + n].to(DEV).contiguous(), z[at:at + n].to(DEV).contiguous(), bias.to(DEV), 2.0, 1.0, st,
                                   torch.zeros(n, dtype=torch.int32, device=DEV), i32([0, n]), i32([0]), out[at:at + n], 1, dim, vdim)
        at += n
    decay = torch.sigmoid(z[far + 1:, 5].double()).pow(0.5).prod().item()
    want = decay * 6 / dim * 2.0
    assert abs(out[-1, 0].item() - want) <= 2e-5 * want


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("width", [7, 64, 200, 1030])
@pytest.mark.parametrize("segments", [LONG, [(0, 1), (7, 1), (3, 1)], [(0, 64), (2, 65), (0, 63)], [(0, 3), (1, 40)]])
def test_min_recurrence_in_parts_and_single_rows(ops, ref, width, segments, dtype):
    b = Batch(segments, 16, width)
    g = gen(width)
    zxg = torch.randn(b.rows, 3 * width, generator=g).to(dtype)
    zxg[:, :width] -= 2.0                                    # slow gates: the state reaches back over parts
    bias, state = torch.randn(2 * width, generator=g), torch.randn(b.num_slots, width, generator=g)
    results = []
    for o, dev, kind in ((ref, "cpu", F64), (ops, DEV, dtype)):
        _, row_seg, seg_start, slots, _ = b.on(dev)
        st, out = state.to(dev), torch.full((b.rows, width), float("nan"), dtype=kind, device=dev)
        st = st.double() if kind == F64 else st
        o.min_recurrence(zxg.to(dev, kind), bias.to(dev), st, row_seg, seg_start, slots, out)
        results.append((out, st))
    close(results[1][0], results[0][0], *((1e-5, 1e-5) if dtype == F32 else (BF16_EPS, 1e-3)), "outputs")
    close(results[1][1], results[0][1], 1e-5, 1e-5, "states")


# ---------------------------------------------------------------------------------------------
# the engine
# ---------------------------------------------------------------------------------------------
LENGTHS = {"A": [5, 30, 61, 120], "B": [45, 83, 2], "C": [9, 50, 77], "D": [100, 37, 260]}
TOL = {"float32": 2e-5, "bfloat16": 4e-2}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """(configuration, precision) -> folder, configuration, requests, plain logits, weights.  float32 runs random routers;
    bfloat16 runs routers whose every pick has a margin, since a pick that flips under rounding is a large error that says
    nothing about the kernels."""
    out = {}
    for name, cfg in zc.CONFIGS.items():
        for dtype in ("float32", "bfloat16"):
            # A side input of few lanes is divided by its own size: where all of them are nearly zero, the logits follow the last bit
            # of every sum before it.  float32 runs a seed under which no position is such a one, bfloat16 more lanes as well.
            if dtype == "bfloat16":
                cfg = dict(cfg, token_side={"dim": 16})
            tensors = zc.weights(cfg, 32 + ord(name), decided_router=dtype == "bfloat16")
            folder = zc.write_model(str(tmp_path_factory.mktemp(f"zoguzen_{name}_{dtype}")), cfg, tensors)
            requests = {f"r{i}": zc.random_ids(n, cfg["vocab"], 100 * ord(name) + i) for i, n in enumerate(LENGTHS[name])}
            w64 = zc.to_float64(tensors)
            plain = {rid: pz.forward(cfg, w64, toks) for rid, toks in requests.items()}
            out[name, dtype] = (folder, cfg, requests, plain, w64)
    return out


def make_runner(folder, dtype, page_size, max_tokens, **kw):
    from fllm_amd.engine import ModelRunner
    return ModelRunner.from_folder(folder, dtype=dtype, page_size=page_size, max_tokens=max_tokens, max_requests=4, **kw)


def check(got, plain, dtype, what):
    for rid, want in plain.items():
        assert rid in got and got[rid].shape == want.shape, f"{what}: request {rid}"
        err = np.abs(got[rid].astype(np.float64) - want)
        scale = np.abs(want).max()
        tt.observe(f"zoguzen {what.split()[0]} {dtype}", err.max() / scale)
        over = err.max(axis=1) > TOL[dtype] * scale
        assert not over.any(), (f"{what}: request {rid}: max error {err.max():.3e} (limit {TOL[dtype] * scale:.3e}); first "
                                f"position over the limit: {int(np.argmax(over))}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
@pytest.mark.parametrize("family", ["whole", "last40", "portions", "mixed"])
def test_replay(models, tmp_path, name, dtype, family):
    folder, cfg, requests, plain, _ = models[name, dtype]
    refed = [rid for rid, toks in requests.items() if len(toks) >= 60][:1]
    steps = {"whole": tt.whole, "last40": lambda r: tt.last_tokens_one_by_one(r, 40), "portions": tt.portions,
             "mixed": lambda r: tt.mixed(r, seed=5, refeed=refed)}[family](requests)
    steps = tt.number(steps)
    runner = make_runner(folder, dtype, zc.PAGE_SIZES[name], tt.live_tokens_bound(steps))
    handed_out = tt.record_allocations(runner.cache)
    got = tt.run_in_process(runner, steps, cfg["vocab"], str(tmp_path))
    check(got, plain, dtype, f"{family} {name} {dtype}")
    runner.cache.check_invariants()
    assert all(pool.available == pool.num_pages for pool in runner.cache.pools), "pages were lost"
    if family == "mixed":
        assert all(len(pages) > len(set(pages)) for pages in handed_out), "the trace was meant to use pages again"


@pytest.mark.parametrize("page_size", [4, 32, 64])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_replay_at_other_page_sizes(models, tmp_path, page_size, dtype):
    folder, cfg, requests, plain, _ = models["D", dtype]
    steps = tt.number(tt.mixed(requests, seed=8))
    runner = make_runner(folder, dtype, page_size, tt.live_tokens_bound(steps, round_to=max(64, page_size)))
    got = tt.run_in_process(runner, steps, cfg["vocab"], str(tmp_path))
    check(got, plain, dtype, f"pages-of-{page_size} D {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "D"])
def test_first_tokens_and_long_decoding(models, tmp_path, name, dtype):
    """Token by token from the very first token, across windows and chunks."""
    folder, cfg, requests, plain, _ = models[name, dtype]
    rid = max(requests, key=lambda r: len(requests[r]))
    steps = tt.number(tt.last_tokens_one_by_one({rid: requests[rid]}, tail=len(requests[rid])))
    runner = make_runner(folder, dtype, zc.PAGE_SIZES[name], 320)
    got = tt.run_in_process(runner, steps, cfg["vocab"], str(tmp_path))
    check(got, {rid: plain[rid]}, dtype, f"token-by-token {name} {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "C", "D"])
def test_decode_graphs_and_eager_steps_agree(models, tmp_path, name, dtype):
    folder, cfg, requests, plain, _ = models[name, dtype]
    steps = tt.number(tt.last_tokens_one_by_one(requests) + tt.mixed(requests, seed=21, decode_tail=40))
    results = []
    for i, use_graphs in enumerate((True, False)):
        runner = make_runner(folder, dtype, zc.PAGE_SIZES[name], tt.live_tokens_bound(steps), use_graphs=use_graphs)
        results.append(tt.run_in_process(runner, steps, cfg["vocab"], str(tmp_path / str(i))))
        assert (runner.graph_replays > 30) == use_graphs
    for rid, want in plain.items():
        a, b = results[0][rid].astype(np.float64), results[1][rid].astype(np.float64)
        if dtype == "float32":
            assert np.array_equal(a, b), f"{rid}: graph and eager steps differ in float32"
        else:
            assert np.abs(a - b).max() <= TOL[dtype] * np.abs(want).max()
    check(results[0], plain, dtype, f"graphs {name} {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_long_prompt_whole_and_in_portions(models, tmp_path, dtype):
    """1,100 tokens in one step, in two portions, and with the last 40 decoded one by one: states carried over a thousand tokens, the
    first tokens a thousand positions back, twenty chunks."""
    folder, cfg, _, _, w64 = models["D", dtype]
    toks = zc.random_ids(1100, cfg["vocab"], 77)
    want = {"long": pz.forward(cfg, w64, toks)}
    from fllm_amd.engine import StepEntry
    for cuts in ([1100], [600, 500], [1060] + [1] * 40):
        runner = make_runner(folder, dtype, 16, 1152, max_context=2048)
        got, at = [], 0
        for n in cuts:
            got.append(runner.step([StepEntry("long", toks[at:at + n], list(range(n)))]).float().cpu().numpy())
            at += n
        check({"long": np.concatenate(got)}, want, dtype, f"long-prompt-{len(cuts)} D {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_program(models, tmp_path, dtype):
    folder, cfg, requests, plain, _ = models["A", dtype]
    steps = tt.number(tt.mixed(requests, seed=9))
    got = tt.run_subprocess(folder, dtype, steps, cfg["vocab"], str(tmp_path), tt.live_tokens_bound(steps))
    check(got, plain, dtype, f"trace_run A {dtype}")


def test_the_residual_stream_after_every_layer(models):
    folder, cfg, requests, plain, w64 = models["A", "float32"]
    runner = make_runner(folder, "float32", 8, 320)
    from fllm_amd.engine import StepEntry
    seen = []
    for block in runner.model.blocks:
        def wrapped(ctx, x, binding, _inner=block.forward):
            _inner(ctx, x, binding)
            seen.append(x.clone().cpu().numpy())
        block.forward = wrapped
    toks = requests["r2"]
    runner.step([StepEntry("a", toks, [])])
    want, _ = pz.layer_outputs(cfg, w64, toks)
    assert len(seen) == len(want) == 4
    for got, ref_x in zip(seen, want):
        assert np.abs(got - ref_x).max() <= 1e-5 * np.abs(ref_x).max()


def test_decode_steps_take_the_fused_forms_and_prompts_the_tile_kernels(models, monkeypatch):
    """D in bfloat16: a decode step norms a row for both branches and shifts the mixer's input in one kernel, gates the side input in
    another, and runs no norm of its own but the model's last; a prompt's experts go to the matrix cores grouped by expert."""
    from fllm_amd.engine import StepEntry
    from fllm_amd.kernels import Ops
    folder, cfg, requests, _, _ = models["D", "bfloat16"]
    runner = make_runner(folder, "bfloat16", 16, 256, use_graphs=False)
    kinds = [layer["type"] for layer in cfg["layers"]]
    pairs, chunks, grus = (kinds.count(k) for k in ("parallel", "attention", "mingru"))
    routed = sum(1 for layer in cfg["layers"] if layer["mlp"])
    calls = []
    for name in ("layernorm", "layernorm_pair", "layernorm_conv", "short_conv", "side_gate", "gelu_side", "cast_rows", "conv_qkv_store",
                 "masked_attention", "gated_linear_attention", "min_recurrence", "normed_pair_sum", "experts_grouped", "experts_gate_up"):
        inner = getattr(Ops, name)
        monkeypatch.setattr(Ops, name, lambda self, *a, _n=name, _i=inner, **k: (calls.append(_n), _i(self, *a, **k))[1])
    toks = requests["r0"]
    runner.step([StepEntry("a", toks[:40], [])])
    assert calls.count("layernorm_pair") == routed and calls.count("short_conv") == len(kinds) and calls.count("layernorm_conv") == 0
    assert calls.count("experts_grouped") == routed and calls.count("experts_gate_up") == 0 and calls.count("gelu_side") == len(kinds)
    assert calls.count("conv_qkv_store") == calls.count("masked_attention") == pairs + chunks
    assert calls.count("gated_linear_attention") == calls.count("normed_pair_sum") == pairs and calls.count("min_recurrence") == grus
    calls.clear()
    runner.step([StepEntry("a", toks[40:41], [0])])
    assert calls.count("layernorm_conv") == calls.count("side_gate") == len(kinds)
    assert calls.count("layernorm") == 1 and not set(calls) & {"layernorm_pair", "short_conv", "cast_rows", "gelu_side"}
    assert calls.count("conv_qkv_store") == calls.count("masked_attention") == pairs + chunks


@pytest.mark.parametrize("name", ["A", "D"])
def test_greedy_generation_through_the_scheduler(models, name):
    from fllm_amd import Engine, SamplingParams
    folder, cfg, _, _, w64 = models[name, "float32"]
    prompts = [zc.random_ids(n, cfg["vocab"], 20 + n) for n in (3, 26, 41, 90)]
    want = []
    for p in prompts:
        toks = list(p)
        for _ in range(10):
            toks.append(int(np.argmax(pz.forward(cfg, w64, toks)[-1])))
        want.append(toks[len(p):])
    for opts in (dict(num_blocks=64), dict(num_blocks=14, max_batched_tokens=16)):
        engine = Engine(folder, dtype="float32", ctx=256, max_seqs=3, block_size=zc.PAGE_SIZES[name],
                        **{"max_batched_tokens": 64, **opts})
        assert engine.generate(prompts, SamplingParams(max_tokens=10)) == want
        engine.runner.cache.check_invariants()
    folder, cfg, _, _, w64 = models[name, "bfloat16"]
    engine = Engine(folder, dtype="bfloat16", ctx=256, max_seqs=4, block_size=zc.PAGE_SIZES[name])
    out = engine.generate(prompts, SamplingParams(max_tokens=10))
    assert [len(o) for o in out] == [10] * 4


def test_the_command_line_generates(models):
    folder, cfg, _, _, w64 = models["A", "float32"]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    prompt = zc.random_ids(30, cfg["vocab"], 4)
    cmd = [sys.executable, "-m", "fllm_amd", "run", folder, "--prompt-ids", ",".join(map(str, prompt)), "--max-tokens", "8",
           "--dtype", "float32", "--ctx", "256", "--kv-blocks", "32", "--max-seqs", "2"]
    proc = subprocess.run(cmd, cwd=root, capture_output=True, text=True, timeout=110)
    assert proc.returncode == 0, proc.stderr[-2000:]
    record = json.loads(proc.stdout.strip().splitlines()[0])
    toks = list(prompt)
    for _ in range(8):
        toks.append(int(np.argmax(pz.forward(cfg, w64, toks)[-1])))
    assert record["finish_reason"] == "length" and record["token_ids"] == toks[30:]
    proc = subprocess.run([sys.executable, "-m", "fllm_amd", "inspect", folder], cwd=root, capture_output=True, text=True, timeout=110)
    assert proc.returncode == 0 and "architecture: zoguzen" in proc.stdout
