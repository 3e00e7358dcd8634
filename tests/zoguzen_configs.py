"""Tiny Zoguzen configurations and weights for tests.  The weights are drawn here, larger than a checkpoint's random init, so
that scores differ between keys and experts, and windows, first tokens, chunks, sinks, mixed heads and gates are felt."""
import json
import os

import numpy as np
import torch


def _mlp(mlp):
    """None or (ff, experts, top)."""
    return None if mlp is None else {"kind": "moe", "expert": {"ff": mlp[0]}, "router": {"experts": mlp[1], "top": mlp[2]}}


def chunked(heads, kv_heads, dim, vdim, taps, size, softcap, scale=None, kv_from=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps, "mask": {"size": size}, "softcap": softcap,
         "scale": scale or dim ** -0.5}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": _mlp(mlp)}


def mingru(width, mlp=None):
    return {"type": "mingru", "mixer": {"width": width}, "mlp": _mlp(mlp)}


def pair(left, right, mlp=None):
    """left: (heads, kv_heads, dim, vdim, taps, window, first tokens, rot, scale); right: (heads, dim, vdim, tau)."""
    heads, kv_heads, dim, vdim, taps, size, first, rot, scale = left
    L = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps, "mask": {"size": size, "keep_first": first}, "scale": scale}
    if rot is not None:
        L["rot"] = rot
    return {"type": "parallel", "mlp": _mlp(mlp), "mixer": {"left": L, "right": dict(zip(("heads", "dim", "vdim", "tau"), right))}}


def rot(dims, base, scaling=None):
    out = {"dims": dims, "base": base}
    if scaling is not None:
        out["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return out


def config(width, vocab, layers, side, cap, eps=1e-5):
    return {"architecture": "Zoguzen", "width": width, "vocab": vocab, "norm": {"eps": eps}, "logit_softcap": cap, "token_side": {"dim": side},
            "layers": layers}


WAVES = (4.0, 1.0, 4.0, 32)        # a short original context, so that kept, blended and divided frequencies all occur
# A: all three mixers, a layer that reads another's keys and values, a layer without feed-forward, keys and values of two widths
A = config(48, 90, [
    chunked(4, 2, 16, 24, 3, 12, 6.0, mlp=(24, 4, 2)),
    pair((4, 1, 16, 16, 4, 7, 3, rot(8, 100.0, WAVES), 0.3), (2, 12, 20, 4.0), mlp=(24, 4, 2)),
    chunked(4, 2, 16, 24, 3, 9, 9.0, kv_from=0, scale=0.4),
    mingru(40, mlp=(20, 6, 3)),
], side=8, cap=12.0)
# B: the smallest of everything: one tap, chunks of one position, a window of one with no first tokens kept, one head, every expert
# picked, a single expert, as many key/value heads as heads, full rotation without scaling
B = config(64, 77, [
    mingru(7, mlp=(16, 1, 1)),
    chunked(3, 3, 8, 8, 1, 1, 40.0, mlp=(16, 3, 3)),
    pair((1, 1, 32, 24, 1, 1, 0, rot(32, 10000.0), 0.2), (1, 16, 16, 1.0), mlp=(16, 3, 3)),
    chunked(3, 3, 8, 8, 6, 200, 2.0, kv_from=1),
], side=1, cap=40.0, eps=1e-6)
# C: sizes that are multiples of nothing (keys lie lane by lane in the pages), three heads on one key/value head, a source with two
# readers behind other layers, more first tokens than the window has positions
C = config(52, 61, [
    chunked(3, 1, 10, 6, 4, 11, 5.0, scale=0.5, mlp=(18, 5, 2)),
    pair((3, 1, 10, 14, 2, 5, 9, rot(6, 30.0, WAVES), 0.4), (3, 9, 7, 0.5), mlp=(18, 5, 2)),
    chunked(3, 1, 10, 6, 4, 30, 3.0, kv_from=0, mlp=(18, 5, 2)),
    chunked(3, 1, 10, 6, 2, 7, 8.0, kv_from=0),
    pair((2, 2, 12, 5, 5, 3, 1, None, 0.3), (2, 5, 11, 3.0)),
], side=5, cap=9.0)
# D: head sizes that the matrix-core kernels take, chunks and windows of several pages
D = config(128, 160, [
    chunked(8, 2, 64, 64, 4, 50, 30.0, mlp=(48, 8, 3)),
    mingru(192, mlp=(48, 8, 3)),
    pair((8, 4, 64, 32, 3, 45, 21, rot(64, 20000.0, (8.0, 1.0, 4.0, 64)), 0.125), (4, 64, 32, 8.0), mlp=(48, 8, 3)),
    chunked(8, 2, 64, 64, 2, 70, 30.0, kv_from=0),
    pair((6, 3, 32, 96, 4, 33, 5, rot(16, 500.0), 0.2), (3, 96, 48, 16.0), mlp=(48, 8, 3)),
], side=16, cap=25.0, eps=1e-6)
CONFIGS = {"A": A, "B": B, "C": C, "D": D}
PAGE_SIZES = {"A": 8, "B": 4, "C": 16, "D": 16}


def bf16_round(a):
    return torch.from_numpy(np.asarray(a, dtype=np.float32)).to(torch.bfloat16).to(torch.float32)


def weights(cfg, seed, decided_router=False, rank=6):
    """name -> float32 torch tensor whose values are exact in bfloat16 (both precisions load the same numbers).

    `decided_router`: for comparisons in bfloat16, where a random router has close calls that rounding flips, which is a large
    error that says nothing about the kernels.  Two lanes of the stream then carry a direction that depends on the token alone
    (nothing else is added to them), and the router rows look at these two lanes only, row e along the angle 2 pi e / E, the
    tokens' angles a quarter of the way between two experts: every pick has a margin far above the rounding."""
    rng = np.random.default_rng(seed)
    W, side, n = cfg["width"], cfg["token_side"]["dim"], len(cfg["layers"])
    out = {"embed": rng.normal(0, 0.7, (cfg["vocab"], W)), "final.norm": 1 + rng.uniform(-0.3, 0.3, W),
           "side.embed": rng.normal(0, 1.0, (cfg["vocab"], n * side))}
    counts = {spec["mlp"]["router"]["experts"] for spec in cfg["layers"] if spec["mlp"]}
    if decided_router:
        E = max(counts)
        angle = (np.arange(cfg["vocab"]) % (2 * E) + 0.5) * np.pi / E
        out["embed"][:, 0], out["embed"][:, 1] = 4.0 * np.cos(angle), 4.0 * np.sin(angle)

    def projection(p, name, size, taps=None, bias=False, gain=1.5):
        out[p + name] = rng.normal(0, gain * W ** -0.5, (size, W))
        if bias:
            out[p + name + ".b"] = rng.normal(0, 0.5, size)
        if taps is not None:      # the newest tap leads, the others are felt
            out[p + name + ".conv"] = rng.normal(0, 0.4, (size, taps)) + np.eye(taps)[-1]

    def back(p, name, size):
        out[p + name] = rng.normal(0, size ** -0.5, (W, size))
        if decided_router:
            out[p + name][:2] = 0.0

    for i, spec in enumerate(cfg["layers"]):
        m, p = spec["mixer"], f"l{i}."
        out[p + "norm1"] = 1 + rng.uniform(-0.3, 0.3, W)
        out[p + "shift"] = rng.uniform(0.0, 1.0, W)
        out[p + "side.gate"] = rng.normal(0, 1.5 * W ** -0.5, (side, W))
        out[p + "side.proj"] = rng.normal(0, side ** -0.5, (W, side))
        out[p + "side.norm"] = 0.3 + rng.uniform(-0.2, 0.2, W)
        if decided_router:
            out[p + "side.norm"][:2] = 0.0
        mp = p + "mix."
        if spec["type"] == "attention":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            projection(mp, "q", H * d, m["conv"], True)
            out[mp + "q.norm"] = 1.5 + rng.uniform(-0.5, 0.5, d)
            if m.get("kv_from") is None:
                projection(mp, "k", G * d, m["conv"], True)
                projection(mp, "v", G * dv, m["conv"], True, gain=1.0)
                out[mp + "k.norm"] = 1.5 + rng.uniform(-0.5, 0.5, d)
            out[mp + "talk"] = np.eye(H) * 0.8 + rng.normal(0, 0.4, (H, H))
            back(mp, "o", H * dv)
        elif spec["type"] == "mingru":
            projection(mp, "z", m["width"], bias=True)
            projection(mp, "x", m["width"], bias=True)
            projection(mp, "g", m["width"])
            back(mp, "o", m["width"])
            out[mp + "z.b"] -= 1.0                  # slow gates: the state reaches back
        else:
            L, R, lp, rp = m["left"], m["right"], mp + "left.", mp + "right."
            projection(lp, "q", L["heads"] * L["dim"], L["conv"], gain=2.0)
            projection(lp, "k", L["kv_heads"] * L["dim"], L["conv"], gain=2.0)
            projection(lp, "v", L["kv_heads"] * L["vdim"], L["conv"])
            projection(lp, "g", L["heads"] * L["vdim"])
            out[lp + "o"] = rng.normal(0, (L["heads"] * L["vdim"]) ** -0.5, (W, L["heads"] * L["vdim"]))
            H, d, dv = R["heads"], R["dim"], R["vdim"]
            projection(rp, "q", H * d)
            # keys lean towards their own queries: the sign of a first token's output, all that the norm of a head keeps of it, is
            # no close call then
            out[rp + "k"] = 0.6 * out[rp + "q"] + 0.8 * rng.normal(0, 1.5 * W ** -0.5, (H * d, W))
            projection(rp, "v", H * dv)
            projection(rp, "g", H * dv)
            out[rp + "a1"] = rng.normal(0, W ** -0.5, (rank, W))
            out[rp + "a2"] = rng.normal(0, 1.5 * rank ** -0.5, (H * d, rank))
            out[rp + "a2.b"] = rng.normal(1.5, 1.0, H * d)
            out[rp + "norm"] = 1 + rng.uniform(-0.3, 0.3, dv)
            out[rp + "o"] = rng.normal(0, (H * dv) ** -0.5, (W, H * dv))
            for name in ("left.out", "right.out"):
                out[mp + name] = 1 + rng.uniform(-0.3, 0.3, W)
                if decided_router:
                    out[mp + name][:2] = 0.0
        mlp = spec["mlp"]
        if mlp is None:
            continue
        out[p + "norm2"] = 1 + rng.uniform(-0.3, 0.3, W)
        ff, E = mlp["expert"]["ff"], mlp["router"]["experts"]
        out[p + "mlp.router"] = rng.normal(0, 1.5 * W ** -0.5, (E, W))
        if decided_router:
            out[p + "norm2"][:2] = 1.0
            at = 2 * np.pi * np.arange(E) / E
            out[p + "mlp.router"][:] = 0.0
            out[p + "mlp.router"][:, 0], out[p + "mlp.router"][:, 1] = 0.6 * np.cos(at), 0.6 * np.sin(at)
        for e in range(E):
            out[f"{p}mlp.e{e}.gate"] = rng.normal(0, 1.5 * W ** -0.5, (ff, W))
            out[f"{p}mlp.e{e}.up"] = rng.normal(0, 1.5 * W ** -0.5, (ff, W))
            back(p, f"mlp.e{e}.down", ff)
    return {k: bf16_round(a) for k, a in out.items()}


def to_float64(tensors):
    return {n: t.to(torch.float64).numpy() for n, t in tensors.items()}


def write_model(folder, cfg, tensors, dtype=torch.bfloat16):
    from fllm_amd.weights.safetensors_io import write_safetensors
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    write_safetensors(os.path.join(folder, "model.safetensors"), {n: t.to(dtype) for n, t in tensors.items()})
    return folder


def random_ids(n, vocab, seed):
    return np.random.default_rng(seed).integers(0, vocab, size=n).tolist()
