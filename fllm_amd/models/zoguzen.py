"""Zoguzen: the description of the architecture in terms of parts.

x = E[token].  A layer adds both of its branches to the same stream, x += mixer(ln_1(x)) + ff(ln_2(x)), ln a layer norm with a
weight and no bias (`parts/norm.py: LayerNorm`, `parts/block.py: ParallelBlock`), and then what the token itself brings: x +=
rms(W_p (gelu(W_g x) * t_i)), t_i the layer's part of the token's row in a table of its own (`parts/token_side.py`).  What a
mixer reads moves towards the token's before it, lane by lane (`parts/conv_input.py`, the shift).  Three mixers.  "attention":
grouped-query attention without positions whose biased q, k and v pass a short convolution over time, every head of q and of k
normed with one weight vector, scores capped, keys of the row's own chunk, a sink of score 0, and the heads' softmax weights
mixed across heads before they meet the values; a layer may read the keys and values of an earlier one
(`parts/conv_attention.py`).  "mingru": a gated recurrence lane by lane whose gates read the current token alone
(`parts/min_gru.py`).  "parallel": two mixers on the same input, half the sum of their outputs, each behind an RMS norm
(`parts/pair.py`): on the left attention with convolved and rotated q and k over a window that keeps the first tokens, with an
output gate (`parts/conv_attention.py`); on the right linear attention with a decay a key channel that the token chooses
(`parts/gated_linear.py`).  The feed-forward is a set of small gated experts under a router whose weights are the softmax over
the picked logits (`parts/experts.py`).  logits = cap * tanh(E ln(x) / cap) with the embedding table itself.

Tensor names: `embed`, `side.embed`, `final.norm`, and per layer `l<i>.norm1`, `l<i>.norm2`, `l<i>.shift`,
`l<i>.side.{gate,proj,norm}`, `l<i>.mix.*` (q, k, v with `.b` and `.conv`, `q.norm`, `k.norm`, `talk`, o; or z, x with `.b`, g,
o; or `left.*`, `right.*` with `left.out` and `right.out`) and `l<i>.mlp.router`, `l<i>.mlp.e<j>.{gate,up,down}`.
"""
from __future__ import annotations

from ..config.spec import LayerSpec, ModelSpec, PartSpec, RunEntry
from ..config.zoguzen import ZoguzenConfig
from ..registry import Architecture, register_architecture


def _position(rot, max_position):
    if rot is None:
        return None
    position = {"kind": "rotary", "dims": rot.dims, "theta": rot.base, "pairing": "interleaved", "scaling": "none",
                "max_position": max_position, "precise": True}
    if rot.scaling is not None:
        s = rot.scaling
        position.update(scaling="llama3", factor=s.factor, low_freq_factor=s.low, high_freq_factor=s.high,
                        original_max_position=s.original)
    return position


def _attention(cfg, a, p: str, left: bool) -> PartSpec:
    own = ("q",) if a.kv_from is not None else ("q", "k", "v")
    names = {n: f"{p}{n}" for n in own + ("o",)}
    names.update({f"{n}_conv": f"{p}{n}.conv" for n in own})
    params = {"hidden_size": cfg.width, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim, "value_head_dim": a.vdim,
              "scale": a.scale, "taps": a.taps, "own_keys": a.kv_from is None}
    if left:
        names["g"] = f"{p}g"
        params.update(window=a.size, keep_first=a.keep_first, position=_position(a.rot, cfg.max_position), output_gate=True)
    else:
        names.update({f"{n}_bias": f"{p}{n}.b" for n in own})
        names.update({f"{n}_norm": f"{p}{n}.norm" for n in own if n != "v"}, talk=f"{p}talk")
        params.update(chunk=a.size, softcap=a.softcap, qk_norm_eps=cfg.eps, sink="zero", mix_weights=True)
    return PartSpec("conv_attention", params, names)


def _mixer(cfg: ZoguzenConfig, m, p: str) -> PartSpec:
    if m.kind == "attention":
        return _attention(cfg, m.attention, p, False)
    if m.kind == "mingru":
        return PartSpec("min_gru", {"hidden_size": cfg.width, "size": m.width},
                        {"z": f"{p}z", "x": f"{p}x", "g": f"{p}g", "o": f"{p}o", "z_bias": f"{p}z.b", "x_bias": f"{p}x.b"})
    r = m.linear
    left = _attention(cfg, m.attention, f"{p}left.", True)
    right = PartSpec("gated_linear",
                     {"hidden_size": cfg.width, "num_heads": r.heads, "head_dim": r.dim, "value_head_dim": r.vdim, "tau": r.tau,
                      "query_scale": r.dim ** -0.5, "eps": cfg.eps},
                     {"q": f"{p}right.q", "k": f"{p}right.k", "v": f"{p}right.v", "g": f"{p}right.g", "o": f"{p}right.o",
                      "norm": f"{p}right.norm", "a1": f"{p}right.a1", "a2": f"{p}right.a2", "a2_bias": f"{p}right.a2.b"})
    tensors = {"left." + n: t for n, t in left.tensors.items()}
    tensors.update({"right." + n: t for n, t in right.tensors.items()})
    tensors.update(left_out=f"{p}left.out", right_out=f"{p}right.out")
    return PartSpec("mixer_pair", {"size": cfg.width, "left": left, "right": right, "left_scale": 0.5, "right_scale": 0.5,
                                   "out_norm_eps": cfg.eps}, tensors)


def build_spec(cfg: ZoguzenConfig) -> ModelSpec:
    layers, order = [], []
    ignorable = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}"
        norm = lambda name: PartSpec("layer", {"size": cfg.width, "eps": cfg.eps}, {"weight": f"{p}.{name}"})
        inner = _mixer(cfg, layer.mixer, f"{p}.mix.")
        mixer = PartSpec("conv_input", {"size": cfg.width, "form": "shift", "inner": inner},
                         dict({"inner." + n: t for n, t in inner.tensors.items()}, shift=f"{p}.shift"))
        norms = {"mixer": norm("norm1")}
        ffn = None
        if layer.mlp is None:
            ignorable.append(f"{p}.norm2")
        else:
            norms["feed_forward"] = norm("norm2")
            names = {"router": f"{p}.mlp.router"}
            for e in range(layer.mlp.experts):
                names.update({f"{n}_{e}": f"{p}.mlp.e{e}.{n}" for n in ("gate", "up", "down")})
            # the softmax over all logits, divided by the picks' sum, is the softmax over the picked logits
            ffn = PartSpec("routed_experts",
                           {"hidden_size": cfg.width, "intermediate_size": layer.mlp.ff, "experts": layer.mlp.experts,
                            "top": layer.mlp.top, "score": "softmax", "renormalize": True, "weight_on": "output"}, names)
        side = PartSpec("token_side", {"size": cfg.width, "dim": cfg.side_dim, "vocab_size": cfg.vocab, "layers": len(cfg.layers),
                                       "layer": i, "eps": cfg.eps},
                        {"table": "side.embed", "gate": f"{p}.side.gate", "proj": f"{p}.side.proj", "norm": f"{p}.side.norm"})
        layers.append(LayerSpec(block=PartSpec("parallel"), mixer=mixer, feed_forward=ffn, norms=norms,
                                extras={"after": ("stream", side)}))
        source = layer.mixer.attention.kv_from if layer.mixer.kind == "attention" else None
        order.append(RunEntry(layer=i, reads_cache_of=source))       # every layer runs once: entry i is layer i
    table = {"weight": "embed"}
    return ModelSpec(
        architecture="zoguzen",
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        max_position=cfg.max_position,
        embedding=PartSpec("table", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "scale": 1.0}, table),
        layers=tuple(layers),
        run_order=tuple(order),
        final_norm=PartSpec("layer", {"size": cfg.width, "eps": cfg.eps}, {"weight": "final.norm"}),
        head=PartSpec("linear", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "softcap": cfg.logit_softcap}, table),
        ignorable_tensors=tuple(ignorable),
    )


register_architecture(Architecture(
    model_type="zoguzen",
    hf_architectures=(),
    parse_config=ZoguzenConfig.from_dict,
    build_spec=build_spec,
))
