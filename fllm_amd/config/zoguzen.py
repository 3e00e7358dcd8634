"""Typed configuration of the Zoguzen architecture, read from a checkpoint's config.json.

The file names the design under `architecture`; sizes and constants are nested by what they belong to: `width`, `vocab`,
`norm.eps`, `logit_softcap`, `token_side.dim` and `layers`, a list whose entries give the mixer's `type` ("attention",
"mingru" or "parallel"), its sizes under `mixer`, and the feed-forward under `mlp` (null: none): `kind` "moe" with `expert.ff`
and `router` {experts, top}.  Mixer sizes: "attention" {heads, kv_heads, dim, vdim, conv (taps), scale, softcap, `mask` {size},
kv_from (absent: the layer has keys and values of its own)}; "mingru" {width}; "parallel" {`left` {heads, kv_heads, dim, vdim,
conv, scale, `rot` {base, dims, `scaling` {factor, low, high, original}}, `mask` {size, keep_first}}, `right` {heads, dim,
vdim, tau}}.  Everything is checked here, before any weight is read.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .menitar import DEFAULT_MAX_POSITION, _need, _positive
from .spec import ConfigError


@dataclass(frozen=True)
class WaveScaling:
    """Rotary frequencies whose wavelength is below original / high stay, those above original / low are divided by `factor`,
    those between are blended."""
    factor: float
    low: float
    high: float
    original: float


@dataclass(frozen=True)
class Rotation:
    dims: int
    base: float
    scaling: Optional[WaveScaling]


@dataclass(frozen=True)
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    scale: float
    size: int                              # positions of a chunk, or of the window
    softcap: Optional[float] = None        # "attention"
    kv_from: Optional[int] = None          # "attention": the layer whose keys and values this one reads
    rot: Optional[Rotation] = None         # left one of a pair
    keep_first: int = 0                    # left one of a pair: the first tokens that every window keeps


@dataclass(frozen=True)
class GatedLinearSizes:
    heads: int
    dim: int
    vdim: int
    tau: float


@dataclass(frozen=True)
class ZoguzenMixer:
    kind: str                                    # "attention", "mingru" or "parallel"
    attention: Optional[AttentionSizes] = None   # the mixer itself, or the left one of a pair
    linear: Optional[GatedLinearSizes] = None    # the right one of a pair
    width: int = 0                               # "mingru"


@dataclass(frozen=True)
class ZoguzenMLP:
    ff: int
    experts: int
    top: int


@dataclass(frozen=True)
class ZoguzenLayer:
    mixer: ZoguzenMixer
    mlp: Optional[ZoguzenMLP]


@dataclass(frozen=True)
class ZoguzenConfig:
    width: int
    vocab: int
    eps: float
    logit_softcap: Optional[float]
    side_dim: int
    layers: Tuple[ZoguzenLayer, ...]
    max_position: int

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @staticmethod
    def from_dict(cfg: Dict[str, Any]) -> "ZoguzenConfig":
        width = _positive(cfg, "width", "")
        vocab = _positive(cfg, "vocab", "")
        eps = _positive_number(_need(cfg, "norm", dict, ""), "eps", "norm.")
        softcap = None if cfg.get("logit_softcap") is None else _positive_number(cfg, "logit_softcap", "")
        side = _positive(_need(cfg, "token_side", dict, ""), "dim", "token_side.")
        raw_layers = _need(cfg, "layers", list, "")
        if not raw_layers:
            raise ConfigError("layers must list at least one layer")
        layers = []
        for i, raw in enumerate(raw_layers):
            layer = _layer(raw, f"layers[{i}].")
            a = layer.mixer.attention
            if a is not None and a.kv_from is not None:
                _check_source(layers, a, i)
            layers.append(layer)
        max_position = cfg.get("max_position", DEFAULT_MAX_POSITION)
        if isinstance(max_position, bool) or not isinstance(max_position, int) or max_position <= 0:
            raise ConfigError(f"max_position must be a positive integer, is {max_position!r}")
        return ZoguzenConfig(width, vocab, eps, softcap, side, tuple(layers), max_position)


def _positive_number(d, key, where) -> float:
    v = _need(d, key, float, where)
    if not v > 0.0:
        raise ConfigError(f"{where}{key} must be positive, is {v}")
    return v


def _check_source(before, a: AttentionSizes, i: int) -> None:
    """A layer may read the keys and values of an earlier attention layer that has some, in the shape they lie in."""
    where = f"layers[{i}].mixer.kv_from"
    if not 0 <= a.kv_from < i:
        raise ConfigError(f"{where} {a.kv_from} names no layer before this one")
    source = before[a.kv_from].mixer
    if source.kind != "attention" or source.attention.kv_from is not None:
        raise ConfigError(f"{where} {a.kv_from} names a layer without keys and values of its own")
    s = source.attention
    if (s.kv_heads, s.dim, s.vdim) != (a.kv_heads, a.dim, a.vdim):
        raise ConfigError(f"{where} {a.kv_from}: that layer holds {s.kv_heads} heads of {s.dim} and {s.vdim}, this one reads "
                          f"{a.kv_heads} of {a.dim} and {a.vdim}")


def _rotation(m, where: str, dim: int) -> Optional[Rotation]:
    rot = m.get("rot")
    if rot is None:
        return None
    rw = where + "rot."
    dims, base = _need(rot, "dims", int, rw), _need(rot, "base", float, rw)
    if dims < 0 or dims % 2 != 0 or dims > dim:
        raise ConfigError(f"{rw}dims must be even and at most dim {dim}, is {dims}")
    if dims == 0:
        return None
    if not base > 0.0:
        raise ConfigError(f"{rw}base must be positive, is {base}")
    scaling = None
    if rot.get("scaling") is not None:
        sc, sw = rot["scaling"], rw + "scaling."
        scaling = WaveScaling(*(_positive_number(sc, key, sw) for key in ("factor", "low", "high", "original")))
        if not scaling.high > scaling.low:
            raise ConfigError(f"{sw}high {scaling.high} must be above low {scaling.low}")
    return Rotation(dims, base, scaling)


def _attention(m, where: str, left: bool) -> AttentionSizes:
    heads, kv_heads = _positive(m, "heads", where), _positive(m, "kv_heads", where)
    if heads % kv_heads != 0:
        raise ConfigError(f"{where}heads {heads} is not a multiple of kv_heads {kv_heads}")
    dim, vdim = _positive(m, "dim", where), _positive(m, "vdim", where)
    taps = _positive(m, "conv", where)
    if taps > 16:
        raise ConfigError(f"{where}conv: {taps} taps are more than 16")
    mask = _need(m, "mask", dict, where)
    size = _positive(mask, "size", where + "mask.")
    extra = {}
    if left:
        keep = _need(mask, "keep_first", int, where + "mask.")
        if keep < 0:
            raise ConfigError(f"{where}mask.keep_first must not be negative, is {keep}")
        extra.update(keep_first=keep, rot=_rotation(m, where, dim))
    else:
        if m.get("softcap") is not None:
            extra.update(softcap=_positive_number(m, "softcap", where))
        if m.get("kv_from") is not None:
            extra.update(kv_from=_need(m, "kv_from", int, where))
    return AttentionSizes(heads, kv_heads, dim, vdim, taps, _need(m, "scale", float, where), size, **extra)


def _layer(raw, where: str) -> ZoguzenLayer:
    kind = _need(raw, "type", str, where)
    m, mw = _need(raw, "mixer", dict, where), where + "mixer."
    if kind == "attention":
        mixer = ZoguzenMixer(kind, _attention(m, mw, False))
    elif kind == "mingru":
        mixer = ZoguzenMixer(kind, width=_positive(m, "width", mw))
    elif kind == "parallel":
        right, rw = _need(m, "right", dict, mw), mw + "right."
        linear = GatedLinearSizes(_positive(right, "heads", rw), _positive(right, "dim", rw), _positive(right, "vdim", rw),
                                  _positive_number(right, "tau", rw))
        mixer = ZoguzenMixer(kind, _attention(_need(m, "left", dict, mw), mw + "left.", True), linear)
    else:
        raise ConfigError(f"{where}type {kind!r} is no mixer of this design (known: 'attention', 'mingru', 'parallel')")
    raw_mlp = raw.get("mlp")
    mlp = None
    if raw_mlp is not None:
        pw = where + "mlp."
        mlp_kind = _need(raw_mlp, "kind", str, pw)
        if mlp_kind != "moe":
            raise ConfigError(f"{pw}kind {mlp_kind!r} is no feed-forward of this design (known: 'moe')")
        router, rw = _need(raw_mlp, "router", dict, pw), pw + "router."
        experts, top = _positive(router, "experts", rw), _positive(router, "top", rw)
        if top > experts:
            raise ConfigError(f"{rw}top {top} is more than the {experts} experts")
        mlp = ZoguzenMLP(_positive(_need(raw_mlp, "expert", dict, pw), "ff", pw + "expert."), experts, top)
    return ZoguzenLayer(mixer, mlp)
