"""A plain, slow implementation of the Zoguzen design in float64 numpy, one function per mechanism.

It shares no code with the product: whole sequences at once, no cache, no pages, no state slots.  Weights are a
dictionary name -> float64 array with the checkpoint's names; the configuration is the config.json dictionary.
`forward(cfg, w, tokens)` returns the logits at every position, `layer_outputs` the stream after every layer.
"""
import numpy as np


# ---- small functions ------------------------------------------------------------------------------------------------
def layer_norm(x, weight, eps):
    """Mean taken off, divided by the root of the mean squared deviation plus eps, times a weight; no bias."""
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * weight


def rms_norm(x, weight, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * weight


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def capped(s, cap):
    return cap * np.tanh(s / cap)


def token_shift(h, amount):
    """Every token's h moves towards the token's before it, lane by lane; the first token's neighbour is zero."""
    before = np.concatenate([np.zeros_like(h[:1]), h[:-1]], axis=0)
    return h + (before - h) * amount


def causal_conv(u, taps):
    """u [T, channels], taps [channels, n]: y_t = sum_j taps[:, j] u_(t - n + 1 + j), zeros before the start."""
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, u.shape[1])), u], axis=0)
    return sum(padded[j:j + u.shape[0]] * taps[:, j] for j in range(n))


# ---- rotation -------------------------------------------------------------------------------------------------------
def frequencies(rot):
    """One frequency a pair of lanes: base^(-2i / dims), long waves divided by a factor, a blend between."""
    dims = int(rot["dims"])
    f = float(rot["base"]) ** (-2.0 * np.arange(dims // 2) / dims)
    s = rot.get("scaling")
    if s is None:
        return f
    original, low, high, factor = float(s["original"]), float(s["low"]), float(s["high"]), float(s["factor"])
    out = []
    for fi in f:
        wave = 2.0 * np.pi / fi
        if wave < original / high:
            out.append(fi)
        elif wave > original / low:
            out.append(fi / factor)
        else:
            t = (original / wave - low) / (high - low)
            out.append((1.0 - t) * fi / factor + t * fi)
    return np.asarray(out)


def rotate(x, rot, positions):
    """x [T, heads, dim]: lanes 2i and 2i + 1 of the first rot.dims lanes turn by position * frequency i."""
    if rot is None or not rot.get("dims"):
        return x
    dims = int(rot["dims"])
    a = np.asarray(positions, dtype=np.float64)[:, None] * frequencies(rot)[None, :]
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    out = x.copy()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


# ---- who sees whom --------------------------------------------------------------------------------------------------
def sees_chunk(T, size):
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def sees_window_and_first(T, size, keep_first):
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


# ---- attention over given queries, keys and values ------------------------------------------------------------------
def sink_talking_attention(q, k, v, scale, softcap, sees, talk):
    """q [T, H, d], k [T, G, d], v [T, G, dv].  Capped scores, a softmax with one more term of score 0, then every head's
    weights become a mix of all heads' weights (talk [H, H]) before they meet the values."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    weights = np.zeros((H, T, T))
    for h in range(H):
        s = capped(q[:, h] @ k[:, h // per].T * scale, softcap)
        s = np.where(sees, s, -np.inf)
        top = np.maximum(s.max(axis=1, keepdims=True), 0.0)
        e = np.exp(s - top)
        weights[h] = e / (np.exp(-top) + e.sum(axis=1, keepdims=True))
    mixed = np.einsum("hg,gij->hij", talk, weights)
    return np.stack([mixed[h] @ v[:, h // per] for h in range(H)], axis=1)


def softmax_attention(q, k, v, scale, sees):
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = []
    for h in range(H):
        s = np.where(sees, q[:, h] @ k[:, h // per].T * scale, -np.inf)
        e = np.exp(s - s.max(axis=1, keepdims=True))
        out.append(e / e.sum(axis=1, keepdims=True) @ v[:, h // per])
    return np.stack(out, axis=1)


# ---- mixers ---------------------------------------------------------------------------------------------------------
def attention_keys(h, w, p, m, eps):
    """What a layer's cache holds: keys behind convolution and norm, values behind the convolution."""
    T, G = h.shape[0], m["kv_heads"]
    k = causal_conv(h @ w[p + "k"].T + w[p + "k.b"], w[p + "k.conv"]).reshape(T, G, m["dim"])
    v = causal_conv(h @ w[p + "v"].T + w[p + "v.b"], w[p + "v.conv"]).reshape(T, G, m["vdim"])
    return rms_norm(k, w[p + "k.norm"], eps), v


def attention_mixer(h, w, p, m, eps, k, v):
    T, H = h.shape[0], m["heads"]
    q = causal_conv(h @ w[p + "q"].T + w[p + "q.b"], w[p + "q.conv"]).reshape(T, H, m["dim"])
    q = rms_norm(q, w[p + "q.norm"], eps)
    o = sink_talking_attention(q, k, v, m["scale"], m["softcap"], sees_chunk(T, m["mask"]["size"]), w[p + "talk"])
    return o.reshape(T, -1) @ w[p + "o"].T


def window_mixer(h, w, p, m, positions):
    """The left one of a pair: convolved, rotated, a window beside kept first tokens, gated lane by lane."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = causal_conv(h @ w[p + "q"].T, w[p + "q.conv"]).reshape(T, H, m["dim"])
    k = causal_conv(h @ w[p + "k"].T, w[p + "k.conv"]).reshape(T, G, m["dim"])
    v = causal_conv(h @ w[p + "v"].T, w[p + "v.conv"]).reshape(T, G, m["vdim"])
    q, k = rotate(q, m.get("rot"), positions), rotate(k, m.get("rot"), positions)
    o = softmax_attention(q, k, v, m["scale"], sees_window_and_first(T, m["mask"]["size"], m["mask"]["keep_first"]))
    return (o.reshape(T, -1) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def gated_recurrence(q, k, v, alpha):
    """S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t from S = 0; q, k, alpha [T, H, d], v [T, H, dv]."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]))
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(axis=1)
    return out


def gated_linear_mixer(h, w, p, m, eps):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ w[p + "k"].T).reshape(T, H, d)
    v = (h @ w[p + "v"].T).reshape(T, H, dv)
    z = h @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "a2.b"]
    alpha = (sigmoid(z) ** (1.0 / m["tau"])).reshape(T, H, d)
    o = rms_norm(gated_recurrence(q, k, v, alpha), w[p + "norm"], eps).reshape(T, -1)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel_mixer(h, w, p, m, eps, positions):
    left = window_mixer(h, w, p + "left.", m["left"], positions)
    right = gated_linear_mixer(h, w, p + "right.", m["right"], eps)
    return 0.5 * (rms_norm(left, w[p + "left.out"], eps) + rms_norm(right, w[p + "right.out"], eps))


def min_recurrence(z, u):
    """S_t = (1 - z_t) S_(t-1) + z_t c_t lane by lane from S = 0, c = u + 1/2 from zero on and sigmoid(u) below."""
    c = np.where(u >= 0, u + 0.5, sigmoid(u))
    S = np.zeros(z.shape[1])
    out = np.zeros_like(z)
    for t in range(z.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * c[t]
        out[t] = S
    return out


def mingru_mixer(h, w, p):
    z = sigmoid(h @ w[p + "z"].T + w[p + "z.b"])
    u = h @ w[p + "x"].T + w[p + "x.b"]
    return (min_recurrence(z, u) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---- feed-forward ---------------------------------------------------------------------------------------------------
def route(h, w_router, top):
    """(chosen experts [T, top], weights [T, top]): the largest logits, a softmax over the chosen logits alone."""
    z = h @ w_router.T
    ids = np.argsort(-z, axis=1, kind="stable")[:, :top]
    picked = np.take_along_axis(z, ids, axis=1)
    e = np.exp(picked - picked.max(axis=1, keepdims=True))
    return ids, e / e.sum(axis=1, keepdims=True)


def expert(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def feed_forward(h, w, p, mlp):
    ids, weights = route(h, w[p + "router"], mlp["router"]["top"])
    out = np.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        rows, place = np.nonzero(ids == e)
        if rows.size:
            out[rows] += weights[rows, place][:, None] * expert(h[rows], w[f"{p}e{e}.gate"], w[f"{p}e{e}.up"], w[f"{p}e{e}.down"])
    return out


def side_input(x, e, gate, proj, norm, eps):
    """What a layer adds for the token itself: the stream gates the token's own row of a table."""
    return rms_norm((gelu_tanh(x @ gate.T) * e) @ proj.T, norm, eps)


# ---- the model ------------------------------------------------------------------------------------------------------
def layer_outputs(cfg, w, tokens):
    """The stream after every layer, [layers, T, width], and the logits [T, vocab]."""
    tokens = np.asarray(tokens)
    positions = np.arange(len(tokens))
    eps, sd = cfg["norm"]["eps"], cfg["token_side"]["dim"]
    x = w["embed"][tokens]
    held = {}
    after = []
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        mp = p + "mix."
        h = token_shift(layer_norm(x, w[p + "norm1"], eps), w[p + "shift"])
        if spec["type"] == "attention":
            if m.get("kv_from") is None:
                held[i] = attention_keys(h, w, mp, m, eps)
            y = attention_mixer(h, w, mp, m, eps, *held[i if m.get("kv_from") is None else m["kv_from"]])
        elif spec["type"] == "mingru":
            y = mingru_mixer(h, w, mp)
        elif spec["type"] == "parallel":
            y = parallel_mixer(h, w, mp, m, eps, positions)
        else:
            raise ValueError(spec["type"])
        if spec.get("mlp") is not None:
            y = y + feed_forward(layer_norm(x, w[p + "norm2"], eps), w, p + "mlp.", spec["mlp"])
        x = x + y
        x = x + side_input(x, w["side.embed"][tokens, i * sd:(i + 1) * sd], w[p + "side.gate"], w[p + "side.proj"], w[p + "side.norm"], eps)
        after.append(x.copy())
    logits = capped(layer_norm(x, w["final.norm"], eps) @ w["embed"].T, cfg["logit_softcap"])
    return np.stack(after), logits


def forward(cfg, w, tokens):
    return layer_outputs(cfg, w, tokens)[1]
