"""A plain, slow float64 restatement of the Nubedra design: one function per mechanism, whole sequences only, no cache.

It shares no code with the product path.  `cfg` is the parsed config.json, `w` a dict of float arrays by tensor name.
Linear weights are [out, in]; a sequence of activations is [tokens, width].
"""
import numpy as np


def rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def centred_norm(x, w, eps):
    """The layers' norms: a stored weight of 0 leaves the scale at 1."""
    return rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


# ---------------------------------------------------------------- gated linear attention
def key_decay(z, tau):
    """sigmoid(z) to the power 1 / tau."""
    return np.exp(-np.logaddexp(0.0, -z) / tau)


def gated_recurrence(q, k, v, a):
    """q, k, a [n, heads, d], v [n, heads, dv] -> o [n, heads, dv], the last state [heads, d, dv]"""
    n, heads, d = q.shape
    S = np.zeros((heads, d, v.shape[2]))
    o = np.zeros(v.shape)
    for t in range(n):
        for h in range(heads):
            S[h] = a[t, h][:, None] * S[h] + np.outer(k[t, h], v[t, h])
            o[t, h] = S[h].T @ q[t, h]
    return o, S


def gated_norm(o, weight, z, eps):
    """o [n, heads, dv]: a norm per head with one weight for all of them, then the gate."""
    return (rms(o, eps) * weight).reshape(z.shape) * silu(z)


def gla_mixer(h, mx, w, pre, eps):
    n, H, d, dv = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ w[pre + "q"].T).reshape(n, H, d) * d ** -0.5
    k = (h @ w[pre + "k"].T).reshape(n, H, d)
    v = (h @ w[pre + "v"].T).reshape(n, H, dv)
    z = (h @ w[pre + "a1"].T) @ w[pre + "a2"].T + w[pre + "a2.b"]
    o, _ = gated_recurrence(q, k, v, key_decay(z, mx["tau"]).reshape(n, H, d))
    return gated_norm(o, w[pre + "norm"], h @ w[pre + "g"].T, eps) @ w[pre + "o"].T


# ---------------------------------------------------------------- latent attention
def rotation(rot):
    """(frequency of every pair, factor of cos and sin)"""
    dims, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    i = np.arange(dims // 2)
    f = base ** (-2.0 * i / dims)
    if not sc:
        return f, 1.0

    def at(turns):   # the dimension that turns so often over the original length
        return dims * np.log(sc["original"] / (2 * np.pi * turns)) / (2 * np.log(base))
    lo, hi = max(np.floor(at(sc["fast"])), 0), min(np.ceil(at(sc["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0, 1)
    return f / sc["factor"] * ramp + f * (1 - ramp), 0.1 * np.log(sc["factor"]) + 1.0


def rotate(x, pos, rot):
    """x [n, ..., dims or more] at positions `pos`: neighbouring dimensions turn together."""
    f, m = rotation(rot)
    a = np.asarray(pos, np.float64)[:, None] * f
    a = a.reshape((x.shape[0],) + (1,) * (x.ndim - 2) + (-1,))
    c, s, dims = m * np.cos(a), m * np.sin(a), rot["dims"]
    u, v, y = x[..., 0:dims:2], x[..., 1:dims:2], x.copy()
    y[..., 0:dims:2] = u * c - v * s
    y[..., 1:dims:2] = v * c + u * s
    return y


def visible(n, m, size):
    """[query, key], the queries at the last n of m positions: the key lies at most size - 1 tokens back (size None: anywhere
    before)."""
    d = np.arange(m - n, m)[:, None] - np.arange(m)[None, :]
    return (d >= 0) & (d < (size if size else m))


def sink_softmax(s, sink):
    """Weights over the last axis with e^sink added to the denominator; -inf marks what is not seen."""
    m = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - m)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - m))


def output_gate(z):
    return sigmoid(z)


def latent_kv(h, mx, w, pre, eps):
    """What a latent layer keeps of every token: the normed latent and the rotated key part."""
    y = h @ w[pre + "dkv"].T
    c = rms(y[:, :mx["kv_rank"]], eps) * w[pre + "dkv.norm"]
    return c, rotate(y[:, mx["kv_rank"]:], np.arange(h.shape[0]), mx["rot"])


def latent_attend(q, c, kr, uk, uv, scale, size, sink):
    """q [n, H, d + r] with its last r dimensions rotated, c [m, rank], kr [m, r], uk [H * d, rank], uv [H * dv, rank],
    sink [H]; the queries are the last n of the m positions.  -> [n, H, dv]"""
    n, H, _ = q.shape
    m, r = kr.shape
    d = q.shape[2] - r
    k = (c @ uk.T).reshape(m, H, d)
    v = (c @ uv.T).reshape(m, H, -1)
    seen = visible(n, m, size)
    out = np.zeros((n, H, v.shape[2]))
    for i in range(H):
        s = (q[:, i, :d] @ k[:, i].T + q[:, i, d:] @ kr.T) * scale
        out[:, i] = sink_softmax(np.where(seen, s, -np.inf), sink[i]) @ v[:, i]
    return out


def latent_mixer(h, kv, mx, w, pre, eps):
    n, H, d, r = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"]
    c, kr = kv
    cq = rms(h @ w[pre + "dq"].T, eps) * w[pre + "dq.norm"]
    q = (cq @ w[pre + "uq"].T).reshape(n, H, d + r)
    q = np.concatenate([q[..., :d], rotate(q[..., d:], np.arange(n), mx["rot"])], axis=-1)
    out = latent_attend(q, c, kr, w[pre + "uk"], w[pre + "uv"], mx["scale"], (mx.get("mask") or {}).get("size"), w[pre + "sink"])
    out = out * output_gate(h @ w[pre + "g"].T)[:, :, None]
    return out.reshape(n, -1) @ w[pre + "o"].T


# ---------------------------------------------------------------- the rest
def relu(z):
    return np.maximum(z, 0.0)


def feed_forward(h, w, pre):
    return (relu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def forward(tokens, cfg, w, layers_out=None):
    """-> logits [tokens, vocab]; appends the residual stream after every layer to `layers_out`."""
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][np.asarray(tokens, np.int64)] * cfg["embedding"]["scale"]
    kept = {}
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        h = centred_norm(x, w[p + "norm1"], eps)
        if L["type"] == "gla":
            y = gla_mixer(h, mx, w, p + "mix.", eps)
        else:
            j = mx.get("kv_from")
            if j is None:
                kept[i] = latent_kv(h, mx, w, p + "mix.", eps)
            y = latent_mixer(h, kept[i if j is None else j], mx, w, p + "mix.", eps)
        x = x + mult * centred_norm(y, w[p + "norm1b"], eps)
        if L.get("mlp"):
            y = feed_forward(centred_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
            x = x + mult * centred_norm(y, w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return centred_norm(x, w["final.norm"], eps) @ w["embed"].T
