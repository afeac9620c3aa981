"""A plain, slow float64 restatement of the Serisun design: one function per mechanism, whole sequences only, no cache.

It shares no code with the product path.  `cfg` is the parsed config.json, `w` a dict of float arrays by tensor name.
Linear weights are [out, in]; a sequence of activations is [tokens, width].
"""
import numpy as np


def rms(x, eps):
    """x divided by its root mean square over the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def query_temperature(n, coef, every):
    """[n]: what multiplies the query at positions 0 .. n-1."""
    p = np.arange(n)
    return 1.0 + coef * np.log(np.floor((p + 1) / every) + 1.0)


def head_slopes(n_head):
    return 2.0 ** (-8.0 * (np.arange(n_head) + 1) / n_head)


def sink_softmax(s):
    """Weights over the last axis with exp(0) added to the denominator; -inf marks what is not seen."""
    m = np.maximum(s.max(axis=-1, keepdims=True), 0.0)
    e = np.exp(s - m)
    return e / (np.exp(-m) + e.sum(axis=-1, keepdims=True))


def attend(q, k, v, scale, slopes, sink=True):
    """q [n, H, d], k [m, G, d], v [m, G, dv]; the queries are the last n of the m positions.  -> [n, H, dv]"""
    n, H, _ = q.shape
    m, G, _ = k.shape
    out = np.zeros((n, H, v.shape[2]))
    i = np.arange(m - n, m)[:, None]
    j = np.arange(m)[None, :]
    for h in range(H):
        g = h // (H // G)
        s = q[:, h] @ k[:, g].T * scale - slopes[h] * (i - j)
        s = np.where(j <= i, s, -np.inf)
        if sink:
            p = sink_softmax(s)
        else:
            p = np.exp(s - s.max(axis=-1, keepdims=True))
            p /= p.sum(axis=-1, keepdims=True)
        out[:, h] = p @ v[:, g]
    return out


def attention_mixer(h, mx, w, pre):
    n = h.shape[0]
    H, G = mx["heads"], mx["kv_heads"]
    q = (h @ w[pre + "q"].T).reshape(n, H, mx["dim"])
    k = (h @ w[pre + "k"].T).reshape(n, G, mx["dim"])
    v = (h @ w[pre + "v"].T).reshape(n, G, mx["vdim"])
    if mx.get("q_temp"):
        q = q * query_temperature(n, mx["q_temp"]["coef"], mx["q_temp"]["every"])[:, None, None]
    y = attend(q, k, v, mx["scale"], head_slopes(H))
    return y.reshape(n, -1) @ w[pre + "o"].T


def causal_conv_silu(x, taps, bias):
    """x [n, channels], taps [channels, K] with the last column on the current token; zeros before the start."""
    n, c = x.shape
    K = taps.shape[1]
    pad = np.concatenate([np.zeros((K - 1, c)), x])
    y = np.zeros((n, c))
    for t in range(K):
        y += pad[t:t + n] * taps[:, t]
    return silu(y + bias)


def state_space(x, B, C, dt, A_log, D):
    """x [n, heads, P], B, C [n, groups, N], dt [n, heads] (already positive).  -> y [n, heads, P], last state [heads, N, P]"""
    n, heads, P = x.shape
    groups, N = B.shape[1:]
    S = np.zeros((heads, N, P))
    y = np.zeros_like(x)
    a = np.exp(-np.exp(A_log) * dt)
    for t in range(n):
        for h in range(heads):
            g = h // (heads // groups)
            S[h] = a[t, h] * S[h] + dt[t, h] * np.outer(B[t, g], x[t, h])
            y[t, h] = S[h].T @ C[t, g] + D[h] * x[t, h]
    return y, S


def gated_group_norm(y, z, weight, groups, eps):
    """The gate first, then every one of `groups` equal parts by its own root mean square."""
    g = y * silu(z)
    n, d = g.shape
    return rms(g.reshape(n, groups, d // groups), eps).reshape(n, d) * weight


def mamba2_mixer(h, mx, w, pre, eps):
    n = h.shape[0]
    heads, P, N, G = mx["heads"], mx["vdim"], mx["state"], mx["groups"]
    inner = heads * P
    u = h @ w[pre + "in"].T
    z, xbc, dt = u[:, :inner], u[:, inner:2 * inner + 2 * G * N], u[:, 2 * inner + 2 * G * N:]
    xbc = causal_conv_silu(xbc, w[pre + "conv"], w[pre + "conv.b"])
    x = xbc[:, :inner].reshape(n, heads, P)
    B = xbc[:, inner:inner + G * N].reshape(n, G, N)
    C = xbc[:, inner + G * N:].reshape(n, G, N)
    y, _ = state_space(x, B, C, softplus(dt + w[pre + "dt_bias"]), w[pre + "A_log"], w[pre + "D"])
    y = gated_group_norm(y.reshape(n, inner), z, w[pre + "norm"], mx["norm_groups"], eps)
    return y @ w[pre + "o"].T


def feed_forward(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def layer(x, i, cfg, w):
    L, p, eps = cfg["layers"][i], f"l{i}.", cfg["norm"]["eps"]
    h = rms(x, eps) * w[p + "norm1"]
    if L["type"] == "attention":
        d = attention_mixer(h, L["mixer"], w, p + "mix.") * w[p + "ls1"]
    else:
        d = mamba2_mixer(h, L["mixer"], w, p + "mix.", eps) * w[p + "ls1"]
    if L.get("mlp"):
        d = d + feed_forward(h, w, p + "mlp.") * w[p + "ls2"]
    return x + d


def layer_runs(cfg):
    """The order layers run in: (layer, number of the pass when the layer opens one, else None)."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    runs = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


def forward(tokens, cfg, w, layers_out=None):
    """-> logits [tokens, vocab]; appends the residual stream after every layer run to `layers_out`."""
    emb = w["embed"][np.asarray(tokens, np.int64)]
    x = emb.copy()
    for i, opens in layer_runs(cfg):
        if opens is not None:
            if opens > 0:
                x = x + emb
            x = x + w["loop.step"][opens]
        x = layer(x, i, cfg, w)
        if layers_out is not None:
            layers_out.append(x.copy())
    return (rms(x, cfg["norm"]["eps"]) * w["final.norm"]) @ w["head"].T * cfg["logit_scale"]
