"""A plain, slow statement of the Zabutar design in numpy, one function per mechanism, written from its
equations and sharing nothing with the package.  Weights are a dict of arrays under the names a
checkpoint uses ([out, in] matrices); `cfg` is the parsed config.json.  Everything is computed in
`dtype` (float64 unless said otherwise), every position of a sequence at once, keys in full: no cache."""
import math

import numpy as np


def rms(x, eps):
    return np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def rms_norm_zero_centred(x, w, eps):
    """The stored weight is the distance from 1."""
    return x / rms(x, eps) * (1 + w)


def causal_conv(h, w):
    """h [T, width], w [width, taps]: tap taps - 1 meets the row itself, the ones before it earlier rows."""
    taps = w.shape[1]
    out = np.zeros_like(h)
    for j in range(taps):
        back = taps - 1 - j
        out[back:] += w[:, j] * h[:len(h) - back]
    return out


def sigmoid(z):
    return np.where(z >= 0, 1 / (1 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(z, 0)


def xielu(z, p, q):
    neg = np.minimum(z, 0)
    return np.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (np.exp(neg) - 1 - neg)) + z / 2


def forget_gate(z, lower):
    return lower + (1 - lower) * sigmoid(z)


def gated_state(q, f, v):
    """q, f [T, dim], v [T, vdim] of one head: S <- diag(f) S + (1 - f) v^T, row t of the result S^T q."""
    S = np.zeros((q.shape[1], v.shape[1]), q.dtype)
    out = np.zeros_like(v)
    for t in range(len(q)):
        S = f[t][:, None] * S + (1 - f[t])[:, None] * v[t][None, :]
        out[t] = S.T @ q[t]
    return out


def hgrn2(h, g, m, eps):
    T, H, dim, vdim = len(h), m["heads"], m["dim"], m["vdim"]
    q = silu(h @ g("q").T).reshape(T, H, dim)
    f = forget_gate(h @ g("f").T + g("f.b"), g("lower")).reshape(T, H, dim)
    v = (h @ g("v").T).reshape(T, H, vdim)
    heads = []
    for n in range(H):
        o = gated_state(q[:, n], f[:, n], v[:, n])
        heads.append(o / rms(o, eps) * g("norm"))
    return np.concatenate(heads, -1) @ g("o").T


def distance_bucket(n, rows, far):
    """Exact up to rows / 2 - 1, then logarithmic up to `far`, where the last bucket begins at the latest."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (rows - half)))


def visible(T):
    return np.tril(np.ones((T, T), bool))


def softmax(s, mask):
    e = np.where(mask, np.exp(np.where(mask, s, -np.inf) - np.where(mask, s, -np.inf).max(-1, keepdims=True)), 0)
    return e / e.sum(-1, keepdims=True)


def attention(h, g, m, kv):
    """kv: the layer's own keys and values, or those of the layer it borrows from."""
    T, H, G, dim = len(h), m["heads"], m["kv_heads"], m["dim"]
    q = (h @ g("q").T).reshape(T, H, dim)
    k, v = kv
    rel = g("rel")
    lag = np.maximum(np.arange(T)[:, None] - np.arange(T)[None, :], 0)
    bucket = np.array([distance_bucket(n, len(rel), m["bias_max"]) for n in range(T)])
    heads = []
    for n in range(H):
        s = q[:, n] @ k[:, n // (H // G)].T * m["scale"] + rel[bucket[lag], n]
        heads.append(softmax(s, visible(T)) @ v[:, n // (H // G)])
    return np.concatenate(heads, -1) @ g("o").T


def keys_values(h, g, m):
    T, G = len(h), m["kv_heads"]
    return (h @ g("k").T).reshape(T, G, m["dim"]), (h @ g("v").T).reshape(T, G, m["vdim"])


def dense(h, g):
    p, q = g("act")
    return xielu(h @ g("up").T + g("up.b"), p, q) @ g("down").T + g("down.b")


def expert(h, g):
    return (silu(h @ g("gate").T) * (h @ g("up").T)) @ g("down").T


def choose(s, correction, top, groups, keep):
    """Indices of the chosen ones for one token: the best by s + correction within the best groups."""
    c = s + correction
    best = c.reshape(groups, -1).max(-1)
    kept = np.argsort(-best, kind="stable")[:keep]
    allowed = np.isin(np.arange(len(c)) // (len(c) // groups), kept)
    return np.argsort(-np.where(allowed, c, -np.inf), kind="stable")[:top]


def mixture(h, g, m):
    r = m["router"]
    E = r["experts"]
    z = h @ g("router").T
    s = np.exp(z - z.max(-1, keepdims=True))
    s = s / s.sum(-1, keepdims=True)
    out = np.zeros_like(h)
    for t in range(len(h)):
        chosen = choose(s[t], g("correction"), r["top"], r["groups"]["count"], r["groups"]["keep"])
        weight = s[t][chosen] / (s[t][chosen].sum() + 1e-20) * r["scale"]
        for e, w in zip(chosen, weight):
            out[t] += w * (expert(h[t], lambda n: g(f"e{e}.{n}")) if e < E else h[t])
    if m.get("shared"):
        out += expert(h, lambda n: g("shared." + n))
    return out


def layer(cfg, weights, i, x, kept, dtype=np.float64):
    """The residual after layer i; kept: layer -> its keys and values, filled in by layers that have them."""
    def t(name):
        return np.asarray(weights[f"l{i}." + name]).astype(dtype)

    lc, eps = cfg["layers"][i], dtype(cfg["norm"]["eps"])
    h = rms_norm_zero_centred(x, t("norm1"), eps)
    h = h + causal_conv(h, t("canon1"))
    g = lambda n: t("mix." + n)
    m = lc["mixer"]
    if lc["type"] == "hgrn2":
        y = hgrn2(h, g, m, eps)
    else:
        if m.get("kv_from") is None:
            kept[i] = keys_values(h, g, m)
        y = attention(h, g, m, kept[i if m.get("kv_from") is None else m["kv_from"]])
    x = x + rms_norm_zero_centred(y, t("norm1b"), eps)
    if lc["mlp"] is None:
        return x
    h = rms_norm_zero_centred(x, t("norm2"), eps)
    h = h + causal_conv(h, t("canon2"))
    g = lambda n: t("mlp." + n)
    y = dense(h, g) if lc["mlp"]["kind"] == "dense" else mixture(h, g, lc["mlp"])
    return x + rms_norm_zero_centred(y, t("norm2b"), eps)


def forward(cfg, weights, tokens, dtype=np.float64):
    """(logits [T, vocab], residual after every layer [layers, T, width])."""
    def t(name):
        return np.asarray(weights[name]).astype(dtype)

    x = t("embed")[np.asarray(tokens)] + t("pos")[:len(tokens)]
    after, kept = [], {}
    for i in range(len(cfg["layers"])):
        x = layer(cfg, weights, i, x, kept, dtype)
        after.append(x)
    return rms_norm_zero_centred(x, t("final.norm"), dtype(cfg["norm"]["eps"])) @ t("head").T, np.stack(after)
