"""A plain, slow statement of the Tutilorn design in numpy, one function per mechanism, written from
its equations and sharing nothing with the package.  Weights are a dict of arrays under the names
a checkpoint uses ([out, in] matrices); `cfg` is the parsed config.json.  Everything is computed in
`dtype` (float64 unless said otherwise), every position of a sequence at once, keys in full: no cache."""
import numpy as np


def dynamic_tanh(x, w, b, alpha):
    return np.tanh(alpha * x) * w + b


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def rope_interleaved(x, positions, base, dims):
    """x [T, n]: pairs (2i, 2i + 1) of the first `dims` columns turn by position * base^(-2i / dims)."""
    out = x.copy()
    for i in range(dims // 2):
        a = (np.asarray(positions, np.float64) * float(base) ** (-2.0 * i / dims)).astype(x.dtype)
        c, s = np.cos(a), np.sin(a)
        u, v = x[:, 2 * i], x[:, 2 * i + 1]
        out[:, 2 * i], out[:, 2 * i + 1] = u * c - v * s, v * c + u * s
    return out


def window_mask(T, size):
    """[query, key], True for lags 0 .. size - 1 of the key behind the query (size None: any lag)."""
    d = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (d >= 0) & ((d < size) if size else True)


def softmax_with_sink(scores, mask, sink):
    """Rows of `scores`; the denominator holds exp(sink) once more than the visible keys' exponentials."""
    top = np.maximum(np.where(mask, scores, -np.inf).max(-1, keepdims=True), sink)
    e = np.where(mask, np.exp(np.where(mask, scores, top) - top), 0)
    return e / (e.sum(-1, keepdims=True) + np.exp(sink - top))


def sigmoid(z):
    return 1 / (1 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def latent_attention(h, g, m, eps):
    """h [T, width]; g(name) gives a tensor of the mixer, m its sizes."""
    T, H, dim, rd, vd, r = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    pos = np.arange(T)
    q = (rms_norm(h @ g("dq").T, g("dq.norm"), eps) @ g("uq").T).reshape(T, H, dim + rd)
    down = h @ g("dkv").T
    c = rms_norm(down[:, :r], g("dkv.norm"), eps)
    k_rot = rope_interleaved(down[:, r:], pos, base, dims)
    k = (c @ g("uk").T).reshape(T, H, dim)
    v = (c @ g("uv").T).reshape(T, H, vd)
    gate = sigmoid(h @ g("g").T)
    mask = window_mask(T, m["mask"]["size"] if m.get("mask") else None)
    heads = []
    for n in range(H):
        scores = (q[:, n, :dim] @ k[:, n].T + rope_interleaved(q[:, n, dim:], pos, base, dims) @ k_rot.T) * m["scale"]
        heads.append(softmax_with_sink(scores, mask, g("sink")[n]) @ v[:, n] * gate[:, n:n + 1])
    return np.concatenate(heads, -1) @ g("o").T


def swiglu(h, g):
    return (silu(h @ g("gate").T) * (h @ g("up").T)) @ g("down").T


def owner(cfg, i):
    """The layer whose tensors layer i uses."""
    while "weights_of" in cfg["layers"][i]:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(cfg, weights, tokens, dtype=np.float64):
    """(logits [T, vocab], residual after every layer [layers, T, width])."""
    def t(name):
        return np.asarray(weights[name]).astype(dtype)

    eps = dtype(cfg["norm"]["eps"])

    def norm(x, name):
        return dynamic_tanh(x, t(name), t(name + ".b"), t(name + ".alpha").reshape(()))

    x = t("embed")[np.asarray(tokens)] * dtype(cfg["embedding"]["scale"])
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{owner(cfg, i)}."
        assert layer["type"] == "latent_attention"
        x = x + latent_attention(norm(x, p + "norm1"), lambda n: t(p + "mix." + n), layer["mixer"], eps)
        if layer["mlp"] is not None:
            x = x + swiglu(norm(x, p + "norm2"), lambda n: t(p + "mlp." + n))
        after.append(x)
    return norm(x, "final.norm") @ t("head").T, np.stack(after)
