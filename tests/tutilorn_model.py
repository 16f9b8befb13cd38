"""Small Tutilorn models with random weights, written as checkpoint folders, and the same weights for the oracle."""
import json
import os

import numpy as np


def mixer(heads=3, dim=24, rot_dim=8, vdim=20, kv_rank=36, q_rank=28, window=17, base=5000.0, scale=None, rot_dims=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
         "scale": scale if scale is not None else float(1.3 / np.sqrt(dim + rot_dim)),
         "rot": {"base": base, "dims": rot_dim if rot_dims is None else rot_dims}}
    if window:
        m["mask"] = {"size": window}
    return m


def layer(m, ff=52, weights_of=None):
    out = {"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}
    if weights_of is not None:
        out["weights_of"] = weights_of
    return out


def config(layers, vocab=90, width=60, eps=1e-5, scale=7.5):
    return {"architecture": "Tutilorn", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "layers": layers}


def make_weights(cfg, seed, gain=1.0):
    """name -> float32 array whose values a bfloat16 holds exactly."""
    r = np.random.default_rng(seed)
    w = {}

    def put(name, a):
        bits = np.ascontiguousarray(a, np.float32).reshape(-1).view(np.uint32) & np.uint32(0xFFFF0000)
        w[name] = bits.view(np.float32).reshape(np.shape(a))

    def linear(name, out, inp, g=1.0):
        put(name, g * r.standard_normal((out, inp)) / np.sqrt(inp))

    def norm(name, n, alpha):
        put(name, 1 + 0.3 * r.standard_normal(n))
        put(name + ".b", 0.2 * r.standard_normal(n))
        put(name + ".alpha", np.array(alpha))

    d = cfg["width"]
    put("embed", 0.1 * r.standard_normal((cfg["vocab"], d)))
    for i, lc in enumerate(cfg["layers"]):
        if "weights_of" in lc:
            continue
        m, p = lc["mixer"], f"l{i}."
        H = m["heads"]
        norm(p + "norm1", d, r.uniform(0.3, 1.1))
        linear(p + "mix.dq", m["q_rank"], d)
        put(p + "mix.dq.norm", 1 + 0.3 * r.standard_normal(m["q_rank"]))
        linear(p + "mix.uq", H * (m["dim"] + m["rot_dim"]), m["q_rank"], gain)
        linear(p + "mix.dkv", m["kv_rank"] + m["rot_dim"], d)
        put(p + "mix.dkv.norm", 1 + 0.3 * r.standard_normal(m["kv_rank"]))
        linear(p + "mix.uk", H * m["dim"], m["kv_rank"])
        linear(p + "mix.uv", H * m["vdim"], m["kv_rank"])
        put(p + "mix.sink", 1.5 * r.standard_normal(H))
        linear(p + "mix.g", H, d, 2.0)
        linear(p + "mix.o", d, H * m["vdim"])
        if lc["mlp"]:
            norm(p + "norm2", d, r.uniform(0.3, 1.1))
            linear(p + "mlp.gate", lc["mlp"]["ff"], d)
            linear(p + "mlp.up", lc["mlp"]["ff"], d)
            linear(p + "mlp.down", d, lc["mlp"]["ff"])
    norm("final.norm", d, 0.7)
    linear("head", cfg["vocab"], d, 2.0)
    return w


def write(folder, cfg, weights):
    """config.json and model.safetensors (bfloat16)."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at = {}, [], 0
    for name, a in weights.items():
        b = (np.ascontiguousarray(a).reshape(-1).view(np.uint32) >> 16).astype("<u2").tobytes()
        header[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    text = json.dumps(header).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(len(text).to_bytes(8, "little") + text + b"".join(blobs))
    return str(folder)
