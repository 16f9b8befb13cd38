"""Small Zabutar models with random weights, written as checkpoint folders, and the same weights for the oracle."""
import contextlib

import numpy as np

import tutilorn_model
import zabutar_oracle as zo

write = tutilorn_model.write  # config.json and model.safetensors (bfloat16)


def hgrn2(heads=3, dim=20, vdim=28):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}}


def attention(heads=6, kv_heads=2, dim=20, vdim=12, bias_max=70, scale=None, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "bias_max": bias_max,
         "scale": scale if scale is not None else float(1.3 / np.sqrt(dim))}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def dense(ff=52):
    return {"kind": "dense", "ff": ff}


def moe(ff=28, experts=9, identity=3, top=3, groups=4, keep=2, scale=1.25, shared=36):
    m = {"kind": "moe", "expert": {"ff": ff},
         "router": {"experts": experts, "identity": identity, "top": top, "scale": scale,
                    "groups": {"count": groups, "keep": keep}}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def layer(mixer, mlp=None):
    return dict(mixer, mlp=mlp)


def config(layers, vocab=90, width=60, eps=1e-5, taps=4, max_positions=1400):
    return {"architecture": "Zabutar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "canon": {"taps": taps},
            "max_positions": max_positions, "layers": layers}


def exact(a):
    """The values cut to what a bfloat16 holds."""
    bits = np.ascontiguousarray(a, np.float32).reshape(-1).view(np.uint32) & np.uint32(0xFFFF0000)
    return bits.view(np.float32).reshape(np.shape(a))


def make_weights(cfg, seed, gain=1.0, rel_rows=18):
    """name -> float32 array whose values a bfloat16 holds exactly."""
    r = np.random.default_rng(seed)
    w = {}

    def put(name, a):
        w[name] = exact(a)

    def linear(name, out, inp, g=1.0):
        put(name, g * r.standard_normal((out, inp)) / np.sqrt(inp))

    def norm(name, n):
        put(name, 0.3 * r.standard_normal(n))

    def expert(name, ff):
        linear(name + "gate", ff, d, 1.5)
        linear(name + "up", ff, d)
        linear(name + "down", d, ff)

    d, taps = cfg["width"], cfg["canon"]["taps"]
    put("embed", r.standard_normal((cfg["vocab"], d)))
    put("pos", 0.5 * r.standard_normal((cfg["max_positions"], d)))
    for i, lc in enumerate(cfg["layers"]):
        m, p = lc["mixer"], f"l{i}."
        norm(p + "norm1", d)
        norm(p + "norm1b", d)
        put(p + "canon1", 0.4 * r.standard_normal((d, taps)))
        if lc["type"] == "hgrn2":
            hd, hv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            linear(p + "mix.q", hd, d)
            linear(p + "mix.f", hd, d)
            put(p + "mix.f.b", 1 + 2 * r.standard_normal(hd))
            put(p + "mix.lower", r.uniform(0, 0.9, hd))
            linear(p + "mix.v", hv, d)
            put(p + "mix.norm", 1 + 0.3 * r.standard_normal(m["vdim"]))
            linear(p + "mix.o", d, hv)
        else:
            linear(p + "mix.q", m["heads"] * m["dim"], d, gain)
            if m.get("kv_from") is None:
                linear(p + "mix.k", m["kv_heads"] * m["dim"], d)
                linear(p + "mix.v", m["kv_heads"] * m["vdim"], d)
            put(p + "mix.rel", 1.5 * r.standard_normal((rel_rows, m["heads"])))
            linear(p + "mix.o", d, m["heads"] * m["vdim"])
        ff = lc["mlp"]
        if not ff:
            continue
        norm(p + "norm2", d)
        norm(p + "norm2b", d)
        put(p + "canon2", 0.4 * r.standard_normal((d, taps)))
        if ff["kind"] == "dense":
            linear(p + "mlp.up", ff["ff"], d)
            put(p + "mlp.up.b", 0.3 * r.standard_normal(ff["ff"]))
            linear(p + "mlp.down", d, ff["ff"])
            put(p + "mlp.down.b", 0.3 * r.standard_normal(d))
            put(p + "mlp.act", r.uniform(-1, 1, 2))
        else:
            n = ff["router"]["experts"] + ff["router"].get("identity", 0)
            linear(p + "mlp.router", n, d, 2.0)
            put(p + "mlp.correction", 0.3 * r.standard_normal(n))
            for e in range(ff["router"]["experts"]):
                expert(p + f"mlp.e{e}.", ff["expert"]["ff"])
            if ff.get("shared"):
                expert(p + "mlp.shared.", ff["shared"]["ff"])
    norm("final.norm", d)
    linear("head", cfg["vocab"], d, 2.0)
    return w


@contextlib.contextmanager
def watch_choices():
    """A list that receives, for every choice the oracle makes meanwhile, by how much it was not another one."""
    gaps, plain = [], zo.choose

    def choose(s, correction, top, groups, keep):
        chosen = plain(s, correction, top, groups, keep)
        c = s + correction
        best = np.sort(c.reshape(groups, -1).max(-1))[::-1]
        gap = best[keep - 1] - best[keep] if keep < groups else np.inf
        kept = np.argsort(-c.reshape(groups, -1).max(-1), kind="stable")[:keep]
        rest = np.sort([c[i] for i in range(len(c)) if i // (len(c) // groups) in kept])[::-1]
        if top < len(rest):
            gap = min(gap, rest[top - 1] - rest[top])
        gaps.append(gap)
        return chosen

    zo.choose = choose
    try:
        yield gaps
    finally:
        zo.choose = plain
