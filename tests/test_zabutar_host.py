"""Zabutar without a GPU: the oracle's mechanisms against closed forms, mistakes planted in the oracle that the
GPU tests' tolerance must tell apart, and the reader of config.json."""
import json
import os

import numpy as np
import pytest

import shainet_amd
import zabutar_model as zm
import zabutar_oracle as zo


@pytest.fixture(scope="module")
def sa():
    if not os.path.exists(shainet_amd.library_path()):
        shainet_amd.build_library(force=False)
    return shainet_amd


# ---- the oracle itself

def test_convolution_is_causal():
    h = np.random.default_rng(0).standard_normal((9, 2))
    w = np.array([[1.0, 10.0, 100.0], [0.0, 0.0, 1.0]])
    c = zo.causal_conv(h, w)
    assert np.allclose(c[5, 0], h[3, 0] + 10 * h[4, 0] + 100 * h[5, 0]) and np.allclose(c[:, 1], h[:, 1])
    assert np.allclose(c[0, 0], 100 * h[0, 0]) and np.allclose(zo.causal_conv(h[:2], w), c[:2])


def test_gated_state_is_a_decayed_sum():
    r = np.random.default_rng(1)
    q, f, v = r.standard_normal((7, 3)), r.uniform(0, 1, (7, 3)), r.standard_normal((7, 4))
    o = zo.gated_state(q, f, v)
    for t in range(7):
        want = sum((q[t] * (1 - f[s]) * f[s + 1:t + 1].prod(0)).sum() * v[s] for s in range(t + 1))
        assert np.allclose(o[t], want)


def test_distance_buckets():
    b = [zo.distance_bucket(n, 12, 50) for n in range(400)]
    assert b[:7] == [0, 1, 2, 3, 4, 5, 6] and b[49] == 11 and b[50] == 11 and b[399] == 11
    assert all(0 <= y - x <= 1 for x, y in zip(b, b[1:]))
    edges = [next(n for n in range(6, 60) if b[n] >= k) for k in range(7, 12)]
    assert edges == [int(np.ceil(6 * (50 / 6) ** ((k - 6) / 6))) for k in range(7, 12)]


def test_xielu_and_softplus():
    p, q = 0.3, -0.7
    z = np.linspace(-4, 4, 33)
    y = zo.xielu(z, p, q)
    sp = np.log1p(np.exp([p, q]))
    assert np.allclose(y, np.where(z > 0, sp[0] * z * z + z / 2, (0.5 + sp[1]) * (np.expm1(z) - z) + z / 2))
    slope = np.diff(zo.xielu(np.array([-1e-6, 0, 1e-6]), p, q)) / 1e-6
    assert np.allclose(slope, 0.5, atol=1e-5)


def test_choice_within_groups():
    s = np.array([0.1, 0.3, 0.05, 0.25, 0.2, 0.1])
    none = np.zeros(6)
    assert sorted(zo.choose(s, none, 2, 3, 3)) == [1, 3]
    assert list(zo.choose(s, none, 3, 3, 2)) == [1, 3, 0]
    # a negative correction everywhere: what lies outside the kept groups stays outside
    assert set(zo.choose(s, none - 2, 4, 3, 2)) == {0, 1, 2, 3}
    assert list(zo.choose(s, np.array([0, 0, 0, 0, 0, 9.0]), 1, 3, 1)) == [5]


def test_identity_expert_gives_its_input():
    cfg = zm.config([zm.layer(zm.hgrn2(), zm.moe(experts=2, identity=2, top=1, groups=1, keep=1, scale=0.5, shared=0))])
    w = zm.make_weights(cfg, 0)
    w["l0.mlp.correction"] = np.array([0, 0, 0, 5.0], np.float32)
    h = np.random.default_rng(0).standard_normal((4, 60))
    assert np.allclose(zo.mixture(h, lambda n: w["l0.mlp." + n].astype(float), cfg["layers"][0]["mlp"]), 0.5 * h)


def mixed():
    return zm.config([zm.layer(zm.hgrn2(), zm.dense()), zm.layer(zm.attention(), zm.moe()), zm.layer(zm.attention(kv_from=1), None),
                      zm.layer(zm.hgrn2(heads=2), zm.moe(shared=0))], eps=0.05)


def wrong_gate(f):
    return lambda z, lower: f(z, 0 * lower)


PLANTED = {
    "norm weight not centred at zero": ("rms_norm_zero_centred", lambda f: lambda x, w, e: f(x, w - 1, e)),
    "eps outside the root": ("rms", lambda f: lambda x, e: np.sqrt((x * x).mean(-1, keepdims=True)) + e),
    "convolution without its input": ("causal_conv", lambda f: lambda h, w: f(h, w) - h),
    "convolution one row late": ("causal_conv", lambda f: lambda h, w: np.vstack([np.zeros_like(h[:1]), f(h, w)[:-1]])),
    "taps turned round": ("causal_conv", lambda f: lambda h, w: f(h, w[:, ::-1])),
    "no lower bound": ("forget_gate", wrong_gate),
    "gate not written": ("gated_state", lambda f: lambda q, g, v: f(q / np.maximum(1 - g, 1e-3), g, v)),
    "read before written": ("gated_state", lambda f: lambda q, g, v: np.vstack([0 * v[:1], f(np.roll(q, -1, 0), g, v)[:-1]])),
    "bucket edge one off": ("distance_bucket", lambda f: lambda n, b, m: f(n + 1, b, m)),
    "bucket edge moved": ("distance_bucket", lambda f: lambda n, b, m: f(n, b, m * 1.1)),
    "no linear half in xIELU": ("xielu", lambda f: lambda z, p, q: f(z, p, q) - z / 2),
    "xIELU without its half": ("xielu", lambda f: lambda z, p, q: f(z, p, np.log(np.expm1(np.maximum(zo.softplus(q) - 0.25, 0.01))))),
    "choice without groups": ("choose", lambda f: lambda s, c, top, g, k: f(s, c, top, 1, 1)),
    "choice without correction": ("choose", lambda f: lambda s, c, top, g, k: f(s, 0 * c, top, g, k)),
    "zeros outside the kept groups": ("choose", lambda f: lambda s, c, top, g, k: f(s, np.where(np.isin(np.arange(len(s)), f(s, c, k * len(s) // g, g, k)), c, -s), top, 1, 1)),
    "keys one further": ("visible", lambda f: lambda T: np.tril(np.ones((T, T), bool), 1)),
}


@pytest.mark.parametrize("name", sorted(PLANTED))
def test_a_planted_mistake_shows(monkeypatch, name):
    """What the GPU tests compare moves by far more than their tolerance (1e-4 of the largest logit)."""
    cfg = mixed()
    w = zm.make_weights(cfg, 1)
    for i in (1, 3):  # choice scores below zero
        w[f"l{i}.mlp.correction"] = w[f"l{i}.mlp.correction"] - 1
    ids = np.random.default_rng(0).integers(0, cfg["vocab"], 90)
    want = zo.forward(cfg, w, ids)[0]
    what, wrap = PLANTED[name]
    monkeypatch.setattr(zo, what, wrap(getattr(zo, what)))
    got = zo.forward(cfg, w, ids)[0]
    assert np.abs(got - want).max() / np.abs(want).max() > 1e-3


# ---- config.json

def bad(change):
    cfg = zm.config([zm.layer(zm.hgrn2(), zm.dense()), zm.layer(zm.attention(), zm.moe()), zm.layer(zm.attention(kv_from=1), None)])
    change(cfg)
    return cfg


def put(*path):
    *keys, last, value = path

    def change(c):
        for k in keys:
            c = c[k]
        c[last] = value
    return change


def drop(*path):
    *keys, last = path

    def change(c):
        for k in keys:
            c = c[k]
        del c[last]
    return change


@pytest.mark.parametrize("change,word", [
    (drop("vocab"), "lacks vocab"),
    (drop("max_positions"), "lacks max_positions"),
    (drop("norm", "eps"), "lacks norm.eps"),
    (drop("canon"), "lacks canon"),
    (put("canon", "taps", 0), "canon.taps"),
    (put("canon", "taps", 33), "canon.taps"),
    (put("layers", []), "lacks layers"),
    (put("layers", 0, "type", "latent_attention"), r"layers\[0\].type 'latent_attention'"),
    (drop("layers", 0, "mixer", "vdim"), r"lacks layers\[0\].mixer.vdim"),
    (drop("layers", 1, "mixer", "bias_max"), r"lacks layers\[1\].mixer.bias_max"),
    (drop("layers", 1, "mixer", "scale"), r"lacks layers\[1\].mixer.scale"),
    (put("layers", 2, "mixer", "kv_from", 0), "kv_from"),
    (put("layers", 2, "mixer", "kv_from", 2), "kv_from"),
    (put("layers", 2, "mixer", "kv_from", -1), "kv_from"),
    (put("layers", 2, "mixer", "dim", 24), "kv_from"),
    (put("layers", 0, "mlp", "kind", "gated"), "mlp.kind 'gated'"),
    (drop("layers", 0, "mlp", "ff"), r"mlp.ff"),
    (put("layers", 0, "mlp", "ff", 0), "must be positive"),
    (drop("layers", 1, "mlp", "expert"), "mlp.expert"),
    (drop("layers", 1, "mlp", "router", "top"), "router.top"),
    (put("layers", 1, "mlp", "router", "top", 7), "router"),
    (put("layers", 1, "mlp", "router", "groups", {"count": 5, "keep": 2}), "router"),
    (put("layers", 1, "mlp", "router", "groups", {"count": 4}), "router.groups.keep"),
    (put("layers", 1, "mlp", "shared", {}), "shared.ff"),
])
def test_config_errors_name_what_is_wrong(sa, tmp_path, change, word):
    (tmp_path / "config.json").write_text(json.dumps(bad(change)))
    with pytest.raises(sa.ArgumentError, match=word):
        sa.HFLoader.load_model(str(tmp_path))


def test_a_good_config_gets_as_far_as_the_device(sa, tmp_path):
    if sa.HIP.available():
        pytest.skip("a GPU is present")
    cfg = bad(drop("layers", 1, "mlp", "router", "groups"))  # optional parts left out
    del cfg["layers"][1]["mlp"]["shared"], cfg["layers"][1]["mlp"]["router"]["scale"]
    folder = zm.write(tmp_path, cfg, zm.make_weights(cfg, 0))
    with pytest.raises(sa.HipError, match="no gfx950 device"):
        sa.HFLoader.load_model(folder)
