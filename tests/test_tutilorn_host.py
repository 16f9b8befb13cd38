"""Tutilorn without a GPU: the oracle's mechanisms against closed forms, mistakes planted in the oracle that
the GPU tests' tolerance must tell apart, the reader of config.json, and the trace replay's bookkeeping."""
import io
import json
import sys

import numpy as np
import pytest

import shainet_amd
import tutilorn_model as tm
import tutilorn_oracle as to


@pytest.fixture(scope="module")
def sa():
    import os

    if not os.path.exists(shainet_amd.library_path()):
        shainet_amd.build_library(force=False)
    return shainet_amd


# ---- the oracle itself

def test_rope_is_a_turn_of_neighbouring_pairs():
    r = np.random.default_rng(0)
    x = r.standard_normal((9, 14))
    pos = np.arange(3, 12)
    y = to.rope_interleaved(x, pos, 700.0, 10)
    z = (x[:, 0:10:2] + 1j * x[:, 1:10:2]) * np.exp(1j * pos[:, None] * 700.0 ** (-np.arange(0, 10, 2) / 10))
    assert np.allclose(y[:, 0:10:2], z.real) and np.allclose(y[:, 1:10:2], z.imag) and np.array_equal(y[:, 10:], x[:, 10:])


def test_sink_is_a_key_without_a_value():
    r = np.random.default_rng(1)
    s, mask = r.standard_normal((5, 5)), to.window_mask(5, 3)
    p = to.softmax_with_sink(s, mask, 0.7)
    e = np.exp(s) * mask
    assert np.allclose(p, e / (e.sum(-1, keepdims=True) + np.exp(0.7)))
    assert np.allclose(to.softmax_with_sink(s, mask, -1e9).sum(-1), 1)


def test_window_includes_its_own_row():
    m = to.window_mask(6, 2)
    assert m.sum() == 11 and m[4].tolist() == [False, False, False, True, True, False]
    assert np.array_equal(to.window_mask(6, None), np.tril(np.ones((6, 6), bool)))


def test_borrowed_weights():
    a = tm.layer(tm.mixer(), 20)
    cfg = tm.config([tm.layer(tm.mixer(), 20, weights_of=1), a, tm.layer(tm.mixer(), 20, weights_of=0)])
    assert [to.owner(cfg, i) for i in range(3)] == [1, 1, 1]
    w = tm.make_weights(cfg, 0)
    assert not any(n.startswith(("l0.", "l2.")) for n in w)
    own = dict(w)
    for n, v in w.items():
        if n.startswith("l1."):
            own["l0" + n[2:]] = own["l2" + n[2:]] = v
    ids = [3, 1, 4, 1, 5]
    assert np.array_equal(to.forward(cfg, w, ids)[0], to.forward(tm.config([a] * 3), own, ids)[0])


PLANTED = {
    "no sink": ("softmax_with_sink", lambda f: lambda s, m, k: f(s, m, -1e9)),
    "sink counted twice": ("softmax_with_sink", lambda f: lambda s, m, k: f(s, m, k + np.log(2.0))),
    "window one longer": ("window_mask", lambda f: lambda T, n: f(T, n + 1 if n else n)),
    "window one shorter": ("window_mask", lambda f: lambda T, n: f(T, n - 1 if n else n)),
    "other base": ("rope_interleaved", lambda f: lambda x, p, b, d: f(x, p, 2.0 * b, d)),
    "no gate": ("sigmoid", lambda f: lambda z: np.ones_like(z) if z.shape[-1] < 8 else f(z)),
    "norm without beta": ("dynamic_tanh", lambda f: lambda x, w, b, a: f(x, w, 0 * b, a)),
    "eps outside the root": ("rms_norm", lambda f: lambda x, w, e: x / (np.sqrt((x * x).mean(-1, keepdims=True)) + e) * w),
}


@pytest.mark.parametrize("name", sorted(PLANTED))
def test_a_planted_mistake_shows(monkeypatch, name):
    """What the GPU tests compare moves by far more than their tolerance (1e-4 of the largest logit)."""
    cfg = tm.config([tm.layer(tm.mixer(), 52), tm.layer(tm.mixer(), None)], eps=0.2)
    w = tm.make_weights(cfg, 1)
    ids = np.random.default_rng(0).integers(0, cfg["vocab"], 60)
    want = to.forward(cfg, w, ids)[0]
    what, wrap = PLANTED[name]
    monkeypatch.setattr(to, what, wrap(getattr(to, what)))
    got = to.forward(cfg, w, ids)[0]
    assert np.abs(got - want).max() / np.abs(want).max() > 5e-4


# ---- config.json

def bad(change):
    cfg = tm.config([tm.layer(tm.mixer(), 20), tm.layer(tm.mixer(), None)])
    change(cfg)
    return cfg


@pytest.mark.parametrize("change,word", [
    (lambda c: c.update(architecture="Nobody"), "Unsupported architecture: 'Nobody'"),
    (lambda c: c.pop("vocab"), "lacks vocab"),
    (lambda c: c["norm"].pop("eps"), "lacks norm.eps"),
    (lambda c: c.pop("embedding"), "lacks embedding"),
    (lambda c: c.update(layers=[]), "lacks layers"),
    (lambda c: c["layers"][1].update(type="convolution"), r"layers\[1\].type 'convolution'"),
    (lambda c: c["layers"][1]["mixer"].pop("kv_rank"), r"lacks layers\[1\].mixer.kv_rank"),
    (lambda c: c["layers"][0]["mixer"]["rot"].pop("base"), r"layers\[0\].mixer.rot.base"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "must be positive"),
    (lambda c: c["layers"][0]["mlp"].update(kind="mixture"), "dense"),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), "mlp.ff"),
    (lambda c: c["layers"][1].update(weights_of=0), "differs from the layer"),
    (lambda c: c["layers"][1].update(weights_of=1), "leads to no layer"),
    (lambda c: c["layers"][1].update(weights_of=7), "leads to no layer"),
])
def test_config_errors_name_what_is_wrong(sa, tmp_path, change, word):
    (tmp_path / "config.json").write_text(json.dumps(bad(change)))
    with pytest.raises(sa.ArgumentError, match=word):
        sa.HFLoader.load_model(str(tmp_path))


def test_a_good_config_gets_as_far_as_the_device(sa, tmp_path):
    if sa.HIP.available():
        pytest.skip("a GPU is present")
    cfg = tm.config([tm.layer(tm.mixer(), 20, weights_of=1), tm.layer(tm.mixer(), 20), tm.layer(tm.mixer(window=0), None)])
    folder = tm.write(tmp_path, cfg, tm.make_weights(cfg, 0))
    with pytest.raises(sa.HipError, match="no gfx950 device"):
        sa.HFLoader.load_model(folder)
    st = sa.SafeTensors(folder)
    assert st.info("l1.norm1.alpha")[:2] == ("BF16", []) and st.has_tensor("l2.mix.uk")
    with pytest.raises(sa.ArgumentError, match="config.json"):
        sa.HFLoader.load_model(str(tmp_path / "nowhere"))


# ---- the trace replay

class FakeModel:
    def __init__(self):
        self.held, self.log = [], []

    def run_rows(self, tokens, rows):
        self.held += tokens
        return np.array([[float(tokens[i]), float(len(self.held))] for i in rows], np.float32).reshape(-1, 2)

    def clear_cache(self):
        self.log.append(len(self.held))
        self.held = []

    def reserve(self, n):
        self.log.append(("room", n))

    def close(self):
        self.log.append("closed")


def test_trace_program(sa, tmp_path, monkeypatch, capsys):
    from shainet_amd import trace

    model = FakeModel()
    monkeypatch.setattr(sa.HFLoader, "load_model", staticmethod(lambda d: model))
    lines = [{"step": 3, "entries": [{"id": "x", "tokens": [5, 6, 7], "want": [2, 0]}], "end": []},
             {"step": 4, "entries": [{"id": "x", "tokens": [8], "want": []}], "end": ["x"]},
             {"step": 5, "entries": [{"id": "y", "tokens": [9], "want": [0]}], "end": ["y"]}]
    monkeypatch.setattr(sys, "stdin", io.StringIO("".join(json.dumps(x) + "\n" for x in lines)))
    assert trace.main(["--model", "m", "--dtype", "bfloat16", "--out", str(tmp_path), "--max-tokens", "12"]) == 0
    assert capsys.readouterr().out == "done 3\ndone 4\ndone 5\n"
    assert model.log == [("room", 12), 4, 1, "closed"]
    assert np.fromfile(tmp_path / "3.f32", "<f4").tolist() == [7, 3, 5, 3]
    assert np.fromfile(tmp_path / "5.f32", "<f4").tolist() == [9, 1] and not (tmp_path / "4.f32").exists()


def test_trace_requests_do_not_overlap():
    from shainet_amd.trace import Replay

    r = Replay(FakeModel())
    r.entry("a", [1, 2], [])
    r.end("b")  # not the one that is running
    with pytest.raises(ValueError):
        r.entry("b", [3], [0])
    with pytest.raises(ValueError):
        r.entry("a", [], [])
    r.end("a")
    assert r.entry("b", [3], [0]).tolist() == [[3, 1]]
