"""The Tutilorn design on a real MI355X against the plain statement of its equations in
tutilorn_oracle.py (fp64): each mechanism in a layer of its own, whole models, and the cache under
every cut of a sequence.  Weights and sizes are this file's own."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import tutilorn_model as tm
import tutilorn_oracle as to

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = 1e-4  # of the largest value of the compared rows: fp32 against fp64, with some peaked softmaxes


@pytest.fixture(scope="module")
def hip():
    import shainet_amd as sa

    assert sa.HIP.fully_available(), "no gfx950 device or libshainet_hip_kernels.so missing"
    return sa


def close(got, want, tol=TOL):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape
    err = np.abs(got - want).max() / np.abs(want).max()
    assert err <= tol, err
    return err


class Pair:
    """A model on the device and what the oracle says of it."""

    def __init__(self, hip, folder, cfg, seed=1, gain=1.0, edit=None):
        self.cfg, self.w = cfg, tm.make_weights(cfg, seed, gain)
        if edit:
            edit(self.w)
        self.model = hip.HFLoader.load_model(tm.write(folder, cfg, self.w))

    def logits(self, tokens):
        return to.forward(self.cfg, self.w, tokens)[0]

    def layer(self, i, x):
        """The oracle's residual after layer i for rows x [T, width] before it."""
        p, lc = f"l{to.owner(self.cfg, i)}.", self.cfg["layers"][i]
        t = lambda n: self.w[n].astype(np.float64)
        norm = lambda v, n: to.dynamic_tanh(v, t(n), t(n + ".b"), float(t(n + ".alpha")))
        x = np.asarray(x, np.float64)
        x = x + to.latent_attention(norm(x, p + "norm1"), lambda n: t(p + "mix." + n), lc["mixer"], self.cfg["norm"]["eps"])
        if lc["mlp"]:
            x = x + to.swiglu(norm(x, p + "norm2"), lambda n: t(p + "mlp." + n))
        return x


def tokens(n, vocab, seed=0):
    return [int(t) for t in np.random.default_rng(seed).integers(0, vocab, n)]


def run_cut(model, ids, cuts):
    """Logits of every token, the sequence brought in portions of the given sizes (the last one repeats)."""
    model.clear_cache()
    out, at, k = [], 0, 0
    while at < len(ids):
        n = min(cuts[min(k, len(cuts) - 1)], len(ids) - at)
        out.append(model.run_rows(ids[at:at + n], range(n)))
        at, k = at + n, k + 1
    return np.concatenate(out)


# what each geometry is there for: multiples of 4 throughout; nothing a multiple of 4, an eps that matters;
# nothing rotated; one head, a window of one; sizes that differ from each other everywhere, no window; ranks above a tile, larger heads
GEOMETRIES = {
    "even": dict(width=64, vocab=96, m=dict(heads=4, dim=32, rot_dim=16, vdim=40, kv_rank=48, q_rank=32, window=24), ff=80),
    "odd": dict(width=55, vocab=83, m=dict(heads=5, dim=13, rot_dim=6, vdim=11, kv_rank=35, q_rank=21, window=9), ff=47, eps=0.2),
    "still": dict(width=40, vocab=40, m=dict(heads=3, dim=16, rot_dim=0, vdim=8, kv_rank=16, q_rank=12, window=20), ff=24),
    "one": dict(width=32, vocab=50, m=dict(heads=1, dim=8, rot_dim=2, vdim=4, kv_rank=12, q_rank=8, window=1), ff=16),
    "open": dict(width=72, vocab=61, m=dict(heads=3, dim=20, rot_dim=12, vdim=36, kv_rank=40, q_rank=64, window=0), ff=44),
    "tall": dict(width=96, vocab=130, m=dict(heads=7, dim=96, rot_dim=32, vdim=96, kv_rank=272, q_rank=144, window=70), ff=128),
    "wide": dict(width=128, vocab=70, m=dict(heads=2, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=96, window=50), ff=64),
    "partial": dict(width=48, vocab=64, m=dict(heads=2, dim=12, rot_dim=12, rot_dims=6, vdim=16, kv_rank=20, q_rank=16, window=12), ff=32),
    "vast": dict(width=64, vocab=64, m=dict(heads=2, dim=224, rot_dim=32, vdim=72, kv_rank=1072, q_rank=16, window=33), ff=32),
}


def geometry(name, layers=1, mlp=True):
    g = GEOMETRIES[name]
    return tm.config([tm.layer(tm.mixer(**g["m"]), g["ff"] if mlp else None) for _ in range(layers)], g["vocab"], g["width"],
                     g.get("eps", 1e-5))


@pytest.mark.parametrize("path", ["absorbed", "expanded"])
@pytest.mark.parametrize("name", sorted(GEOMETRIES))
def test_mixer_alone(hip, tmp_path, monkeypatch, name, path):
    """A layer without feed-forward: both forms of the attention, rows in one call and in cuts."""
    monkeypatch.setenv("SHAINET_HIP_LATENT_PATH", path)
    p = Pair(hip, tmp_path, geometry(name, mlp=False))
    x = np.random.default_rng(3).standard_normal((150, p.cfg["width"])).astype(np.float32)
    want = p.layer(0, x)
    b = p.model.blocks[0]
    close(b.forward_cached(x), want)
    assert b.cache_len == 150
    for cuts in ((1,), (2, 3, 60, 17), (128, 1, 5), (33, 16, 31)):
        b.clear_cache()
        got, at, k = [], 0, 0
        while at < 150:
            n = min(cuts[k % len(cuts)], 150 - at)
            got.append(b.forward_cached(x[at:at + n]))
            at, k = at + n, k + 1
        close(np.concatenate(got), want)
    b.clear_cache()
    close(b.forward(x[:40]), p.layer(0, x[:40]))  # without the cache
    assert b.cache_len == 0


@pytest.mark.parametrize("rows", [1, 3, 16, 17, 150])
@pytest.mark.parametrize("name", ["even", "odd", "open"])
def test_feed_forward_and_norms(hip, tmp_path, name, rows):
    """A mixer that adds nothing (W_o = 0): Dynamic Tanh and the feed-forward are what is left."""
    p = Pair(hip, tmp_path, geometry(name), edit=lambda w: w.update({"l0.mix.o": 0 * w["l0.mix.o"]}))
    x = (3 * np.random.default_rng(rows).standard_normal((rows, p.cfg["width"]))).astype(np.float32)
    close(p.model.blocks[0].forward_cached(x), p.layer(0, x), 1e-5)


def test_norm_inside_the_one_row_products(hip, tmp_path):
    """Widths at which one row takes the products over transposed weights (the norm's own prologue there)."""
    for k, width in enumerate((1024, 2048, 4096)):
        cfg = tm.config([tm.layer(tm.mixer(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=24, q_rank=1024, window=5), 64)], 4200, width)
        p = Pair(hip, tmp_path / str(k), cfg)
        ids = tokens(7, cfg["vocab"])
        want = p.logits(ids)
        close(run_cut(p.model, ids, (1,)), want)
        close(run_cut(p.model, ids, (7,)), want)


def test_latents_in_the_cache(hip, tmp_path):
    """The cached rows themselves: RMS-normed latent, rotated key part, at the right positions."""
    p = Pair(hip, tmp_path, geometry("open", mlp=False))
    m = p.cfg["layers"][0]["mixer"]
    x = np.random.default_rng(5).standard_normal((45, p.cfg["width"])).astype(np.float32)
    b = p.model.blocks[0]
    for lo, hi in ((0, 20), (20, 22), (22, 23), (23, 45)):
        b.forward_cached(x[lo:hi])
    t = lambda n: p.w[n].astype(np.float64)
    h = to.dynamic_tanh(x.astype(np.float64), t("l0.norm1"), t("l0.norm1.b"), float(t("l0.norm1.alpha")))
    down = h @ t("l0.mix.dkv").T
    want = np.concatenate([to.rms_norm(down[:, :m["kv_rank"]], t("l0.mix.dkv.norm"), p.cfg["norm"]["eps"]),
                           to.rope_interleaved(down[:, m["kv_rank"]:], np.arange(45), m["rot"]["base"], m["rot"]["dims"])], -1)
    close(b.cache_rows(0, 45), want, 1e-5)


def standout(p, distance, rows, seed):
    """Rows x for layer 0 in which the last query and the key `distance` before it match as no other pair does:
    the best of many candidate rows for that key, by the oracle's own scores."""
    m, t = p.cfg["layers"][0]["mixer"], lambda n: p.w[n].astype(np.float64)
    r = np.random.default_rng(seed)
    x = r.standard_normal((rows, p.cfg["width"]))
    q_at, k_at = rows - 1, rows - 1 - distance
    cand = 1.5 * r.standard_normal((600, p.cfg["width"]))
    norm = lambda v: to.dynamic_tanh(v, t("l0.norm1"), t("l0.norm1.b"), float(t("l0.norm1.alpha")))
    eps, H, dim, rd, kr = p.cfg["norm"]["eps"], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    turn = lambda v, at: to.rope_interleaved(v, np.full(len(v), at), m["rot"]["base"], m["rot"]["dims"])
    q = (to.rms_norm(norm(x[q_at:]) @ t("l0.mix.dq").T, t("l0.mix.dq.norm"), eps) @ t("l0.mix.uq").T).reshape(H, dim + rd)
    down = norm(cand) @ t("l0.mix.dkv").T
    k = (to.rms_norm(down[:, :kr], t("l0.mix.dkv.norm"), eps) @ t("l0.mix.uk").T).reshape(-1, H, dim)
    score = np.einsum("hd,chd->ch", q[:, :dim], k) + turn(down[:, kr:], k_at) @ turn(q[:, dim:], q_at).T
    x[k_at] = cand[score.max(1).argmax()]
    return x.astype(np.float32)


@pytest.mark.parametrize("path", ["absorbed", "expanded"])
@pytest.mark.parametrize("window,rows", [(17, 60), (32, 90), (33, 90), (64, 140), (129, 300)])
def test_window_edges(hip, tmp_path, monkeypatch, window, rows, path):
    """A key that stands out, just inside and just outside the window, in a prompt and decoded."""
    monkeypatch.setenv("SHAINET_HIP_LATENT_PATH", path)
    cfg = tm.config([tm.layer(tm.mixer(heads=2, dim=32, rot_dim=8, vdim=24, kv_rank=40, q_rank=32, window=window), None)], 40, 64)
    p = Pair(hip, tmp_path, cfg, gain=6.0)
    b = p.model.blocks[0]
    for distance in (window - 2, window - 1, window, window + 1):
        x = standout(p, distance, rows, seed=distance)
        want = p.layer(0, x)
        for other in (window - 1, window + 1) if distance in (window - 1, window) else ():
            # the case can tell: with the edge moved over the key the last row is another one
            m = cfg["layers"][0]["mixer"]
            m["mask"]["size"] = other
            moved = np.abs(p.layer(0, x)[-1] - want[-1]).max() / np.abs(want).max()
            m["mask"]["size"] = window
            if (other < window) == (distance == window - 1):
                assert moved > 100 * TOL, (distance, other, moved)
        for cut in ((rows,), (rows - 1, 1), (rows - 2, 2), (rows - 20, 20), (window, rows), (1,)):
            b.clear_cache()
            got, at, k = [], 0, 0
            while at < rows:
                n = min(cut[min(k, len(cut) - 1)], rows - at)
                got.append(b.forward_cached(x[at:at + n]))
                at, k = at + n, k + 1
            close(np.concatenate(got), want)


@pytest.mark.parametrize("path", ["absorbed", "expanded"])
def test_sink(hip, tmp_path, monkeypatch, path):
    """Sinks that take nearly everything, about half and nothing; the first position sees one key only."""
    monkeypatch.setenv("SHAINET_HIP_LATENT_PATH", path)

    def edit(w):
        w["l0.mix.sink"] = np.array([9.0, 0.5, -60.0, 30.0], np.float32)

    p = Pair(hip, tmp_path, geometry("even", mlp=False), edit=edit)
    x = np.random.default_rng(8).standard_normal((70, p.cfg["width"])).astype(np.float32)
    want = p.layer(0, x)
    b = p.model.blocks[0]
    close(b.forward_cached(x), want)
    b.clear_cache()
    close(np.concatenate([b.forward_cached(x[i:i + 1]) for i in range(70)]), want)


def test_far_key_among_hundreds(hip, tmp_path):
    """No window, key splits in both forms: one key far back decides the last row."""
    cfg = tm.config([tm.layer(tm.mixer(heads=3, dim=32, rot_dim=16, vdim=32, kv_rank=64, q_rank=48, window=0), None)], 40, 64)
    p = Pair(hip, tmp_path, cfg, gain=6.0)
    b = p.model.blocks[0]
    for distance in (699, 640, 351, 1):
        x = standout(p, distance, 700, seed=distance)
        want = p.layer(0, x)
        close(b.forward_cached(x), want)
        b.clear_cache()
        for lo, hi in ((0, 511), (511, 640), (640, 698), (698, 700)):
            close(b.forward_cached(x[lo:hi]), want[lo:hi])
        b.clear_cache()
        b.forward_cached(x[:699])
        close(b.forward_cached(x[699:]), want[699:])
        b.clear_cache()


# layers that differ, layers without a feed-forward, borrowed weights before and after their owner, a chain of them
def mixed_config():
    a, b = tm.mixer(), tm.mixer(heads=2, dim=16, rot_dim=4, vdim=28, kv_rank=24, q_rank=20, window=40, base=300.0)
    return tm.config([tm.layer(a, 52, weights_of=2), tm.layer(b, None), tm.layer(a, 52), tm.layer(b, None, weights_of=1),
                      tm.layer(a, 52, weights_of=0), tm.layer(tm.mixer(window=0), 36)])


def test_model_cut_anywhere(hip, tmp_path):
    p = Pair(hip, tmp_path, mixed_config())
    ids = tokens(260, p.cfg["vocab"])
    want = p.logits(ids)
    first = run_cut(p.model, ids, (260,))
    close(first, want)
    for cuts in ((1,), (2,), (3, 2, 64), (64,), (100, 2, 37, 1), (17, 16, 15), (259, 1), (228, 1)):
        close(run_cut(p.model, ids, cuts), want)
    assert np.array_equal(run_cut(p.model, ids, (260,)), first)  # nothing of the runs between is left
    for n in (1, 2, 3):  # the first tokens of a sequence
        close(run_cut(p.model, ids[:n], (n,)), want[:n])
    p.model.clear_cache()
    close(p.model.run_full(ids), want[-1])
    assert p.model.cache_len == 0
    close(p.model.run(ids), want[-1])


def test_requests_after_each_other(hip, tmp_path):
    """Unequal requests over the same caches, each as if it were alone."""
    p = Pair(hip, tmp_path, mixed_config(), seed=4)
    for k, n in enumerate((150, 1, 37, 2, 300, 16, 17)):
        ids = tokens(n, p.cfg["vocab"], seed=k)
        close(run_cut(p.model, ids, (max(1, n // 2), 3)), p.logits(ids))


def test_wanted_rows(hip, tmp_path):
    p = Pair(hip, tmp_path, mixed_config(), seed=2)
    ids = tokens(40, p.cfg["vocab"])
    want = p.logits(ids)
    close(p.model.run_rows(ids[:30], [29, 0, 7, 7]), want[[29, 0, 7, 7]])
    assert p.model.run_rows(ids[30:35], []).shape == (0, p.cfg["vocab"])
    close(p.model.logits(), want[34])  # the last row is there for the sampler whatever was wanted
    close(p.model.run_rows(ids[35:], [4, 1]), want[[39, 36]])
    for bad in ([5], [-1]):
        with pytest.raises(hip.ArgumentError):
            p.model.run_rows(ids[:5], bad)


def test_long_decoding_in_a_window_sized_cache(hip, tmp_path):
    """Rows that nobody sees any more are dropped again and again, and the cache stays as large as the window needs."""
    cfg = tm.config([tm.layer(tm.mixer(window=21), 52), tm.layer(tm.mixer(window=21, heads=2), None)])
    p = Pair(hip, tmp_path, cfg, seed=6)
    ids = tokens(1300, cfg["vocab"])
    want = p.logits(ids)
    p.model.reserve(4000)
    close(run_cut(p.model, ids, (90, 1)), want)
    assert p.model.cache_len == 1300
    for b in p.model.blocks:
        assert b.cache_capacity <= 256 + 21, b.cache_capacity
        with pytest.raises(hip.ArgumentError):
            b.cache_rows(0, 1)  # dropped
    close(run_cut(p.model, ids, (200, 60, 2, 3)), want)


def test_greedy_generation(hip, tmp_path):
    """The framework's own loop, its stop tokens and its sampler, against the oracle's argmax."""
    p = Pair(hip, tmp_path, mixed_config(), seed=9)
    prompt = tokens(33, p.cfg["vocab"], seed=2)
    ids, margin = list(prompt), np.inf
    for _ in range(60):
        row = p.logits(ids)[-1]
        top = np.sort(row)[-2:]
        margin = min(margin, (top[1] - top[0]) / np.abs(row).max())
        ids.append(int(row.argmax()))
    assert margin > 3e-5, margin  # no near-tie in the way
    want = ids[33:]
    p.model.run(prompt, want_logits=False)
    assert hip.Sampler.greedy(p.model) == want[0]
    assert p.model.generate_greedy(60) == want
    assert p.model.cache_len == 33 + 60
    # a stop token ends it and takes the steps after it back
    stop = want[24]
    k = want.index(stop)
    p.model.clear_cache()
    p.model.run(prompt, want_logits=False)
    assert p.model.generate_greedy(60, [stop]) == want[:k]
    assert p.model.cache_len == 33 + k
    close(p.model.run_rows([stop, want[k + 1]], [0, 1]), p.logits(prompt + want[:k] + [stop, want[k + 1]])[-2:])
    sampler = hip.Sampler(temperature=0.7, top_k=5)
    assert sampler.sample_on_device(p.model, 0.0) == hip.Sampler.greedy(p.model)


def test_stop_token_in_a_window_sized_cache(hip, tmp_path):
    """Taking steps back after rows have been dropped."""
    p = Pair(hip, tmp_path, tm.config([tm.layer(tm.mixer(window=5), 52)]), seed=3)
    p.model.run(tokens(240, p.cfg["vocab"]), want_logits=False)
    ids = tokens(240, p.cfg["vocab"]) + p.model.generate_greedy(90)
    p.model.clear_cache()
    p.model.run(ids[:240], want_logits=False)
    assert p.model.generate_greedy(90) == ids[240:]
    p.model.clear_cache()
    p.model.run(ids[:240], want_logits=False)
    got = p.model.generate_greedy(90, [ids[290]])
    at = 240 + len(got)
    assert ids[at] == ids[290] and got == ids[240:at]
    close(p.model.run(ids[at:at + 1]), p.logits(ids[:at + 1])[-1])


def test_trace_replay(hip, tmp_path):
    """bin/trace_run as a program: portions, wanted rows, requests one after the other."""
    p = Pair(hip, tmp_path / "m", mixed_config(), seed=12)
    a, b = tokens(50, p.cfg["vocab"], 1), tokens(20, p.cfg["vocab"], 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:41], "want": [0, 40]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[41:43], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[43:], "want": [6, 2]}], "end": ["a"]},
             {"step": 7, "entries": [{"id": "b", "tokens": b, "want": list(range(20))}], "end": ["b"]}]
    out = tmp_path / "out"
    out.mkdir()
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype",
                          "float32", "--out", str(out), "--max-tokens", "64"], input="\n".join(map(json.dumps, steps)) + "\n",
                         capture_output=True, text=True, timeout=100)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [ln for ln in run.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2", "done 7"]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "7.f32"]
    read = lambda n: np.fromfile(out / f"{n}.f32", "<f4").reshape(-1, p.cfg["vocab"])
    la = p.logits(a)
    close(read(0), la[[0, 40]])
    close(read(2), la[[49, 45]])
    close(read(7), p.logits(b))


def test_llama_through_the_same_entry_point(hip):
    """A "model_type" config takes the LLaMA-family loader."""
    folder = os.path.join(ROOT, "tests", "golden", "tiny-llama")
    m, n = hip.HFLoader.load_model(folder), hip.HFLoader.load_llama(folder)
    ids = [1, 5, 9, 2]
    assert np.array_equal(m.run(ids), n.run(ids))
    m.clear_cache()
    rows = m.run_rows(ids, [1, 3])
    m.clear_cache()
    close(rows[0], m.run(ids[:2]))
