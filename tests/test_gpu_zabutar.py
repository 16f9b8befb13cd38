"""The Zabutar design on a real MI355X against the plain statement of its equations in zabutar_oracle.py (fp64):
each mechanism in a layer of its own, whole models, and the state and cache under every cut of a sequence.
Weights and sizes are this file's own."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import zabutar_model as zm
import zabutar_oracle as zo

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = 1e-4  # of the largest value of the compared rows: fp32 against fp64


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

    def __init__(self, hip, folder, cfg, seed=1, gain=1.0, edit=None, rel_rows=18):
        self.cfg, self.w = cfg, zm.make_weights(cfg, seed, gain, rel_rows)
        if edit:
            edit(self.w)
        self.model = hip.HFLoader.load_model(zm.write(folder, cfg, self.w))

    def logits(self, tokens):
        with zm.watch_choices() as gaps:
            out = zo.forward(self.cfg, self.w, tokens)[0]
        assert not gaps or min(gaps) > 3e-6, "a choice of experts too close to call: another seed"
        return out

    def layer(self, i, x, kept=None):
        with zm.watch_choices() as gaps:
            out = zo.layer(self.cfg, self.w, i, np.asarray(x, np.float64), {} if kept is None else kept)
        assert not gaps or min(gaps) > 3e-6, "a choice of experts too close to call: another seed"
        return out


def tokens(n, vocab, seed=0):
    return [int(t) for t in np.random.default_rng(seed).integers(0, vocab, n)]


def portions(n, cuts, repeat_last=True):
    at, k = 0, 0
    while at < n:
        c = min(cuts[min(k, len(cuts) - 1) if repeat_last else k % len(cuts)], n - at)
        yield at, at + c
        at, k = at + c, k + 1


def run_cut(model, ids, cuts):
    model.clear_cache()
    return np.concatenate([model.run_rows(ids[a:b], range(b - a)) for a, b in portions(len(ids), cuts)])


def block_cut(block, x, cuts, repeat_last=False):
    block.clear_cache()
    return np.concatenate([block.forward_cached(x[a:b]) for a, b in portions(len(x), cuts, repeat_last)])


CUTS = ((1,), (2, 3, 60, 17), (128, 1, 5), (33, 16, 31), (64,), (65, 63, 2))

# dim up to 160 takes chunks of 64 rows, up to 368 chunks of 32, up to 576 of 16, above that row after row
HGRN2 = {
    "even": dict(width=64, m=dict(heads=4, dim=32, vdim=64)),
    "odd": dict(width=55, m=dict(heads=3, dim=13, vdim=11)),
    "one": dict(width=32, m=dict(heads=1, dim=1, vdim=1)),
    "square": dict(width=72, m=dict(heads=2, dim=128, vdim=128)),
    "wide_values": dict(width=40, m=dict(heads=2, dim=36, vdim=300)),
    "very_wide_values": dict(width=40, m=dict(heads=1, dim=8, vdim=1000)),
    "mid": dict(width=48, m=dict(heads=2, dim=200, vdim=48)),
    "tall": dict(width=48, m=dict(heads=2, dim=420, vdim=20)),
    "vast": dict(width=48, m=dict(heads=1, dim=1200, vdim=36)),
}


@pytest.mark.parametrize("name", sorted(HGRN2))
def test_hgrn2_alone(hip, tmp_path, name):
    g = HGRN2[name]
    p = Pair(hip, tmp_path, zm.config([zm.layer(zm.hgrn2(**g["m"]))], width=g["width"]))
    x = np.random.default_rng(3).standard_normal((150, g["width"])).astype(np.float32)
    want = p.layer(0, x)
    b = p.model.blocks[0]
    assert b.mixer == b.HGRN2 and b.cache_capacity is None
    close(b.forward_cached(x), want)
    assert b.cache_len == 150
    for cuts in CUTS:
        close(block_cut(b, x, cuts), want)
    b.clear_cache()
    b.forward_cached(x[:20])
    close(b.forward(x[:40]), want[:40])  # without the state, which stays as it is
    assert b.cache_len == 20
    close(b.forward_cached(x[20:]), want[20:])


@pytest.mark.parametrize("bias,lower", [(-60.0, 0.0), (-12.0, 0.0), (14.0, 0.0), (0.0, 0.96875), (0.0, 0.0), (3.0, 0.5)])
def test_gates_from_closed_to_open(hip, tmp_path, bias, lower):
    """Gates that forget everything at once, that hardly forget, and a lower bound near 1; some channels each way."""
    def edit(w):
        w["l0.mix.f.b"] = np.where(np.arange(w["l0.mix.f.b"].size) % 3 == 0, 1.5, bias).astype(np.float32)
        w["l0.mix.lower"] = np.full_like(w["l0.mix.lower"], lower)

    p = Pair(hip, tmp_path, zm.config([zm.layer(zm.hgrn2(heads=2, dim=24, vdim=32))]), edit=edit)
    x = np.random.default_rng(5).standard_normal((330, 60)).astype(np.float32)
    want = p.layer(0, x)
    b = p.model.blocks[0]
    close(b.forward_cached(x), want)
    close(block_cut(b, x, (100, 1, 1, 2, 70)), want)


def test_the_state_itself(hip, tmp_path):
    p = Pair(hip, tmp_path, zm.config([zm.layer(zm.hgrn2(heads=2, dim=24, vdim=40))]))
    x = np.random.default_rng(6).standard_normal((83, 60)).astype(np.float32)
    t = lambda n: p.w["l0." + n].astype(np.float64)
    h = zo.rms_norm_zero_centred(x.astype(np.float64), t("norm1"), 1e-5)
    h = h + zo.causal_conv(h, t("canon1"))
    f = zo.forget_gate(h @ t("mix.f").T + t("mix.f.b"), t("mix.lower")).reshape(83, 2, 24)
    v = (h @ t("mix.v").T).reshape(83, 2, 40)
    S = np.zeros((2, 24, 40))
    for i in range(83):
        S = f[i][:, :, None] * S + (1 - f[i])[:, :, None] * v[i][:, None, :]
    b = p.model.blocks[0]
    assert not b.state(2, 24, 40).any()
    for cuts in ((83,), (1,), (40, 2, 41)):
        block_cut(b, x, cuts)
        close(b.state(2, 24, 40), S)
    b.clear_cache()
    assert not b.state(2, 24, 40).any()
    with pytest.raises(hip.ArgumentError):
        b.state(2, 24, 41)


def test_more_chunks_than_fit_at_once(hip, tmp_path):
    """A prompt beyond 64 chunks, with gates so open that its first tokens still count."""
    def edit(w):
        w["l0.mix.lower"] = np.full_like(w["l0.mix.lower"], 0.99609375)

    p = Pair(hip, tmp_path, zm.config([zm.layer(zm.hgrn2(heads=1, dim=8, vdim=8))], width=16), edit=edit)
    x = np.random.default_rng(7).standard_normal((4300, 16)).astype(np.float32)
    x[:64] *= 3
    want = p.layer(0, x)
    close(p.model.blocks[0].forward_cached(x), want)
    close(block_cut(p.model.blocks[0], x, (4200, 100)), want)


# equal and unequal key and value heads, the fused append (powers of two) and the plain one, tiles of 64, 128 and 256,
# sizes no MFMA kernel takes, groups of 1, 5 and 20 heads; rows = rows of the table by distance
ATTENTION = {
    "even": dict(width=64, m=dict(heads=4, kv_heads=2, dim=32, vdim=32, bias_max=90), rows=20),
    "narrow_values": dict(width=64, m=dict(heads=4, kv_heads=4, dim=40, vdim=24, bias_max=33), rows=32),
    "wide_values": dict(width=48, m=dict(heads=2, kv_heads=1, dim=16, vdim=100, bias_max=60), rows=8),
    "odd": dict(width=55, m=dict(heads=5, kv_heads=1, dim=13, vdim=11, bias_max=41), rows=10),
    "odd_values": dict(width=40, m=dict(heads=2, kv_heads=2, dim=16, vdim=9, bias_max=41), rows=10),
    "many_heads": dict(width=40, m=dict(heads=20, kv_heads=1, dim=8, vdim=8, bias_max=50), rows=6),
    "large": dict(width=72, m=dict(heads=3, kv_heads=3, dim=128, vdim=128, bias_max=64), rows=16),
    "larger": dict(width=32, m=dict(heads=2, kv_heads=1, dim=200, vdim=136, bias_max=55), rows=12),
    "largest": dict(width=32, m=dict(heads=2, kv_heads=1, dim=300, vdim=520, bias_max=55), rows=12),
    "far_table": dict(width=48, m=dict(heads=2, kv_heads=2, dim=16, vdim=16, bias_max=100000), rows=40),
    "two_buckets": dict(width=48, m=dict(heads=2, kv_heads=2, dim=16, vdim=16, bias_max=7), rows=2),
    "flat": dict(width=48, m=dict(heads=2, kv_heads=2, dim=16, vdim=16, bias_max=7), rows=1),
}


def attention_config(name, layers=1):
    g = ATTENTION[name]
    return zm.config([zm.layer(zm.attention(**g["m"])) for _ in range(layers)], width=g["width"]), g["rows"]


@pytest.mark.parametrize("name", sorted(ATTENTION))
def test_attention_alone(hip, tmp_path, name):
    cfg, rows = attention_config(name)
    p = Pair(hip, tmp_path, cfg, rel_rows=rows)
    x = np.random.default_rng(3).standard_normal((150, cfg["width"])).astype(np.float32)
    if rows == 1:  # one row for all distances: no bias that a softmax would see
        p.w["l0.mix.rel"] = np.zeros((4, 2), np.float32)
    want = p.layer(0, x)
    b = p.model.blocks[0]
    assert b.mixer == b.BIASED
    close(b.forward_cached(x), want)
    assert b.cache_len == 150
    for cuts in CUTS:
        close(block_cut(b, x, cuts), want)
    b.clear_cache()
    b.forward_cached(x[:20])
    close(b.forward(x[:40]), want[:40])
    assert b.cache_len == 20
    close(b.forward_cached(x[20:]), want[20:])


@pytest.mark.parametrize("dim,kv_heads", [(32, 1), (128, 2), (20, 2)])
def test_bucket_edges(hip, tmp_path, dim, kv_heads):
    """A table that is large in one bucket only, for the bucket's first and last distances, in a prompt, in short
    portions and decoded; the far end of the table, where the last bucket begins, too."""
    rows, bias_max, T = 12, 83, 170
    edges = [next(n for n in range(200) if zo.distance_bucket(n, rows, bias_max) == k) for k in range(rows)]
    for bucket in (0, rows // 2 - 1, rows // 2, rows - 3, rows - 1):
        def edit(w):
            w["l0.mix.rel"] = np.zeros_like(w["l0.mix.rel"])
            w["l0.mix.rel"][bucket] = 9.0

        cfg = zm.config([zm.layer(zm.attention(heads=2, kv_heads=kv_heads, dim=dim, vdim=dim, bias_max=bias_max))], width=48)
        p = Pair(hip, tmp_path / str(bucket), cfg, edit=edit, rel_rows=rows)
        x = np.random.default_rng(bucket).standard_normal((T, 48)).astype(np.float32)
        want = p.layer(0, x)
        plain = zo.distance_bucket
        for step in (1, -1):  # the case can tell: with every edge moved by one the rows are others
            zo.distance_bucket = lambda n, r, far: plain(max(n + step, 0), r, far)
            try:
                assert np.abs(p.layer(0, x) - want).max() / np.abs(want).max() > 20 * TOL, (bucket, step)
            finally:
                zo.distance_bucket = plain
        b = p.model.blocks[0]
        first = edges[bucket]
        for cuts in ((T,), (1,), (first or 1, 1, 1, T), (T - 2, 2), (40, 16, 9)):
            close(block_cut(b, x, cuts, repeat_last=True), want)


def standout(p, layer, distance, rows, seed):
    """Rows x in which the last query and the key `distance` before it match as no other pair does: the key's row is
    the best of many candidates by the oracle's own scores (rows whose convolutions are off)."""
    m, t = p.cfg["layers"][layer]["mixer"], lambda n: p.w[f"l{layer}." + n].astype(np.float64)
    r = np.random.default_rng(seed)
    d = p.cfg["width"]
    x = r.standard_normal((rows, d))
    norm = lambda v: zo.rms_norm_zero_centred(v, t("norm1"), p.cfg["norm"]["eps"])
    cand = r.standard_normal((800, d))
    H, G, dim = m["heads"], m["kv_heads"], m["dim"]
    q = (norm(x[-1:]) @ t("mix.q").T).reshape(H, dim)
    k = (norm(cand) @ t("mix.k").T).reshape(-1, G, dim)
    score = np.stack([k[:, h // (H // G)] @ q[h] for h in range(H)], 1)
    x[rows - 1 - distance] = cand[score.max(1).argmax()]
    return x.astype(np.float32)


def test_far_key_among_hundreds(hip, tmp_path):
    """One key far back decides the last row: key splits in the prompt's and the decode step's kernels."""
    for k, dim in enumerate((32, 128)):
        cfg = zm.config([zm.layer(zm.attention(heads=4, kv_heads=2, dim=dim, vdim=dim, bias_max=70))], width=64, taps=1)
        p = Pair(hip, tmp_path / str(k), cfg, gain=6.0, edit=lambda w: w.update({"l0.canon1": 0 * w["l0.canon1"]}))
        b = p.model.blocks[0]
        for distance in (799, 640, 351, 70, 1):
            x = standout(p, 0, distance, 800, seed=distance)
            want = p.layer(0, x)
            close(b.forward_cached(x), want)
            close(block_cut(b, x, (511, 129, 157, 2, 1), repeat_last=True), want)
            b.clear_cache()


def test_borrowed_keys(hip, tmp_path):
    """Layers that attend over an earlier layer's keys: with a table, scale and output of their own, over other layers between."""
    a = dict(heads=4, kv_heads=2, dim=16, vdim=24, bias_max=40)
    cfg = zm.config([zm.layer(zm.attention(**a), zm.dense()), zm.layer(zm.attention(**a, kv_from=0, scale=0.11)),
                     zm.layer(zm.hgrn2()), zm.layer(zm.attention(**a, kv_from=0), zm.dense(20)),
                     zm.layer(zm.attention(**dict(a, heads=6))), zm.layer(zm.attention(**dict(a, heads=6), kv_from=4))])
    p = Pair(hip, tmp_path, cfg)
    ids = tokens(230, cfg["vocab"])
    want = p.logits(ids)
    for cuts in ((230,), (1,), (100, 2, 37, 1), (17, 16, 15)):
        close(run_cut(p.model, ids, cuts), want)
    close(p.model.run_full(ids[:50]), want[49])
    assert p.model.cache_len == 230
    p.model.clear_cache()
    # a block by itself: its rows have to come behind the owner's
    with pytest.raises(hip.ArgumentError):
        p.model.blocks[1].forward_cached(np.zeros((3, 60), np.float32))


@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 9, 32])
@pytest.mark.parametrize("width", [60, 55])
def test_convolutions(hip, tmp_path, taps, width):
    """Every number of taps in portions shorter and longer than it: both sublayers' earlier rows."""
    cfg = zm.config([zm.layer(zm.hgrn2(heads=2, dim=12, vdim=16), zm.dense(28))], width=width, taps=taps)
    p = Pair(hip, tmp_path, cfg)
    x = np.random.default_rng(taps).standard_normal((75, width)).astype(np.float32)
    want = p.layer(0, x)
    b = p.model.blocks[0]
    close(b.forward_cached(x), want)
    for cuts in ((1,), (2, 3, 1), (8, 9, 7, 1), (30, 2)):
        close(block_cut(b, x, cuts), want)


@pytest.mark.parametrize("rows", [1, 3, 16, 17, 150])
@pytest.mark.parametrize("width,ff", [(64, 96), (55, 47), (60, 1), (1024, 2048)])
def test_dense_feed_forward(hip, tmp_path, rows, width, ff):
    """A mixer that adds nothing (W_o = 0: norm of zeros): norms, convolution and xIELU are what is left."""
    cfg = zm.config([zm.layer(zm.hgrn2(heads=1, dim=4, vdim=4), zm.dense(ff))], width=width, vocab=16, max_positions=160)
    p = Pair(hip, tmp_path, cfg, edit=lambda w: w.update({"l0.mix.o": 0 * w["l0.mix.o"], "l0.mlp.up": 2 * w["l0.mlp.up"]}))
    x = (3 * np.random.default_rng(rows).standard_normal((rows, width))).astype(np.float32)
    close(p.model.blocks[0].forward_cached(x), p.layer(0, x), 2e-5)


MOE = {
    "plain": dict(width=64, moe=dict()),
    "odd": dict(width=55, moe=dict(ff=19, experts=7, identity=2, top=2, groups=3, keep=1, shared=11)),
    "no_identity": dict(width=48, moe=dict(experts=8, identity=0, top=2, groups=2, keep=2)),
    "no_shared": dict(width=48, moe=dict(experts=6, identity=2, top=4, groups=4, keep=3, shared=0, scale=1.0)),
    "one": dict(width=48, moe=dict(experts=1, identity=0, top=1, groups=1, keep=1)),
    "top_one": dict(width=64, moe=dict(experts=12, identity=4, top=1, groups=4, keep=1, scale=2.5)),
    "mostly_identity": dict(width=48, moe=dict(experts=2, identity=14, top=6, groups=4, keep=4)),
    "many": dict(width=64, moe=dict(ff=36, experts=150, identity=10, top=12, groups=8, keep=4)),
    "all": dict(width=48, moe=dict(experts=4, identity=2, top=6, groups=3, keep=3)),
    "big": dict(width=256, moe=dict(ff=160, experts=3, identity=1, top=2, groups=2, keep=2, shared=192)),
}


@pytest.mark.parametrize("name", sorted(MOE))
def test_experts(hip, tmp_path, name):
    """Few rows (a wavefront per output) and many (tiles of 32, 64 and 128 rows per expert), alone and behind each
    other; choice scores below zero."""
    g = MOE[name]
    cfg = zm.config([zm.layer(zm.hgrn2(heads=1, dim=4, vdim=4), zm.moe(**g["moe"]))], width=g["width"])
    off = lambda w: w.update({"l0.mix.o": 0 * w["l0.mix.o"], "l0.mlp.correction": zm.exact(w["l0.mlp.correction"] - 1)})
    p = Pair(hip, tmp_path, cfg, edit=off, seed=3)
    x = (2 * np.random.default_rng(4).standard_normal((420, g["width"]))).astype(np.float32)
    want = p.layer(0, x)
    b = p.model.blocks[0]
    close(b.forward_cached(x), want)
    for cuts in ((1,), (8, 9), (2, 3, 5), (40, 200, 7, 64)):
        close(block_cut(b, x, cuts), want)


def test_optional_parts_left_out(hip, tmp_path):
    """No groups, scale, identity or shared expert in the configuration; a layer without a feed-forward."""
    cfg = zm.config([zm.layer(zm.attention(), zm.moe(experts=5, identity=0, top=2, groups=1, keep=1, scale=1.0, shared=0)),
                     zm.layer(zm.hgrn2(), None)])
    w = zm.make_weights(cfg, 5)
    bare = json.loads(json.dumps(cfg))
    r = bare["layers"][0]["mlp"]["router"]
    del r["groups"], r["scale"], r["identity"]
    m = hip.HFLoader.load_model(zm.write(tmp_path, bare, w))
    ids = tokens(70, cfg["vocab"])
    close(run_cut(m, ids, (70,)), zo.forward(cfg, w, ids)[0])
    close(run_cut(m, ids, (30, 1)), zo.forward(cfg, w, ids)[0])


def test_sizes_of_the_one_row_products(hip, tmp_path):
    """Widths at which one row takes the products over transposed weights: unrotated append, bias and activation there."""
    for k, (width, ff, dim) in enumerate(((1024, 1024, 32), (2048, 4096, 64), (1024, 8192, 128))):
        a = dict(heads=width // dim, kv_heads=2, dim=dim, vdim=dim, bias_max=9)
        cfg = zm.config([zm.layer(zm.attention(**a), zm.dense(ff)), zm.layer(zm.attention(**a, kv_from=0)),
                         zm.layer(zm.hgrn2(heads=2, dim=16, vdim=512), zm.moe(ff=48, shared=64))], 300, width, max_positions=16)
        p = Pair(hip, tmp_path / str(k), cfg, rel_rows=6)
        ids = tokens(11, cfg["vocab"])
        want = p.logits(ids)
        for cuts in ((1,), (11,), (4, 3, 1)):
            close(run_cut(p.model, ids, cuts), want)


def mixed_config(**more):
    return zm.config([zm.layer(zm.hgrn2(), zm.dense()), zm.layer(zm.attention(), zm.moe()), zm.layer(zm.attention(kv_from=1), None),
                      zm.layer(zm.hgrn2(heads=2, dim=33, vdim=20), zm.moe(shared=0, top=2)),
                      zm.layer(zm.attention(heads=4, kv_heads=4, dim=16, vdim=16), zm.dense(36))], **more)


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


def test_one_layer_and_taps_of_one(hip, tmp_path):
    """A single layer, a single tap: nothing carried between layers, no earlier rows kept."""
    p = Pair(hip, tmp_path, zm.config([zm.layer(zm.hgrn2(), zm.moe())], taps=1, eps=0.3))
    ids = tokens(90, p.cfg["vocab"])
    want = p.logits(ids)
    for cuts in ((90,), (1,), (40, 2, 1)):
        close(run_cut(p.model, ids, cuts), want)


def test_requests_after_each_other(hip, tmp_path):
    """Unequal requests over the same state and caches, each as if it were alone."""
    p = Pair(hip, tmp_path, mixed_config(), seed=4)
    for k, n in enumerate((150, 1, 37, 2, 300, 16, 17)):
        ids = tokens(n, p.cfg["vocab"], seed=k)
        close(run_cut(p.model, ids, (max(1, n // 2), 3)), p.logits(ids))


def test_long_decoding(hip, tmp_path):
    p = Pair(hip, tmp_path, mixed_config(), seed=6)
    ids = tokens(1100, p.cfg["vocab"])
    want = p.logits(ids)
    p.model.reserve(1100)
    close(run_cut(p.model, ids, (90, 1)), want)
    assert p.model.cache_len == 1100


def test_positions_end(hip, tmp_path):
    """Position vectors of its own for every position, and no more tokens than there are."""
    p = Pair(hip, tmp_path, mixed_config(max_positions=50))
    ids = tokens(50, p.cfg["vocab"])
    close(run_cut(p.model, ids, (30, 19, 1)), p.logits(ids))
    with pytest.raises(hip.HipError, match="50"):
        p.model.run([1])
    p.model.clear_cache()
    with pytest.raises(hip.HipError, match="50"):
        p.model.run(ids + [1])
    close(run_cut(p.model, ids, (50,)), p.logits(ids))


def test_wanted_rows(hip, tmp_path):
    p = Pair(hip, tmp_path, mixed_config(), seed=2)
    ids = tokens(40, p.cfg["vocab"])
    want = p.logits(ids)
    close(p.model.run_rows(ids[:30], [29, 0, 7, 7]), want[[29, 0, 7, 7]])
    assert p.model.run_rows(ids[30:35], []).shape == (0, p.cfg["vocab"])
    close(p.model.logits(), want[34])
    close(p.model.run_rows(ids[35:], [4, 1]), want[[39, 36]])


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
    # a stop token ends it, and state and caches are those of the tokens before it
    for at in (0, 5, 24, 31):
        stop = want[at]
        k = want.index(stop)
        p.model.clear_cache()
        p.model.run(prompt, want_logits=False)
        assert p.model.generate_greedy(60, [stop]) == want[:k]
        assert p.model.cache_len == 33 + k
        close(p.model.run_rows([stop, want[k + 1]], [0, 1]), p.logits(prompt + want[:k] + [stop, want[k + 1]])[-2:])
    sampler = hip.Sampler(temperature=0.7, top_k=5)
    assert sampler.sample_on_device(p.model, 0.0) == hip.Sampler.greedy(p.model)


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
                          "bfloat16", "--out", str(out), "--max-tokens", "64"], input="\n".join(map(json.dumps, steps)) + "\n",
                         capture_output=True, text=True, timeout=100)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [ln for ln in run.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2", "done 7"]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "7.f32"]
    read = lambda n: np.fromfile(out / f"{n}.f32", "<f4").reshape(-1, p.cfg["vocab"])
    la = p.logits(a)
    close(read(0), la[[0, 40]])
    close(read(2), la[[49, 45]])
    close(read(7), p.logits(b))


def test_what_belongs_to_other_blocks_is_refused(hip, tmp_path):
    p = Pair(hip, tmp_path, mixed_config())
    with pytest.raises(hip.ArgumentError):
        p.model.set_decode_mode(p.model.DECODE_PERSISTENT)
        p.model.run([1])
    p.model.set_decode_mode(p.model.DECODE_AUTO)
    p.model.clear_cache()
    close(p.model.run([1]), p.logits([1])[0])
    with pytest.raises(hip.ArgumentError):
        p.model.blocks[1].state(1, 1, 1)
