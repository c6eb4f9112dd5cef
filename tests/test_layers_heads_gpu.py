"""Grouped-head layer-list models (Gusorax) on the GPU against the plain reference (oracle/hybrid_ref.py): each mechanism
alone, prompts, portions, decoding, batches, cache rows that are used again, keys at every edge, generation."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import layers_util as U
from kuiperllama_amd import _ffi, checkpoint
from oracle import hybrid_ref as R

pytestmark = pytest.mark.gpu
BOTH = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
ROOT = os.path.abspath(os.path.join(os.path.dirname(__file__), ".."))


@pytest.fixture
def hook():
    """Set library hooks for one test."""
    keys = []

    def set_(k, v):
        keys.append(k)
        _ffi.debug_set(k, v)
    yield set_
    for k in keys:
        _ffi.debug_set(k, None)


@pytest.fixture(scope="module")
def mixed():
    return U.Model(U.heads_mixed())


def against_reference(mod, dtype, n=75, cuts=(), **kw):
    m = mod.load(dtype, **kw)
    toks = mod.tokens(n)
    want = mod.logits(toks)
    U.check(U.run_alone(m, toks, cuts), want, dtype, "prompt")
    s = m.open_seq()  # token by token through the fused decode step
    got = np.concatenate([m.forward([(s, [t], [0])]) for t in toks])
    m.close()
    U.check(got, want, dtype, "decode")


# ---- each mechanism alone ---------------------------------------------------------------------------------------
SHAPES = [dict(), dict(heads=1, kv_heads=1, dim=1, vdim=1), dict(heads=3, kv_heads=3, dim=64, vdim=80),
          dict(heads=8, kv_heads=1, dim=80, vdim=64), dict(heads=34, kv_heads=2, dim=16, vdim=16),
          dict(heads=4, kv_heads=2, dim=130, vdim=33, scale=0.1), dict(heads=2, kv_heads=1, dim=65, vdim=200, scale=0.2),
          dict(heads=2, kv_heads=2, dim=256, vdim=256, scale=0.06)]


@BOTH
@pytest.mark.parametrize("kw", SHAPES)
def test_window_attention_alone(gpu, dtype, kw):
    against_reference(U.Model(U.gusorax([U.windowed(**kw)])), dtype)


@BOTH
@pytest.mark.parametrize("kw", SHAPES)
def test_chunk_attention_alone(gpu, dtype, kw):
    against_reference(U.Model(U.gusorax([U.chunked(**kw)])), dtype)


@pytest.mark.parametrize("size", [1, 2, 15, 16, 17, 31, 32, 33, 63, 64, 65, 127, 128, 129, 300])
def test_span_sizes(gpu, size):
    against_reference(U.Model(U.gusorax([U.windowed(window=size), U.chunked(chunk=size)])), "float32", n=150)


@BOTH
@pytest.mark.parametrize("ff", [U.dense(1), U.dense(40), U.dense(130), U.clamped(1, 1, 5), U.clamped(6, 6, 64, 0.1),
                                U.clamped(70, 5, 8, 3.0), U.clamped(300, 2, 4, 0.5)])
def test_feed_forwards_alone(gpu, dtype, ff):
    against_reference(U.Model(U.gusorax([dict(U.windowed(), mlp=ff)])), dtype, n=41)


@BOTH
@pytest.mark.parametrize("loop", [None, (0, 1, 1), (0, 2, 3), (1, 3, 2), (2, 3, 2), (0, 3, 2)])
def test_loop_ranges(gpu, dtype, loop):
    layers = [dict(U.chunked(), mlp=U.clamped()), U.windowed(), dict(U.windowed(2, 1), mlp=U.dense())]
    against_reference(U.Model(U.gusorax(layers, loop=loop)), dtype, n=30)


@pytest.mark.parametrize("kw", [dict(width=64, vocab=64), dict(width=33, vocab=7, eps=1e-1), dict(width=300, vocab=1001, mult=1.0),
                                dict(width=90, scale=1.0, mult=-0.7), dict(width=1, vocab=2)])
def test_widths_vocabularies_and_constants(gpu, kw):
    against_reference(U.Model(U.gusorax([dict(U.windowed(), mlp=U.clamped()), dict(U.chunked(), mlp=U.dense())], **kw)), "float32", n=19)


@BOTH
def test_residual_after_every_layer_run(gpu, mixed, dtype):
    toks = mixed.tokens(45)
    want = []
    mixed.logits(toks, residuals=want)
    m = mixed.load(dtype)
    buf = np.zeros(len(want) * len(toks) * 72, np.float32)
    m.probe_residual(buf)
    m.forward([(m.open_seq(), toks, [])])
    assert m.probe_residual(None) == buf.size and len(want) == 8
    m.close()
    for i, (g, w) in enumerate(zip(buf.reshape(len(want), len(toks), 72), want)):
        U.check(g, w, dtype, f"run {i}")


# ---- prompts, portions, decoding --------------------------------------------------------------------------------
@BOTH
@pytest.mark.parametrize("cuts", [(2,), (1, 3, 5, 7), (63,), (64,), (33, 38, 40, 67), (32, 64, 96, 128), (100, 101, 102, 150),
                                  tuple(range(2, 170, 2))])
def test_portions(gpu, mixed, dtype, cuts):
    toks = mixed.tokens(171)
    m = mixed.load(dtype)
    got = U.run_alone(m, toks, cuts)
    m.close()
    U.check(got, mixed.logits(toks), dtype, str(cuts))


@pytest.mark.parametrize("n", [1, 2, 3, 10, 11, 12, 18, 19, 20, 31, 32, 33, 64, 65, 129])
def test_prompt_lengths_and_first_tokens(gpu, mixed, n):
    toks = mixed.tokens(n, seed=n)
    m = mixed.load()
    got = U.run_alone(m, toks)
    m.close()
    U.check(got, mixed.logits(toks), "float32", str(n))


@BOTH
@pytest.mark.parametrize("tmax", ["32", "64", None])
def test_long_decoding_and_cache_rows_used_again(gpu, mixed, dtype, tmax, hook):
    """Small passes make small rings of cache rows: positions wrap around them several times, in prompts and decoding."""
    if tmax:
        hook("KH_HY_TMAX", tmax)
    toks = mixed.tokens(430)
    want = mixed.logits(toks)
    m = mixed.load(dtype)
    for cuts in ((), (29,) + tuple(range(30, 430)), (200, 231, 233) + tuple(range(300, 340))):
        U.check(U.run_alone(m, toks, cuts), want, dtype, str(cuts[:2]))
    m.close()


def test_cache_rows_are_bounded_by_the_span(gpu):
    mod = U.Model(U.gusorax([U.windowed(heads=8, kv_heads=8, dim=64, vdim=64), U.chunked()], positions=60000))
    a, b = mod.load("bfloat16", max_seq_len=5000), mod.load("bfloat16", max_seq_len=60000)
    assert a.kv_bytes()[0] == b.kv_bytes()[0] < 60000 * 8 * 128 * 2
    a.close()
    b.close()


@BOTH
@pytest.mark.parametrize("rows", ["16", "64", "128"])
@pytest.mark.parametrize("kw", [dict(), dict(dim=128, vdim=100), dict(heads=9, kv_heads=3, dim=70, vdim=40)])
def test_every_row_tile(gpu, dtype, rows, kw, hook):
    """The attention kernel's tile heights on prompts that start anywhere (fp32 and large heads take 64 for 128)."""
    hook("KH_HY_ROWS", rows)
    mod = U.Model(U.gusorax([U.windowed(window=45, **kw), U.chunked(chunk=70, **kw), U.windowed(window=150, rows=16, far=100.0, **kw)]))
    toks = mod.tokens(300)
    want = mod.logits(toks)
    m = mod.load(dtype)
    for cuts in ((), (101, 233)):
        U.check(U.run_alone(m, toks, cuts), want, dtype, str(cuts))
    m.close()


def test_prompt_of_several_passes(gpu):
    """More tokens than one pass holds."""
    mod = U.Model(U.gusorax([U.windowed(8, 2, 16, 16, 0.4, 300, 16, 100.0), dict(U.chunked(16, 8, 8, 8, 0.5, 256), mlp=U.clamped(3, 2, 8))],
                            width=40, vocab=50, positions=2300))
    toks = mod.tokens(2200)
    want = mod.logits(toks)
    for dtype in ("float32", "bfloat16"):
        m = mod.load(dtype, max_seq_len=2200)
        U.check(U.run_alone(m, toks), want, dtype, "one call")
        U.check(U.run_alone(m, toks, (700, 2100)), want, dtype, "three calls")
        m.close()


def test_unfused_and_fused_steps_agree(gpu, mixed, hook):
    toks = mixed.tokens(70)
    m = mixed.load()
    fused = U.run_alone(m, toks, tuple(range(1, 70)))
    hook("KH_HY_DECODE", "0")
    plain = U.run_alone(m, toks, tuple(range(1, 70)))
    m.close()
    U.check(fused, plain.astype(np.float64), "float32")


# ---- keys that matter -------------------------------------------------------------------------------------------
def planted_key(layer, distance, T):
    """Positions do not enter the tokens; token 1's queries of head 0 point at token 2's key: its score is 24 there."""
    cfg = U.gusorax([layer], width=64, vocab=40, eps=1e-6)
    mx, p = layer["mixer"], "l0.mix"
    dk = mx["dim"]
    cfg["layers"][0]["mixer"]["scale"] = 24.0 / dk

    def edit(W):
        W["pos"][:] = 0
        W[p + ".q.norm"][:] = 1
        W[p + ".k.norm"][:] = 1
        if p + ".rel" in W:
            W[p + ".rel"] *= 0.2
        for n in (".q.b", ".k.b"):
            if p + n in W:
                W[p + n][:] = 0
        key = W[p + ".k"][:dk] @ R.rms_norm(W["embed"][2].astype(np.float64) * 6.5, 1.0 + W["l0.norm1"], 1e-6)
        ask = R.rms_norm(W["embed"][1].astype(np.float64) * 6.5, 1.0 + W["l0.norm1"], 1e-6)
        W[p + ".q"][:dk] = np.outer(key, ask / np.dot(ask, ask))
    toks = [int(t) for t in np.random.default_rng(5).integers(3, 40, T)]
    toks[T - 1], toks[T - 1 - distance] = 1, 2
    return U.Model(cfg, edit=edit), toks


def planted_check(mod, toks, distance, seen):
    T = len(toks)
    want = mod.logits(toks)
    moved = list(toks)
    moved[T - 1 - distance] = 3
    change = U.errors(mod.logits(moved)[-1:], want[-1:])[0]
    assert change > 0.05 if seen else change == 0  # the planted key decides the last position, or is not seen at all
    m = mod.load()
    for cuts in ((), (T - 1,), (T - 2,), (T // 3, 2 * T // 3, T - 5) + tuple(range(T - 4, T))):
        U.check(U.run_alone(m, toks, cuts)[-3:], want[-3:], "float32", str((distance, cuts)))
    m.close()


@pytest.mark.parametrize("window", [3, 32, 64, 100, 129])
@pytest.mark.parametrize("back", [1, 2, -1, 0, 1000])
def test_one_key_at_the_edge_of_a_window(gpu, window, back):
    """Just inside (back 1: the last key the window keeps), just outside, and next to the query."""
    distance = 1 if back == 1000 else window - back
    mod, toks = planted_key(U.windowed(4, 2, 32, 32, window=window, rows=16, far=90.0), distance, 260)
    planted_check(mod, toks, distance, distance < window)


@pytest.mark.parametrize("chunk,offset", [(c, o) for c in (3, 32, 50, 64, 128) for o in (0, 1, 2, -1) if c - 1 - o > 0])
def test_one_key_at_the_edge_of_a_chunk(gpu, chunk, offset):
    """The query is the last position of its chunk; the key is the chunk's first, second, third, or the one before it."""
    T = 4 * chunk if chunk > 3 else 66
    distance = chunk - 1 - offset
    mod, toks = planted_key(U.chunked(4, 2, 32, 32, chunk=chunk), distance, T)
    planted_check(mod, toks, distance, offset >= 0)


@pytest.mark.parametrize("distance", [1, 31, 32, 33, 64, 127, 128, 255, 399])
def test_one_key_among_hundreds(gpu, distance):
    for layer in (U.windowed(4, 1, 32, 32, window=420, rows=16, far=90.0), U.chunked(4, 1, 32, 32, chunk=500)):
        mod, toks = planted_key(layer, distance, 400)
        planted_check(mod, toks, distance, True)


@BOTH
@pytest.mark.parametrize("kw", [dict(), dict(rows=16, far=40.0, window=150), dict(heads=64, kv_heads=1, rows=8, far=140.0, window=170),
                                dict(rows=2, far=9.0, window=40), dict(rows=40, far=500.0, window=200)])
def test_bias_by_distance_alone(gpu, dtype, kw):
    """No content scores: the weights are the softmax of the distance table, also beyond its last border and when the
    table does not fit the staging memory."""
    def edit(W):
        W["l0.mix.q.norm"][:] = 0
        W["l0.mix.rel"] = W["l0.mix.rel"] * 3
    mod = U.Model(U.gusorax([U.windowed(**kw)]), edit=edit)
    flat = U.Model(mod.cfg, edit=lambda W: (edit(W), W["l0.mix.rel"].fill(0)))
    toks = mod.tokens(190)
    assert np.median(U.errors(flat.logits(toks), mod.logits(toks))) > 0.02
    against_reference(mod, dtype, n=190, cuts=(33, 160))


@BOTH
def test_sink_takes_its_share(gpu, dtype):
    """Equal scores of 0: position i of a chunk gives each of its i + 1 keys the weight 1 / (i + 2)."""
    mod = U.Model(U.gusorax([U.chunked()]), edit=lambda W: W["l0.mix.q.norm"].fill(0))
    toks = mod.tokens(60)
    W = {k: v.astype(np.float64) for k, v in mod.W.items()}
    h = R.rms_norm(R.Gusorax.embed(W, mod.cfg, np.array(toks)), 1.0 + W["l0.norm1"], 2e-4)
    m = mod.cfg["layers"][0]["mixer"]
    none = R.grouped_attention(W, "l0.mix", m, h, 2e-4, R.visible(60, chunk=19), extra=0.0, gate=True)
    assert np.abs(none - R.chunk_attention(W, "l0.mix", m, h, 2e-4))[19].max() > 0.05  # first of a chunk: half the weight
    against_reference(mod, dtype, n=60)


@BOTH
def test_output_gate_and_biases_count(gpu, dtype):
    def edit(W):
        W["l0.mix.g"] = W["l0.mix.g"] * 4
        for n in (".q.b", ".k.b", ".v.b", ".o.b"):
            W["l0.mix" + n] = W["l0.mix" + n] * 10
    against_reference(U.Model(U.gusorax([U.chunked()]), edit=edit), dtype, n=60)


def test_every_pass_keeps_its_own_cache(gpu):
    """Different inputs per pass: shared rows would show at the second token already."""
    mod = U.Model(U.gusorax([U.windowed(scale=1.0), U.chunked(scale=1.0)], loop=(0, 2, 4)))
    toks = mod.tokens(50)
    m = mod.load()
    U.check(U.run_alone(m, toks, tuple(range(1, 50))), mod.logits(toks), "float32")
    m.close()


# ---- batches and slots ------------------------------------------------------------------------------------------
@BOTH
@pytest.mark.parametrize("lens", [(1, 40, 7), (65, 64, 63, 2), (3, 3), (90, 1, 33, 12, 5, 70, 2)])
def test_batches_of_unequal_requests(gpu, mixed, dtype, lens):
    reqs = [mixed.tokens(n + 12, seed=10 + i) for i, n in enumerate(lens)]
    want = [mixed.logits(r) for r in reqs]
    m = mixed.load(dtype)
    seqs = [m.open_seq() for _ in lens]
    z = m.forward([(s, r[:n], list(range(n))) for s, r, n in zip(seqs, reqs, lens)])
    at = 0
    for w, n in zip(want, lens):
        U.check(z[at:at + n], w[:n], dtype, "prompt")
        at += n
    got = [[] for _ in lens]
    for k in range(12):  # shorter requests end earlier
        live = [i for i in range(len(lens)) if k < 12 - i]
        z = m.forward([(seqs[i], [reqs[i][lens[i] + k]], [0]) for i in live])
        for i, row in zip(live, z):
            got[i].append(row)
    for i, g in enumerate(got):
        U.check(np.array(g), want[i][lens[i]:lens[i] + len(g)], dtype, f"decoded {i}")
    m.close()


def test_prompt_portion_and_decode_in_one_batch(gpu, mixed):
    a, b, c = mixed.tokens(50, 1), mixed.tokens(45, 2), mixed.tokens(90, 3)
    m = mixed.load()
    sa, sb, sc = m.open_seq(), m.open_seq(), m.open_seq()
    m.forward([(sa, a[:49], []), (sc, c[:30], [])])
    z = m.forward([(sa, a[49:], [0]), (sb, b, [0, 44]), (sc, c[30:], [0, 59])])
    U.check(z, np.stack([mixed.logits(a)[49], mixed.logits(b)[0], mixed.logits(b)[44], mixed.logits(c)[30], mixed.logits(c)[89]]), "float32")
    m.close()


@pytest.mark.parametrize("tmax", ["32", None])
def test_freed_slots_start_clean(gpu, mixed, tmax, hook):
    if tmax:
        hook("KH_HY_TMAX", tmax)
    m = mixed.load(max_seqs=2)
    long, short = mixed.tokens(240, 3), mixed.tokens(41, 4)
    want = mixed.logits(short)
    keep = m.open_seq()
    m.forward([(keep, long[:170], [])])
    for prompt_first in (True, False):
        s = m.open_seq()
        m.forward([(s, long, [])])
        m.close_seq(s)
        s = m.open_seq()
        assert m.seq_length(s) == 0
        if prompt_first:
            got = m.forward([(s, short, list(range(41)))])
        else:
            got = np.concatenate([m.forward([(s, [t], [0])]) for t in short])
        U.check(got, want, "float32")
        m.close_seq(s)
    U.check(m.forward([(keep, long[170:], list(range(70)))]), mixed.logits(long)[170:], "float32", "the other sequence")
    m.close()


def test_positions_end_where_the_table_ends(gpu):
    mod = U.Model(U.gusorax([U.windowed()], positions=20))
    m = mod.load(max_seq_len=512)
    s, toks = m.open_seq(), mod.tokens(21)
    U.check(m.forward([(s, toks[:20], list(range(20)))]), mod.logits(toks[:20]), "float32")
    with pytest.raises(_ffi.KhError):
        m.forward([(s, toks[20:], [0])])
    m.close()


def test_loader_refuses_what_does_not_fit(gpu, mixed):
    from kuiperllama_amd.model import KuiperModel

    def change(**kw):
        c = json.loads(json.dumps(mixed.cfg))
        c["layers"][0]["mixer"].update(kw)
        return c
    no_loop_matrix = {k: v for k, v in mixed.bits.items() if k != "loop.in"}
    for cfg, img in ((change(kv_heads=4), mixed.image), (change(mask={}), mixed.image), (change(dim=21), mixed.image),
                     (change(bias_max=0), mixed.image), (dict(mixed.cfg, max_positions=701), mixed.image),
                     (mixed.cfg, checkpoint.safetensors_image(no_loop_matrix))):
        with pytest.raises(_ffi.KhError):
            KuiperModel.from_tensors(cfg, img)


# ---- generation -------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("n_prompt", [1, 2, 5, 40])
def test_greedy_generation(gpu, mixed, n_prompt):
    p = mixed.tokens(n_prompt, seed=20)
    total = n_prompt + 30
    want = p[1:] + mixed.greedy(p, 31)
    m = mixed.load()
    for ex in ("graph", "fused", "unfused", "graph"):  # the graphs are replayed after other work on the stream
        assert m.generate(p, total, exec=ex)[0] == want, ex
    stop = want[n_prompt + 5]
    first = want[n_prompt - 1:].index(stop) + n_prompt - 1
    assert m.generate(p, total, exec="graph", stop=[stop])[0] == want[:first]
    m.close()


def test_greedy_batch(gpu, mixed):
    ps = [mixed.tokens(n, seed=30 + n) for n in (3, 17, 1, 8, 33)]
    want = [mixed.greedy(p, 9 + i) for i, p in enumerate(ps)]
    m = mixed.load()
    assert m.generate_batch(ps, [9 + i for i in range(5)]) == want
    assert m.generate_batch(ps[:2], [9, 10], stop=[want[0][4]])[0] == want[0][:want[0].index(want[0][4])]
    m.close()


def test_geometry_beyond_the_fused_step(gpu):
    """A mixer vector that does not fit LDS: decoding and generation run on the pass kernels."""
    mod = U.Model(U.gusorax([U.chunked(170, 1, 4, 250), dict(U.windowed(), mlp=U.dense())], width=16, vocab=30))
    toks = mod.tokens(30)
    for dtype in ("float32", "bfloat16"):
        m = mod.load(dtype)
        U.check(U.run_alone(m, toks, (4, 5, 6, 7) + tuple(range(15, 30))), mod.logits(toks), dtype)
        if dtype == "float32":
            want = toks[1:3] + mod.greedy(toks[:3], 6)
            for ex in ("graph", "fused", "unfused", "graph"):
                assert m.generate(toks[:3], 8, exec=ex)[0] == want, ex
        m.close()


def test_trace_runner_and_command_line(gpu, mixed, tmp_path):
    from kuiperllama_amd import build
    checkpoint.save(str(tmp_path / "model"), mixed.cfg, mixed.bits)
    a, b = mixed.tokens(42, 6), mixed.tokens(25, 7)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:41], "want": [0, 40]}, {"id": "b", "tokens": b[:24], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[41:], "want": [0]}, {"id": "b", "tokens": b[24:], "want": [0]}], "end": ["a", "b"]},
             {"step": 2, "entries": [{"id": "c", "tokens": b, "want": [24]}], "end": ["c"]}]
    (tmp_path / "out").mkdir()
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "model"), "--dtype", "float32",
                        "--out", str(tmp_path / "out"), "--max-tokens", "80"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    za, zb = mixed.logits(a), mixed.logits(b)
    for n, want in ((0, [za[0], za[40]]), (1, [za[41], zb[24]]), (2, [zb[24]])):
        U.check(np.fromfile(tmp_path / "out" / f"{n}.f32", "<f4").reshape(len(want), -1), np.stack(want), "float32", f"step {n}")
    p = mixed.tokens(6, seed=40)
    want = p[1:] + mixed.greedy(p, 10)
    r = subprocess.run([build.build_demo(), str(tmp_path / "model"), "--dtype", "float32", "--prompt", ",".join(map(str, p)), "--steps", "15"],
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert any(line.split() == [str(t) for t in want] for line in r.stdout.splitlines()), r.stdout
