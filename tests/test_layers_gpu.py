"""Layer-list models on the GPU against the plain reference (oracle/hybrid_ref.py): each mechanism alone, prompts,
portions, decoding, batches, slot reuse, far keys, generation, the trace runner."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import layers_util as U
from kuiperllama_amd import _ffi, checkpoint

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
    return U.Model(U.mixed())


def against_reference(mod, dtype, n=37, cuts=(), **kw):
    m = mod.load(dtype, **kw)
    toks = mod.tokens(n)
    U.check(U.run_alone(m, toks, cuts), mod.logits(toks), dtype, "prompt")
    s = m.open_seq()  # token by token through the fused decode step
    got = np.concatenate([m.forward([(s, [t], [0])]) for t in toks])
    m.close()
    U.check(got, mod.logits(toks), dtype, "decode")


# ---- each mechanism alone ---------------------------------------------------------------------------------------
@BOTH
@pytest.mark.parametrize("kw", [dict(), dict(inner=33, state=1, dt_rank=1, conv=1), dict(inner=130, state=20, dt_rank=70, conv=2),
                                dict(inner=64, state=33, dt_rank=16, conv=7), dict(inner=20, state=130, dt_rank=3, conv=4)])
def test_mamba_alone(gpu, dtype, kw):
    against_reference(U.Model(U.config([U.mamba(**kw)])), dtype, n=75)


@BOTH
@pytest.mark.parametrize("kw", [dict(), dict(heads=1, dim=7, rot_dim=2, vdim=5, kv_rank=9, q_rank=11, scale=0.9),
                                dict(heads=17, dim=16, rot_dim=16, vdim=16, kv_rank=66, q_rank=64),
                                dict(heads=5, dim=70, rot_dim=80, vdim=66, kv_rank=140, q_rank=24, scale=0.2),
                                dict(heads=2, dim=130, rot_dim=64, vdim=128, kv_rank=300, q_rank=40, scale=0.1),
                                dict(heads=70, dim=4, rot_dim=4, vdim=4, kv_rank=20, q_rank=20)])
def test_latent_attention_alone(gpu, dtype, kw):
    against_reference(U.Model(U.config([U.latent(**kw)])), dtype, n=75)


@BOTH
@pytest.mark.parametrize("kw", [dict(), dict(identity=0, shared=0), dict(experts=3, identity=1, top=4, ff=17, shared=33),
                                dict(experts=1, identity=0, top=1), dict(experts=70, identity=10, top=6, ff=8, shared=0),
                                dict(experts=300, identity=3, top=2, ff=4, shared=8)])
def test_experts_alone(gpu, dtype, kw):
    against_reference(U.Model(U.config([U.with_ff(U.mamba(), **kw)])), dtype, n=41)


@BOTH
@pytest.mark.parametrize("loop", [None, (0, 1, 1), (0, 2, 3), (1, 3, 2), (2, 3, 2)])
def test_loop_ranges(gpu, dtype, loop):
    layers = [U.with_ff(U.latent()), U.mamba(), U.with_ff(U.latent(2), identity=0)]
    against_reference(U.Model(U.config(layers, loop=loop)), dtype, n=20)


@pytest.mark.parametrize("kw", [dict(width=64, vocab=64), dict(width=33, vocab=7, eps=1e-2), dict(width=300, vocab=1000, cap=None),
                                dict(width=90, cap=1.5)])
def test_widths_vocabularies_and_constants(gpu, kw):
    against_reference(U.Model(U.config([U.with_ff(U.mamba()), U.with_ff(U.latent())], **kw)), "float32", n=19)


@BOTH
def test_residual_after_every_layer_run(gpu, mixed, dtype):
    toks = mixed.tokens(21)
    want = []
    mixed.logits(toks, residuals=want)
    m = mixed.load(dtype)
    buf = np.zeros(len(want) * len(toks) * 88, np.float32)
    m.probe_residual(buf)
    m.forward([(m.open_seq(), toks, [])])
    assert m.probe_residual(None) == buf.size
    m.close()
    for i, (g, w) in enumerate(zip(buf.reshape(len(want), len(toks), 88), want)):
        U.check(g, w, dtype, f"run {i}")


# ---- prompts, portions, decoding --------------------------------------------------------------------------------
@BOTH
@pytest.mark.parametrize("cuts", [(2,), (1, 3, 5, 7), (63,), (64,), (65, 67), (32, 64, 96, 128), (100, 101, 102, 150), tuple(range(2, 170, 2))])
def test_portions(gpu, mixed, dtype, cuts):
    toks = mixed.tokens(171)
    m = mixed.load(dtype)
    got = U.run_alone(m, toks, cuts)
    m.close()
    U.check(got, mixed.logits(toks), dtype, str(cuts))


@pytest.mark.parametrize("n", [1, 2, 3, 31, 32, 33, 63, 64, 65, 127, 128, 129])
def test_prompt_lengths_and_first_tokens(gpu, mixed, n):
    toks = mixed.tokens(n, seed=n)
    m = mixed.load()
    got = U.run_alone(m, toks)
    m.close()
    U.check(got, mixed.logits(toks), "float32", str(n))


def test_long_decoding_after_a_prompt(gpu, mixed):
    toks = mixed.tokens(330)
    m = mixed.load()
    got = U.run_alone(m, toks, (29,) + tuple(range(30, 330)))
    m.close()
    U.check(got, mixed.logits(toks), "float32")


def test_unfused_and_fused_steps_agree(gpu, mixed, hook):
    toks = mixed.tokens(70)
    m = mixed.load()
    fused = U.run_alone(m, toks, tuple(range(1, 70)))
    hook("KH_HY_DECODE", "0")
    plain = U.run_alone(m, toks, tuple(range(1, 70)))
    m.close()
    U.check(fused, plain.astype(np.float64), "float32")


def test_prompt_of_several_passes(gpu):
    """More tokens than one pass holds: state, cache and expanded attention carry over."""
    mod = U.Model(U.config([U.mamba(24, 4, 3, 4), U.with_ff(U.latent(2, 12, 8, 12, 24, 16, 0.6), experts=3, identity=1, top=2, ff=8, shared=8)],
                           width=40, vocab=50))
    toks = mod.tokens(2150)
    want = mod.logits(toks)
    m = mod.load(max_seq_len=2200)
    U.check(U.run_alone(m, toks), want, "float32", "one call")
    U.check(U.run_alone(m, toks, (700, 2100)), want, "float32", "three calls")
    m.close()


# ---- keys that matter -------------------------------------------------------------------------------------------
def sharpen(factor):
    def edit(W):
        for k in W:
            if k.endswith((".uq", ".uk")):
                W[k] = W[k] * factor
    return edit


@BOTH
@pytest.mark.parametrize("expand", ["1", "0"])
def test_far_keys_stand_out(gpu, dtype, expand, hook):
    """Scores so sharp that a position sees one or two keys, anywhere in the sequence."""
    hook("KH_HY_EXPAND", expand)
    mod = U.Model(U.config([U.latent(4, 24, 8, 24, 48, 48, 1.0), U.mamba(), U.latent(2, 40, 24, 20, 100, 48, 1.0)]), edit=sharpen(2.0))
    toks = mod.tokens(300)
    want = mod.logits(toks)
    m = mod.load(dtype)
    for cuts in ((), (128, 256), (161,) + tuple(range(162, 300))):
        got = U.run_alone(m, toks, cuts)
        if dtype == "float32":
            e = U.errors(got, want)
            assert e.max() < 1e-3, (cuts, e.max())
        else:  # sharp scores amplify rounding: most positions still agree
            assert np.median(U.errors(got, want)) < 0.1
    m.close()


def planted_key(distance, T=260):
    """One head attends by content: token 1 asks for token 2 planted `distance` positions before it."""
    mod = U.Model(U.config([U.latent(2, 32, 8, 32, 48, 48, 1.0)], width=64, vocab=40, cap=None))
    toks = [int(t) for t in np.random.default_rng(5).integers(3, 40, T)]
    toks[T - 1], toks[T - 1 - distance] = 1, 2
    from oracle import hybrid_ref as R

    def normed(t):
        return R.layer_norm(mod.W["embed"][t].astype(np.float64), mod.W["l0.norm1"], mod.W["l0.norm1.b"], mod.cfg["norm"]["eps"])

    p, eps = "l0.mix", mod.cfg["norm"]["eps"]
    cq = R.rms_norm(mod.W[p + ".dq"] @ normed(1), mod.W[p + ".dq.norm"], eps)
    c = R.rms_norm((mod.W[p + ".dkv"] @ normed(2))[:48], mod.W[p + ".dkv.norm"], eps)
    key = mod.W[p + ".uk"][:32] @ c  # head 0's key of the planted token

    def edit(W):
        uq = W[p + ".uq"].copy()  # head 0's unrotated query of the asking token: its score with that key is 24
        uq[:32] = 24.0 * np.outer(key / np.dot(key, key), cq / np.dot(cq, cq))
        W[p + ".uq"] = uq
    return U.Model(mod.cfg, edit=edit), toks


@pytest.mark.parametrize("distance", [1, 2, 31, 32, 33, 63, 64, 65, 127, 128, 129, 255, 256, 259])
def test_one_key_at_a_distance(gpu, distance):
    mod, toks = planted_key(distance)
    want = mod.logits(toks)
    moved = list(toks)
    moved[len(toks) - 1 - distance] = 3
    assert U.errors(mod.logits(moved)[-1:], want[-1:])[0] > 0.02  # the planted key decides the last position
    m = mod.load()
    for cuts in ((), (len(toks) - 1,), (64, 128, len(toks) - 2)):
        U.check(U.run_alone(m, toks, cuts)[-3:], want[-3:], "float32", str((distance, cuts)))
    m.close()


def test_sink_takes_its_share(gpu):
    def edit(W):
        W["l0.mix.sink"] = np.array([6.0, -20.0, 0.0], np.float32)
    mod = U.Model(U.config([U.latent()], cap=None), edit=edit)
    none = U.Model(U.config([U.latent()], cap=None), edit=lambda W: W.update({"l0.mix.sink": np.full(3, -30.0, np.float32)}))
    toks = mod.tokens(50)
    want = mod.logits(toks)
    assert np.median(U.errors(none.logits(toks), want)) > 0.05
    m = mod.load()
    U.check(U.run_alone(m, toks), want, "float32", "prompt")
    U.check(U.run_alone(m, toks, tuple(range(1, 50))), want, "float32", "decode")
    m.close()


def test_state_reaches_far(gpu):
    """Slow decays: the first token still shows hundreds of tokens later, across scan chunks and portions."""
    def edit(W):
        W["l0.mix.A_log"] = np.full_like(W["l0.mix.A_log"], -6.0)
    mod = U.Model(U.config([U.mamba()], cap=None), edit=edit)
    toks = mod.tokens(260)
    want = mod.logits(toks)
    other = [toks[0] ^ 1] + toks[1:]
    assert U.errors(mod.logits(other)[-1:], want[-1:])[0] > 1e-3
    m = mod.load()
    for cuts in ((), (1,), (64, 65, 192), (200,) + tuple(range(201, 260))):
        U.check(U.run_alone(m, toks, cuts), want, "float32", str(cuts))
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


def test_prompt_and_decode_in_one_batch(gpu, mixed):
    a, b = mixed.tokens(30, 1), mixed.tokens(45, 2)
    m = mixed.load()
    sa, sb = m.open_seq(), m.open_seq()
    m.forward([(sa, a[:29], [])])
    z = m.forward([(sa, a[29:], [0]), (sb, b, [0, 44])])
    U.check(z, np.stack([mixed.logits(a)[29], mixed.logits(b)[0], mixed.logits(b)[44]]), "float32")
    m.close()


def test_freed_slots_start_clean(gpu, mixed):
    m = mixed.load(max_seqs=2)
    long, short = mixed.tokens(140, 3), mixed.tokens(9, 4)
    want = mixed.logits(short)
    keep = m.open_seq()
    m.forward([(keep, long[:70], [])])
    for prompt_first in (True, False):
        s = m.open_seq()
        m.forward([(s, long, [])])
        m.close_seq(s)
        s = m.open_seq()
        assert m.seq_length(s) == 0
        if prompt_first:
            got = m.forward([(s, short, list(range(9)))])
        else:
            got = np.concatenate([m.forward([(s, [t], [0])]) for t in short])
        U.check(got, want, "float32")
        m.close_seq(s)
    U.check(m.forward([(keep, long[70:], list(range(70)))]), mixed.logits(long)[70:], "float32", "the other sequence")
    m.close()


def test_sequence_errors(gpu, mixed):
    m = mixed.load(max_seqs=1, max_seq_len=16)
    s = m.open_seq()
    for bad in ([(s, [1], []), (s, [2], [])], [(5, [1], [])], [(s, [101], [])], [(s, [-1], [])], [(s, [1] * 17, [])], [(s, [1], [1])]):
        with pytest.raises(_ffi.KhError):
            m.forward(bad)
    with pytest.raises(_ffi.KhError):
        m.open_seq()
    assert m.seq_length(s) == 0
    m.close_seq(s)
    with pytest.raises(_ffi.KhError):
        m.forward([(s, [1], [])])
    m.close()


def test_loader_refuses_what_it_does_not_know(gpu, mixed):
    from kuiperllama_amd.model import KuiperModel
    for cfg in (dict(mixed.cfg, architecture="other"), dict(mixed.cfg, width=89), dict(mixed.cfg, layers=[dict(mixed.cfg["layers"][0], type="x")])):
        with pytest.raises(_ffi.KhError):
            KuiperModel.from_tensors(cfg, mixed.image)
    with pytest.raises(_ffi.KhError):
        KuiperModel.from_tensors(mixed.cfg, mixed.image[:-2])


# ---- generation -------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("n_prompt", [1, 2, 5, 40])
def test_greedy_generation(gpu, mixed, n_prompt):
    p = mixed.tokens(n_prompt, seed=20)
    total = n_prompt + 20
    want = p[1:] + mixed.greedy(p, 21)
    m = mixed.load()
    for ex in ("graph", "fused", "unfused", "graph"):  # the graphs are replayed after other work on the stream
        assert m.generate(p, total, exec=ex)[0] == want, ex
    stop = want[n_prompt + 5]
    first = want[n_prompt - 1:].index(stop) + n_prompt - 1
    assert m.generate(p, total, exec="graph", stop=[stop])[0] == want[:first]
    m.close()


def test_geometry_beyond_the_fused_step(gpu):
    """A mixer vector that does not fit LDS: decoding and generation run on the pass kernels."""
    mod = U.Model(U.config([U.mamba(40000, 2, 2, 4), U.with_ff(U.latent())], width=16, vocab=30))
    toks = mod.tokens(9)
    m = mod.load()
    U.check(U.run_alone(m, toks, (4, 5, 6, 7, 8)), mod.logits(toks), "float32")
    want = toks[1:3] + mod.greedy(toks[:3], 6)
    for ex in ("graph", "fused", "unfused", "graph"):
        assert m.generate(toks[:3], 8, exec=ex)[0] == want, ex
    m.close()


def test_greedy_batch(gpu, mixed):
    ps = [mixed.tokens(n, seed=30 + n) for n in (3, 17, 1, 8, 33)]
    want = [mixed.greedy(p, 9 + i) for i, p in enumerate(ps)]
    m = mixed.load()
    assert m.generate_batch(ps, [9 + i for i in range(5)]) == want
    assert m.generate_batch(ps[:2], [9, 10], stop=[want[0][4]])[0] == want[0][:want[0].index(want[0][4])]
    m.close()


def test_bin_models_take_the_same_entry_points(gpu, oracle):
    from conftest import load_golden
    from kuiperllama_amd.model import KuiperModel
    spec, img, toks, ref = load_golden("ref_llama_gqa_tied")
    m = KuiperModel.from_host_image(img, spec)
    s = m.open_seq()
    z = m.forward([(s, [int(t) for t in toks], [0, len(toks) - 1])])
    assert np.abs(z - ref[[0, len(toks) - 1]]).max() < 1e-4
    m.close()


# ---- trace runner -----------------------------------------------------------------------------------------------
def test_trace_runner(gpu, mixed, tmp_path):
    checkpoint.save(str(tmp_path / "model"), mixed.cfg, mixed.bits)
    a, b = mixed.tokens(12, 6), mixed.tokens(25, 7)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:11], "want": [0, 10]}, {"id": "b", "tokens": b[:24], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[11:], "want": [0]}, {"id": "b", "tokens": b[24:], "want": [0]}], "end": ["a", "b"]},
             {"step": 2, "entries": [{"id": "c", "tokens": b, "want": [24]}], "end": ["c"]}]
    (tmp_path / "out").mkdir()
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "model"), "--dtype", "float32",
                        "--out", str(tmp_path / "out"), "--max-tokens", "64"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    za, zb = mixed.logits(a), mixed.logits(b)
    for n, want in ((0, [za[0], za[10]]), (1, [za[11], zb[24]]), (2, [zb[24]])):
        got = np.fromfile(tmp_path / "out" / f"{n}.f32", "<f4").reshape(len(want), -1)
        U.check(got, np.stack(want), "float32", f"step {n}")


def test_command_line_generates_from_a_folder(gpu, mixed, tmp_path):
    from kuiperllama_amd import build
    checkpoint.save(str(tmp_path), mixed.cfg, mixed.bits)
    p = mixed.tokens(6, seed=40)
    want = p[1:] + mixed.greedy(p, 10)
    r = subprocess.run([build.build_demo(), str(tmp_path), "--dtype", "float32", "--prompt", ",".join(map(str, p)), "--steps", "15"],
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert any(line.split() == [str(t) for t in want] for line in r.stdout.splitlines()), r.stdout
