"""Grouped-head layer-list models without a GPU: the tensors of a configuration, the reference functions."""
import numpy as np
import pytest

import layers_util as U
from kuiperllama_amd import checkpoint
from oracle import hybrid_ref as R


def test_tensor_shapes_follow_the_configuration():
    s = checkpoint.tensor_shapes(U.heads_mixed())
    assert s["pos"] == (700, 72) and s["loop.in"] == (72, 144) and "loop.step" not in s
    assert s["l0.mix.q"] == (120, 72) and s["l0.mix.k"] == (40, 72) and s["l0.mix.v"] == (56, 72) and s["l0.mix.o"] == (72, 168)
    assert s["l0.mix.rel"] == (12, 6) and s["l0.mix.q.norm"] == (20,) and "l0.mix.q.b" not in s and "l0.mix.g" not in s
    assert s["l1.mix.g"] == (72, 72) and s["l1.mix.v.b"] == (36,) and s["l1.mix.o.b"] == (72,) and "l1.mix.rel" not in s
    assert s["l0.mlp.gate"] == (40, 72) and s["l1.mlp.e6.down"] == (72, 24) and s["l1.mlp.router"] == (7, 72)
    assert not any(k.startswith("l2.mlp") or k.endswith(("correction", "norm1.b", "norm2")) for k in s)


@pytest.mark.parametrize("rows,far", [(16, 100), (32, 128), (8, 9), (12, 100), (2, 7), (6, 4096), (64, 200), (16, 2048)])
def test_distance_buckets_are_exact(rows, far):
    """Against integers: entry half + k starts at the first n with (n / half)^(rows - half) >= (far / half)^k."""
    half = rows // 2
    for n in list(range(0, 300)) + [far - 1, far, far + 1, 5 * far]:
        if n < half:
            want = n
        else:
            k = 0
            while k < rows and n ** (rows - half) * half ** (k + 1) >= far ** (k + 1) * half ** (rows - half):
                k += 1
            want = min(rows - 1, half + k)
        assert R.distance_bucket(n, rows, far) == want, n


def test_visible_keys():
    w, c = R.visible(7, window=3), R.visible(7, chunk=3)
    assert [list(np.flatnonzero(r)) for r in w][4:] == [[2, 3, 4], [3, 4, 5], [4, 5, 6]] and list(np.flatnonzero(w[1])) == [0, 1]
    assert [list(np.flatnonzero(r)) for r in c] == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]


def test_extra_term_of_the_softmax():
    s = np.array([[[0.0, 0.0, -np.inf], [-900.0, -np.inf, -np.inf], [800.0, 800.0, -np.inf]]])
    p = R.softmax_extra(s, 1.0)
    assert np.allclose(p[0], [[1 / 3, 1 / 3, 0], [0, 0, 0], [0.5, 0.5, 0]])
    assert np.allclose(R.softmax_extra(s, 0.0)[0, :2], [[0.5, 0.5, 0], [1, 0, 0]])


def test_choice_weights_cover_the_chosen_only():
    ids, w = R.route_chosen(np.array([[1.0, 3.0, 2.0, 3.0]]), 3)
    assert list(ids[0]) == [1, 3, 2]
    e = np.exp([0.0, 0.0, -1.0])
    assert np.allclose(w[0], e / e.sum())


def test_clamped_expert_limits_both_sides():
    W = {"e.gate": np.eye(2), "e.up": np.array([[0.0, 1.0], [1.0, 0.0]]), "e.down": np.eye(2)}
    y = R.clamped_expert(W, "e", np.array([[5.0, -5.0]]), 0.5)
    g = np.array([0.5, -5.0])  # the gate has an upper limit only
    assert np.allclose(y[0], g / (1 + np.exp(-1.702 * g)) * (np.array([-0.5, 0.5]) + 1))


def test_loop_enters_through_its_matrix():
    m = U.Model(U.gusorax([U.windowed(), U.windowed()], loop=(0, 1, 2)))
    m.W["loop.in"] = np.concatenate([np.zeros((72, 72)), np.eye(72)], axis=1).astype(np.float32)  # forget x, keep the embedding
    res = []
    m.logits([3, 1, 4], residuals=res)
    assert len(res) == 3 and np.allclose(res[0], res[1]) and not np.allclose(res[1], res[2])


def test_norm_weights_are_around_zero_and_the_pass_is_scaled():
    m = U.Model(U.gusorax([U.windowed()], mult=0.0))
    m.W["final.norm"] = np.zeros(72, np.float32)
    x = m.W["embed"][[7]].astype(np.float64) * 6.5 + m.W["pos"][:1]
    want = x / np.sqrt((x * x).mean() + 2e-4) @ m.W["head"].astype(np.float64).T
    assert np.allclose(m.logits([7]), want)


def test_layers_bench_configuration_counts_its_weights():
    import bench
    cfg = bench.layers_config(512, 3, arch="Gusorax")
    elems, head, prompt = bench.layers_work(cfg)
    H, G = cfg["layers"][0]["mixer"]["heads"], cfg["layers"][0]["mixer"]["kv_heads"]
    win = 512 * 128 * (2 * H + 2 * G)
    chk = 512 * 128 * (3 * H + 2 * G)
    dense, moe = 3 * 512 * 1792, 32 * 512 + 7 * 3 * 512 * 256
    assert abs(elems - head - (2 * win + chk + dense + 2 * moe)) < 1
    assert abs(prompt - (win + chk + dense + moe + 512 * 128 * 2 * G)) < 1
