"""Layer-list models without a GPU: the checkpoint container, the tensors of a configuration, the reference functions."""
import json
import struct

import numpy as np
import pytest

from kuiperllama_amd import checkpoint
from oracle import hybrid_ref as R
import layers_util as U


def test_safetensors_image_layout():
    t = {"a": np.arange(6, dtype=np.float32).reshape(2, 3), "b.c": checkpoint.to_bf16(np.array([1.5, -2.0], np.float32))}
    img = checkpoint.safetensors_image(t).tobytes()
    n = struct.unpack("<Q", img[:8])[0]
    h = json.loads(img[8:8 + n])
    assert (8 + n) % 8 == 0 and h["a"]["shape"] == [2, 3] and h["b.c"]["dtype"] == "BF16"
    lo, hi = h["a"]["data_offsets"]
    got = checkpoint.from_bf16(np.frombuffer(img[8 + n + lo:8 + n + hi], np.uint16)).reshape(2, 3)
    assert np.array_equal(got, t["a"])
    assert h["b.c"]["data_offsets"][1] == len(img) - 8 - n


def test_safetensors_image_agrees_with_the_safetensors_package(tmp_path):
    st = pytest.importorskip("safetensors.torch")
    cfg = U.mixed()
    m = U.Model(cfg)
    checkpoint.save(str(tmp_path), cfg, m.bits)
    assert checkpoint.is_checkpoint(str(tmp_path)) and checkpoint.load_config(str(tmp_path)) == cfg
    got = st.load_file(str(tmp_path / "model.safetensors"))
    assert set(got) == set(checkpoint.tensor_shapes(cfg))
    for k, v in got.items():
        assert np.array_equal(v.float().numpy(), m.W[k]), k


def test_bf16_rounds_to_nearest_even():
    import torch
    x = np.random.default_rng(0).standard_normal(4096).astype(np.float32)
    x[:2] = [1.00390625, 1.01171875]  # ties
    assert np.array_equal(checkpoint.from_bf16(checkpoint.to_bf16(x)), torch.from_numpy(x).bfloat16().float().numpy())


def test_tensor_shapes_follow_the_configuration():
    s = checkpoint.tensor_shapes(U.mixed())
    assert s["loop.step"] == (3, 88) and s["l0.mix.x"] == (5 + 12, 72) and s["l2.mix.conv"] == (40, 3)
    assert s["l1.mix.uq"] == (3 * 32, 36) and s["l1.mix.dkv"] == (52, 88) and s["l1.mlp.router"] == (7, 88)
    assert "l2.norm2" not in s and "l3.mlp.shared.gate" not in s and s["l3.mlp.router"] == (5, 88)
    with pytest.raises(ValueError):
        checkpoint.tensor_shapes({"architecture": "other"})


def test_schedule_repeats_the_looped_range():
    assert R.schedule(U.mixed()) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None)]
    assert R.schedule(U.config([U.mamba(), U.mamba()])) == [(0, None), (1, None)]


def test_reference_scan_matches_the_unrolled_sum():
    rng = np.random.default_rng(3)
    T, c, n = 7, 3, 4
    x, dt = rng.standard_normal((T, c)), np.exp(rng.standard_normal((T, c)))
    A, B, C, D = -np.exp(rng.standard_normal((c, n))), rng.standard_normal((T, n)), rng.standard_normal((T, n)), rng.standard_normal(c)
    y = R.selective_scan(x, dt, A, B, C, D)
    for t in range(T):
        want = D * x[t]
        for s in range(t + 1):
            want = want + (np.exp(dt[s + 1:t + 1].sum(0)[:, None] * A) * (dt[s] * x[s])[:, None] * B[s] * C[t]).sum(1)
        assert np.allclose(y[t], want)


def test_reference_rotation_and_sink():
    v = np.random.default_rng(4).standard_normal((9, 2, 12))
    r = R.rope_interleaved(v, 100.0, 8)
    assert np.allclose(np.linalg.norm(r, axis=-1), np.linalg.norm(v, axis=-1)) and np.array_equal(r[:, :, 8:], v[:, :, 8:])
    assert np.array_equal(r[0], v[0])
    s = np.array([[[0.3, -np.inf], [1.0, -np.inf]]])
    a = R.softmax_sink(s, np.array([0.3, 50.0]))
    assert np.isclose(a[0, 0, 0], 0.5) and a[0, 1, 0] < 1e-20 and a[0, 0, 1] == 0


def test_reference_routing_uses_the_correction_for_the_choice_only():
    z = np.array([[0.0, 0.1, 0.2]])
    ids, w = R.route(z, np.array([1.0, 0.0, 0.0]), 2)
    s = np.exp(z[0]) / np.exp(z[0]).sum()
    assert list(ids[0]) == [0, 2] and np.allclose(w[0], s[[0, 2]])


def test_trace_runner_asks_for_its_arguments(capsys):
    from kuiperllama_amd import trace
    with pytest.raises(SystemExit):
        trace.main(["--model", "x"])
    assert "--out" in capsys.readouterr().err


def test_layers_bench_configuration_counts_its_weights():
    import bench
    cfg = bench.layers_config(512, 2)
    elems, head, prompt = bench.layers_work(cfg)
    assert head == 512 * cfg["vocab"]
    m, a = cfg["layers"][0]["mixer"], cfg["layers"][1]["mixer"]
    mam = 512 * 2 * m["inner"] + (m["dt_rank"] + 32) * m["inner"] + m["inner"] * m["dt_rank"] + 512 * m["inner"]
    H, down = a["heads"], 512 * (1536 + 512 + 64)
    lat = down + 1536 * H * 192 + 512 * H * 256 + 512 * H * 128
    ff = 36 * 512 + 512 + 3 * 512 * 512 + 6 * (32 / 36) * 3 * 512 * 256
    assert abs(elems - head - (mam + lat + 2 * ff)) < 1 and abs(prompt - (mam + ff + down)) < 1
