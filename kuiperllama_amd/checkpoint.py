"""Checkpoint folders of layer-list models: config.json (architecture, layers and their sizes, constants) beside
model.safetensors.  The library reads both itself (csrc/kh_hybrid_load.hip); this module is the host-side mirror of the
format: the tensors a configuration asks for, a writer for the safetensors container, and seeded random models.
"""
from __future__ import annotations

import json
import os
import struct
from typing import Dict, Iterator, Optional, Sequence, Tuple

import numpy as np

ARCHITECTURES = ("Gufanex",)


def load_config(folder: str) -> dict:
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)


def is_checkpoint(path: str) -> bool:
    return os.path.isdir(path) and os.path.exists(os.path.join(path, "config.json"))


def _mixer_tensors(p: str, kind: str, m: dict, W: int) -> Iterator[Tuple[str, tuple]]:
    if kind == "mamba1":
        c, n, r = m["inner"], m["state"], m["dt_rank"]
        yield from ((p + ".in", (2 * c, W)), (p + ".conv", (c, m["conv"])), (p + ".conv.b", (c,)),
                    (p + ".x", (r + 2 * n, c)), (p + ".dt", (c, r)), (p + ".dt.b", (c,)), (p + ".A_log", (c, n)),
                    (p + ".D", (c,)), (p + ".o", (W, c)))
    elif kind == "latent_attention":
        H, dn, dr, dv, R, q = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
        yield from ((p + ".dq", (q, W)), (p + ".dq.norm", (q,)), (p + ".uq", (H * (dn + dr), q)),
                    (p + ".dkv", (R + dr, W)), (p + ".dkv.norm", (R,)), (p + ".uk", (H * dn, R)),
                    (p + ".uv", (H * dv, R)), (p + ".sink", (H,)), (p + ".o", (W, H * dv)))
    else:
        raise ValueError(f"unknown mixer {kind!r}")


def _gated(p: str, ff: int, W: int) -> Iterator[Tuple[str, tuple]]:
    yield from ((p + ".gate", (ff, W)), (p + ".up", (ff, W)), (p + ".down", (W, ff)))


def _moe_tensors(p: str, m: dict, W: int) -> Iterator[Tuple[str, tuple]]:
    r = m["router"]
    n_out = r["experts"] + r.get("identity", 0)
    for e in range(r["experts"]):
        yield from _gated(f"{p}.e{e}", m["expert"]["ff"], W)
    yield from ((p + ".router", (n_out, W)), (p + ".correction", (n_out,)))
    if m.get("shared"):
        yield from _gated(p + ".shared", m["shared"]["ff"], W)
        yield p + ".shared.sg", (1, W)


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    """Name -> shape of every tensor of a configuration, in file order."""
    if cfg.get("architecture") not in ARCHITECTURES:
        raise ValueError(f"unknown architecture {cfg.get('architecture')!r}")
    W, V = cfg["width"], cfg["vocab"]
    out: Dict[str, tuple] = {"embed": (V, W)}
    if cfg.get("loop"):
        out["loop.step"] = (cfg["loop"]["times"], W)
    for i, l in enumerate(cfg["layers"]):
        p = f"l{i}"
        for n in (".norm1", ".norm2") if l.get("mlp") else (".norm1",):
            out[p + n] = out[p + n + ".b"] = (W,)
        out.update(_mixer_tensors(p + ".mix", l["type"], l["mixer"], W))
        if l.get("mlp"):
            out.update(_moe_tensors(p + ".mlp", l["mlp"], W))
    out["final.norm"] = out["final.norm.b"] = (W,)
    out["head"] = (V, W)
    return out


def to_bf16(a: np.ndarray) -> np.ndarray:
    """fp32 -> bf16 bits (uint16), round to nearest even."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def from_bf16(u: np.ndarray) -> np.ndarray:
    return (u.astype(np.uint32) << 16).view(np.float32)


def safetensors_image(tensors: Dict[str, np.ndarray]) -> np.ndarray:
    """The bytes of a safetensors file with every tensor in bf16 (uint16 arrays are taken as bf16 bits)."""
    head, off = {}, 0
    for k, v in tensors.items():
        n = v.size * 2
        head[k] = {"dtype": "BF16", "shape": list(v.shape), "data_offsets": [off, off + n]}
        off += n
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    img = np.empty(8 + len(h) + off, np.uint8)
    img[:8] = np.frombuffer(struct.pack("<Q", len(h)), np.uint8)
    img[8:8 + len(h)] = np.frombuffer(h, np.uint8)
    at = 8 + len(h)
    for v in tensors.values():
        b = v if v.dtype == np.uint16 else to_bf16(v)
        img[at:at + b.size * 2] = np.ascontiguousarray(b).reshape(-1).view(np.uint8)
        at += b.size * 2
    return img


def save(folder: str, cfg: dict, tensors: Dict[str, np.ndarray]) -> None:
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    safetensors_image(tensors).tofile(os.path.join(folder, "model.safetensors"))


def random_tensors(cfg: dict, seed: int = 0, only: Optional[Sequence[str]] = None) -> Dict[str, np.ndarray]:
    """Seeded random weights (bf16 bits) whose activations stay of order one: linear weights N(0, 1 / fan_in), norm
    weights around 1, A_log = log(1 .. state), dt biases that make softplus small."""
    rng = np.random.default_rng(seed)
    out: Dict[str, np.ndarray] = {}
    for k, s in tensor_shapes(cfg).items():
        if only is not None and k not in only:
            continue
        last = k.rsplit(".", 1)[-1]
        if k.endswith("norm") or last in ("norm1", "norm2", "D"):
            v = 1.0 + 0.1 * rng.standard_normal(s, np.float32)
        elif k.endswith("A_log"):
            v = np.log(np.arange(1, s[1] + 1, dtype=np.float32))[None, :] + 0.1 * rng.standard_normal(s, np.float32)
        elif k.endswith("dt.b"):
            v = -3.0 + rng.standard_normal(s, np.float32)
        elif k.endswith("conv"):
            v = rng.standard_normal(s, np.float32) * 0.5
        elif k.endswith("correction"):
            v = 0.02 * rng.standard_normal(s, np.float32)
        elif len(s) == 1 or k == "loop.step":
            v = 0.1 * rng.standard_normal(s, np.float32)
        elif k == "embed":
            v = rng.standard_normal(s, np.float32)
        else:
            v = rng.standard_normal(s, np.float32) * (1.0 / np.sqrt(s[-1]))
        out[k] = to_bf16(v)
    return out
