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

ARCHITECTURES = ("Gufanex", "Gusorax")


DISTANCE_ROWS = 32  # rows of a distance table that a configuration does not size (the loader reads them off the tensor)


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
    elif kind in ("attention", "attention_2"):
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        biased = kind == "attention_2"
        for n, rows in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
            yield f"{p}.{n}", (rows, W)
            if biased:
                yield f"{p}.{n}.b", (rows,)
        yield from ((p + ".q.norm", (dk,)), (p + ".k.norm", (dk,)))
        yield (p + ".g", (H * dv, W)) if biased else (p + ".rel", (m.get("rel_rows", DISTANCE_ROWS), H))
        yield p + ".o", (W, H * dv)
        if biased:
            yield p + ".o.b", (W,)
    else:
        raise ValueError(f"unknown mixer {kind!r}")


def _gated(p: str, ff: int, W: int) -> Iterator[Tuple[str, tuple]]:
    yield from ((p + ".gate", (ff, W)), (p + ".up", (ff, W)), (p + ".down", (W, ff)))


def _moe_tensors(p: str, m: dict, W: int, correction: bool = True) -> Iterator[Tuple[str, tuple]]:
    if m["kind"] == "dense":
        yield from _gated(p, m["ff"], W)
        return
    r = m["router"]
    n_out = r["experts"] + r.get("identity", 0)
    for e in range(r["experts"]):
        yield from _gated(f"{p}.e{e}", m["expert"]["ff"], W)
    yield p + ".router", (n_out, W)
    if correction:
        yield p + ".correction", (n_out,)
    if m.get("shared"):
        yield from _gated(p + ".shared", m["shared"]["ff"], W)
        yield p + ".shared.sg", (1, W)


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    """Name -> shape of every tensor of a configuration, in file order."""
    if cfg.get("architecture") not in ARCHITECTURES:
        raise ValueError(f"unknown architecture {cfg.get('architecture')!r}")
    W, V = cfg["width"], cfg["vocab"]
    gufanex = cfg["architecture"] == "Gufanex"  # else: one RMS norm per layer, positions, a matrix into the loop
    out: Dict[str, tuple] = {"embed": (V, W)}
    if not gufanex:
        out["pos"] = (cfg["max_positions"], W)
    if cfg.get("loop"):
        out.update({"loop.step": (cfg["loop"]["times"], W)} if gufanex else {"loop.in": (W, 2 * W)})

    def norm(name):
        out[name] = (W,)
        if gufanex:
            out[name + ".b"] = (W,)

    for i, l in enumerate(cfg["layers"]):
        p = f"l{i}"
        norm(p + ".norm1")
        if l.get("mlp") and gufanex:
            norm(p + ".norm2")
        out.update(_mixer_tensors(p + ".mix", l["type"], l["mixer"], W))
        if l.get("mlp"):
            out.update(_moe_tensors(p + ".mlp", l["mlp"], W, gufanex))
    norm("final.norm")
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
    weights around 1 (around 0 where the norm adds one), A_log = log(1 .. state), dt biases that make softplus small,
    embeddings that the configuration's scale brings to order one."""
    one_plus = cfg["architecture"] != "Gufanex"
    rng = np.random.default_rng(seed)
    out: Dict[str, np.ndarray] = {}
    for k, s in tensor_shapes(cfg).items():
        if only is not None and k not in only:
            continue
        last = k.rsplit(".", 1)[-1]
        if one_plus and (last == "norm1" or k == "final.norm"):
            v = 0.1 * rng.standard_normal(s, np.float32)
        elif k == "pos":
            v = 0.3 * rng.standard_normal(s, np.float32)
        elif k.endswith(".rel"):
            v = rng.standard_normal(s, np.float32)
        elif k.endswith("norm") or last in ("norm1", "norm2", "D"):
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
            v = rng.standard_normal(s, np.float32) / float(cfg.get("embedding", {}).get("scale", 1.0))
        else:
            v = rng.standard_normal(s, np.float32) * (1.0 / np.sqrt(s[-1]))
        out[k] = to_bf16(v)
    return out
