"""Small layer-list configurations and error measures for the layer-list model tests."""
import copy

import numpy as np

from kuiperllama_amd import checkpoint
from oracle import hybrid_ref as R


def mamba(inner=72, state=6, dt_rank=5, conv=4):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}, "mlp": None}


def latent(heads=3, dim=20, rot_dim=12, vdim=28, kv_rank=40, q_rank=36, scale=0.5, base=500.0):
    return {"type": "latent_attention", "mlp": None,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
                      "q_rank": q_rank, "scale": scale, "rot": {"base": base, "dims": rot_dim}}}


def moe(experts=5, identity=2, top=3, ff=24, shared=40):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "identity": identity, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def with_ff(layer, **kw):
    return dict(layer, mlp=moe(**kw))


def config(layers, width=88, vocab=101, eps=3e-5, cap=20.0, loop=None):
    c = {"architecture": "Gufanex", "layers": layers, "width": width, "vocab": vocab, "norm": {"eps": eps}}
    if cap is not None:
        c["logit_softcap"] = cap
    if loop is not None:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return copy.deepcopy(c)


def windowed(heads=6, kv_heads=2, dim=20, vdim=28, scale=0.3, window=11, rows=12, far=30.0):
    return {"type": "attention", "mlp": None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": window},
                      "rel_rows": rows, "bias_max": far}}


def chunked(heads=4, kv_heads=2, dim=24, vdim=18, scale=0.25, chunk=19):
    return {"type": "attention_2", "mlp": None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": chunk}}}


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def clamped(experts=7, top=2, ff=24, limit=0.8):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


def gusorax(layers, width=72, vocab=93, eps=2e-4, mult=0.45, scale=6.5, positions=700, loop=None):
    c = {"architecture": "Gusorax", "layers": layers, "width": width, "vocab": vocab, "norm": {"eps": eps}, "residual_mult": mult,
         "embedding": {"scale": scale}, "max_positions": positions}
    if loop is not None:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return copy.deepcopy(c)


def heads_mixed(**kw):
    """Both attention mixers, every feed-forward and none, a loop in the middle."""
    return gusorax([dict(windowed(), mlp=dense()), dict(chunked(), mlp=clamped()), windowed(3, 3, 9, 40, 0.5, 33, 8, 20.0),
                    dict(chunked(5, 1, 33, 7, 0.2, 40), mlp=clamped(4, 4, 10, 0.3)), dict(windowed(window=70), mlp=clamped(9, 1, 33))],
                   loop=kw.pop("loop", (1, 4, 2)), **kw)


def mixed(**kw):
    """Every mechanism and branch once: both mixers, with and without feed-forward, a loop in the middle."""
    return config([with_ff(mamba()), with_ff(latent()), mamba(40, 17, 3, 3), with_ff(latent(2, 36, 8, 16, 70, 50, 0.4), identity=0,
                                                                                    shared=0, top=2)],
                  loop=(1, 3, 3), **kw)


class Model:
    """A configuration with random weights: oracle side (fp64 forward) and the bytes the library loads."""

    def __init__(self, cfg, seed=0, edit=None):
        self.cfg = cfg
        bits = checkpoint.random_tensors(cfg, seed)
        self.W = {k: checkpoint.from_bf16(v) for k, v in bits.items()}
        # decisive routers: a close call would turn rounding into another expert
        for k in self.W:
            if k.endswith(".router"):
                self.W[k] = self.W[k] * 3.0
        if edit:
            edit(self.W)
        bits = {k: checkpoint.to_bf16(v) for k, v in self.W.items()}
        self.W = {k: checkpoint.from_bf16(v) for k, v in bits.items()}
        self.bits = bits
        self.image = checkpoint.safetensors_image(bits)

    def load(self, dtype="float32", max_seq_len=512, max_seqs=8):
        from kuiperllama_amd.model import KuiperModel
        return KuiperModel.from_tensors(self.cfg, self.image, max_seq_len=max_seq_len, dtype=dtype, max_seqs=max_seqs)

    def logits(self, tokens, residuals=None):
        return R.forward(self.W, self.cfg, tokens, residuals=residuals)

    def tokens(self, n, seed=1):
        return [int(t) for t in np.random.default_rng(seed).integers(0, self.cfg["vocab"], n)]

    def greedy(self, prompt, n):
        t = list(prompt)
        for _ in range(n):
            t.append(int(np.argmax(self.logits(t)[-1])))
        return t[len(prompt):]


def errors(got, want):
    """RMS difference per row relative to the spread of the wanted logits."""
    d = np.asarray(got, np.float64) - want
    return np.sqrt((d * d).mean(axis=-1)) / want.std()


def check(got, want, dtype, what=""):
    e = errors(got, want)
    if dtype == "float32":
        assert e.max() < 5e-5, (what, e.max(), int(e.argmax()))
    else:  # rounding may turn a router's close call at a few positions
        assert np.quantile(e, 0.85) < 0.03, (what, np.quantile(e, 0.85), e.max())
        assert e.max() < 0.6, (what, e.max())


def run_alone(m, toks, cuts=()):
    """Logits of every token of one sequence, fed in portions that end at `cuts`."""
    s = m.open_seq()
    out, at = [], 0
    for end in list(cuts) + [len(toks)]:
        if end > at:
            out.append(m.forward([(s, toks[at:end], list(range(end - at)))]))
            at = end
    m.close_seq(s)
    return np.concatenate(out)
