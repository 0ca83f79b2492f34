"""Small random Zivitar checkpoints for the tests: config dicts, bf16 weights with the checkpoint's tensor names, a folder on
disk for the loader.  Sizes are deliberately unequal (heads != kv_heads, dim != vdim, rot.dims < dim, short windows, different
feed-forward sizes per layer, borrowed tensors with a window and decays of the borrowing layer's own) so that a swapped size shows."""
from __future__ import annotations

import torch

from tests.garesun_helpers import rel_rms, write_checkpoint  # noqa: F401


def dense(ff=40, limit=1.5):
    return dict(kind="dense", ff=ff, limit=limit)


def _mlp(mlp):
    return dense() if mlp == "dense" else mlp


def lightning(heads=3, dim=10, vdim=14, decay=None, mlp="dense", weights_of=None):
    d = dict(type="lightning", mixer=dict(heads=heads, dim=dim, vdim=vdim, decay=decay or [0.5 + 0.49 * (h + 1) / heads for h in range(heads)]),
             mlp=_mlp(mlp))
    if weights_of is not None:
        d["weights_of"] = weights_of
    return d


YARN = dict(factor=3.0, original=64, fast=16.0, slow=0.7)


def attention(heads=4, kv_heads=2, dim=12, vdim=20, scale=0.3, diff=0.4, conv=3, size=9, keep=2, rot_dims=8, base=50.0, scaling=YARN, mlp="dense",
              weights_of=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, diff=diff, conv=conv)
    if size:
        m["mask"] = dict(size=size, keep_first=keep)
    if rot_dims:
        m["rot"] = dict(base=base, dims=rot_dims)
        if scaling:
            m["rot"]["scaling"] = dict(scaling)
    d = dict(type="attention", mixer=m, mlp=_mlp(mlp))
    if weights_of is not None:
        d["weights_of"] = weights_of
    return d


def config(layers, vocab=101, width=56, eps=1e-5, streams=3, logit_scale=0.8, cap=6.0):
    cfg = dict(architecture="Zivitar", vocab=vocab, width=width, layers=layers, norm=dict(eps=eps), streams=streams, logit_scale=logit_scale)
    if cap:
        cfg["logit_softcap"] = cap
    return cfg


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W, width, S = {}, cfg["width"], cfg["streams"]

    def lin(name, out, inn, s=1.0):
        W[name] = (torch.randn(out, inn, generator=g) * (s / inn ** 0.5)).to(torch.bfloat16)

    def vec(name, n, center=0.0, s=0.2):
        W[name] = (center + s * torch.randn(n, generator=g)).to(torch.bfloat16)

    def hyper(p):
        vec(p + "in", S, 1.0 / S, 0.2)
        vec(p + "out", S, 0.8, 0.3)
        W[p + "mix"] = (torch.eye(S) + 0.3 * torch.randn(S, S, generator=g)).to(torch.bfloat16)

    W["embed"] = torch.randn(cfg["vocab"], width, generator=g).to(torch.bfloat16)
    for i, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        p, m = f"l{i}.", L["mixer"]
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        vec(p + "norm1", width, 1.0, 0.2)
        hyper(p + "hc1.")
        if L["type"] == "lightning":
            for n, rows in (("q", H * D), ("k", H * D), ("v", H * Dv), ("g", H * Dv)):
                lin(p + "mix." + n, rows, width, 2.0)
            vec(p + "mix.norm", H * Dv, 1.0, 0.3)
        else:
            for n, rows in (("q", H * 2 * D), ("k", m["kv_heads"] * 2 * D), ("v", m["kv_heads"] * Dv)):
                lin(p + "mix." + n, rows, width, 2.0)
                if m["conv"]:
                    W[p + f"mix.{n}.conv"] = (0.6 * torch.randn(rows, m["conv"], generator=g)).to(torch.bfloat16)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                vec(p + "mix." + n, D, 0.0, 0.3)
        lin(p + "mix.o", width, H * Dv, 1.5)
        if L.get("mlp"):
            ff = L["mlp"]["ff"]
            vec(p + "norm2", width, 1.0, 0.2)
            hyper(p + "hc2.")
            lin(p + "mlp.gate", ff, width, 2.0)
            lin(p + "mlp.up", ff, width, 2.0)
            lin(p + "mlp.down", width, ff, 1.5)
    vec("final.norm", width, 1.0, 0.2)
    lin("head", cfg["vocab"], width, 2.0)
    return W


def as_f64(W):
    return {k: v.to(torch.float64) for k, v in W.items()}


def mixed_layers():
    """both mixers with and without a feed-forward, a window longer than a page, no window, kept tokens that reach over a page's
    tiles and none, kv_heads = heads and = 1, full, partial and no rotation with and without scaled frequencies, one tap and none,
    tensors borrowed from an earlier and from a later layer with a window / decays / rotation of the borrowing layer's own"""
    return [lightning(),
            attention(),
            attention(heads=2, kv_heads=2, dim=8, vdim=8, size=70, keep=18, conv=4, rot_dims=8, base=1000.0, scaling=None, mlp=dense(24, 0.7)),
            lightning(decay=[0.9, 0.3, 0.99], weights_of=0),
            attention(size=5, keep=0, diff=0.7, scale=0.2, weights_of=1),
            attention(heads=3, kv_heads=1, dim=6, vdim=33, size=0, conv=1, rot_dims=0, mlp=None, weights_of=6),
            attention(heads=3, kv_heads=1, dim=6, vdim=33, size=30, keep=1, conv=1, rot_dims=2, base=9.0, scaling=None, mlp=None),
            lightning(heads=1, dim=40, vdim=8, mlp=None)]


def mixed_config(**kw):
    return config(mixed_layers(), **kw)
