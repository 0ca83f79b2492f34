"""Small random Rorovik checkpoints for the tests: config dicts, bf16 weights with the checkpoint's tensor names, a folder on disk
for the loader.  Sizes are deliberately unequal (heads != kv_heads, dim != vdim != rot_dim, q_rank != kv_rank, short windows, one or several
identity experts, different feed-forwards per layer) so that a swapped size shows."""
from __future__ import annotations

import torch

from tests.garesun_helpers import rel_rms, write_checkpoint  # noqa: F401

YARN = dict(factor=3.0, original=64, fast=16.0, slow=0.7)


def dense(ff=40):
    return dict(kind="dense", ff=ff)


def moe(experts=5, identity=1, top=2, ff=16, limit=1.2):
    r = dict(experts=experts, top=top)
    if identity:
        r["identity"] = identity
    e = dict(ff=ff)
    if limit is not None:
        e["limit"] = limit
    return dict(kind="moe", expert=e, router=r)


def attention(heads=4, kv_heads=2, dim=12, vdim=20, scale=0.3, window=9, coef=0.3, every=6, v_mix=True, mlp="dense"):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if window:
        m["mask"] = dict(size=window)
    if every:
        m["q_temp"] = dict(coef=coef, every=every)
    if v_mix:
        m["v_mix"] = True
    return dict(type="attention", mixer=m, mlp=dense() if mlp == "dense" else mlp)


def latent(heads=3, dim=14, rot_dim=8, vdim=10, kv_rank=40, q_rank=24, scale=0.25, base=500.0, scaling=YARN, mlp="moe"):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale)
    if rot_dim:
        m["rot"] = dict(base=base, dims=rot_dim)
        if scaling:
            m["rot"]["scaling"] = dict(scaling)
    return dict(type="latent_attention", mixer=m, mlp=moe() if mlp == "moe" else (dense() if mlp == "dense" else mlp))


def config(layers, vocab=101, width=56, eps=1e-5, mult=0.6, side=12):
    cfg = dict(architecture="Rorovik", vocab=vocab, width=width, layers=layers, norm=dict(eps=eps), residual_mult=mult)
    if side:
        cfg["token_side"] = dict(dim=side)
    return cfg


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W, width = {}, cfg["width"]
    side = (cfg.get("token_side") or {}).get("dim", 0)

    def lin(name, out, inn, s=1.0):
        W[name] = (torch.randn(out, inn, generator=g) * (s / inn ** 0.5)).to(torch.bfloat16)

    def vec(name, n, center=0.0, s=0.2):
        W[name] = (center + s * torch.randn(n, generator=g)).to(torch.bfloat16)

    W["embed"] = torch.randn(cfg["vocab"], width, generator=g).to(torch.bfloat16)
    vec("embed.norm", width, 1.0)
    if side:
        W["side.embed"] = torch.randn(cfg["vocab"], side * len(cfg["layers"]), generator=g).to(torch.bfloat16)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        for n in ("norm1", "norm1b"):
            vec(p + n, width, 1.0)
        vec(p + "mix.sink", H, 0.5, 1.0)
        if L["type"] == "attention":
            G = m["kv_heads"]
            for n, r in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                lin(p + "mix." + n, r, width, 2.0)
                vec(p + f"mix.{n}.b", r, 0.0, 0.5)
            vec(p + "mix.q.norm", H * D, 1.0, 0.3)
            vec(p + "mix.k.norm", G * D, 1.0, 0.3)
            lin(p + "mix.g", H, width, 3.0)
            if m.get("v_mix"):
                W[p + "mix.vmix"] = (0.2 + 0.6 * torch.rand((), generator=g)).to(torch.bfloat16)
        else:
            Dr, R, Rq = m["rot_dim"], m["kv_rank"], m["q_rank"]
            lin(p + "mix.dq", Rq, width, 2.0)
            vec(p + "mix.dq.norm", Rq, 1.0, 0.3)
            lin(p + "mix.uq", H * (D + Dr), Rq, 1.5)
            lin(p + "mix.dkv", R + Dr, width, 1.5)
            vec(p + "mix.dkv.norm", R, 1.0, 0.3)
            lin(p + "mix.uk", H * D, R, 1.5)
            lin(p + "mix.uv", H * Dv, R, 1.5)
        lin(p + "mix.o", width, H * Dv)
        ml = L.get("mlp")
        if ml:
            for n in ("norm2", "norm2b"):
                vec(p + n, width, 1.0)
            if ml["kind"] == "moe":
                E, ff = ml["router"]["experts"], ml["expert"]["ff"]
                cols = E + ml["router"].get("identity", 0)
                lin(p + "mlp.router", cols, width, 4.0)                  # spread logits: few near ties between experts
                vec(p + "mlp.correction", cols, 0.0, 0.1)
                for e in range(E):
                    lin(p + f"mlp.e{e}.gate", ff, width, 1.5)
                    lin(p + f"mlp.e{e}.up", ff, width, 1.5)
                    lin(p + f"mlp.e{e}.down", width, ff)
            else:
                for n, r, k in (("gate", ml["ff"], width), ("up", ml["ff"], width), ("down", width, ml["ff"])):
                    lin(p + "mlp." + n, r, k, 1.5)
                    vec(p + f"mlp.{n}.b", r, 0.0, 0.4)
        if side:
            lin(p + "side.gate", side, width, 1.5)
            lin(p + "side.proj", width, side)
            vec(p + "side.norm", width, 1.0)
    vec("final.norm", width, 1.0)
    lin("head", cfg["vocab"], width, 2.0)
    return W


def mixed_layers():
    """both mixers with both feed-forwards and none, a window longer than a page and none at all, a layer that mixes no values before the
    first that does and between those that do, every expert chosen, several identity experts and none, no limit, kv_heads = heads and = 1, scaled
    and plain frequencies, one rotated pair"""
    mix = dict(kv_heads=2, vdim=20)
    return [attention(heads=6, kv_heads=1, dim=10, vdim=16, window=5, v_mix=False, every=None),
            latent(),
            attention(**mix, mlp=moe(experts=3, identity=2, top=3)),
            latent(heads=2, dim=8, rot_dim=16, vdim=8, kv_rank=24, q_rank=40, scaling=None, mlp="dense"),
            attention(heads=2, dim=24, window=70, every=64, **mix),
            attention(heads=3, kv_heads=3, dim=8, vdim=33, window=0, v_mix=False, mlp=moe(experts=4, identity=0, top=4, limit=None)),
            attention(heads=8, dim=5, window=12, every=1, coef=0.1, mlp=None, **mix),
            latent(heads=5, dim=8, rot_dim=2, vdim=24, kv_rank=16, q_rank=9, mlp=None)]


def mixed_config(**kw):
    return config(mixed_layers(), **kw)
