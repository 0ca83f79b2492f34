"""Host side of the Zivitar model package (no GPU): config parsing, its defaults and refusals, the rotation table, borrowed
tensors, the registry lookup by config.json, weight loading with its shape checks and the per-layer caches / states / carried
inputs on the CPU device, and the plain oracle against itself (causality, the window's edge and the kept tokens, the
convolution's reach, the difference of the maps, the streams' mix)."""
import copy
import math

import numpy as np
import pytest
import torch

from tests import zivitar_helpers as H
from tests import zivitar_oracle as O

F64 = torch.float64


def test_config_reads_every_size_and_refuses_what_the_design_does_not_have():
    from mlx_vlm_amd.models.zivitar import ModelConfig

    cfg = H.mixed_config(vocab=123, width=56, eps=3e-4, streams=4, logit_scale=0.25, cap=9.0)
    mc = ModelConfig.from_dict(cfg)
    assert (mc.vocab, mc.width, mc.norm_eps, mc.streams, mc.logit_scale, mc.logit_softcap, len(mc.layers)) == (123, 56, 3e-4, 4, 0.25, 9.0, 8)
    assert mc.layers[1].window == (9, 2) and mc.layers[4].window == (5, 0) and mc.layers[5].window == (0, 0)
    assert mc.layers[1].taps == 3 and mc.layers[2].ff == 24 and mc.layers[2].limit == 0.7 and mc.layers[5].ff == 0
    assert [L.weights_of for L in mc.layers] == [None, None, None, 0, 1, 6, None, None]
    chain = copy.deepcopy(cfg)
    chain["layers"].append(H.lightning(weights_of=3))                             # a source that borrows itself
    assert ModelConfig.from_dict(chain).layers[8].weights_of == 0
    plain = H.config([H.attention(rot_dims=0, size=0, conv=0, mlp=dict(ff=16)), H.lightning(dim=8, vdim=8)], cap=0.0)
    del plain["streams"], plain["logit_scale"], plain["layers"][0]["mixer"]["vdim"], plain["layers"][1]["mixer"]["vdim"]
    mp = ModelConfig.from_dict(plain)                                             # what a config leaves out
    assert (mp.streams, mp.logit_scale, mp.logit_softcap) == (0, 1.0, 0.0) and mp.layers[0].limit == math.inf and mp.layers[0].mixer["vdim"] == 12
    assert mp.layers[1].mixer["vdim"] == 8 and mp.layers[0].taps == 0
    for layers in ([dict(H.lightning(), type="convolution")], [H.attention(heads=5, kv_heads=2)], [H.attention(rot_dims=5)],
                   [H.attention(rot_dims=14)], [H.attention(size=-3)], [H.attention(keep=-1)], [H.attention(conv=17)], [H.attention(vdim=300)],
                   [H.lightning(heads=2, decay=[0.5])], [H.lightning(mlp=dict(kind="moe", ff=8))], [H.lightning(mlp=dict(kind="dense"))],
                   [H.lightning(mlp=H.dense(limit=-1.0))], [H.lightning(weights_of=0)], [H.lightning(weights_of=4)],
                   [H.lightning(), H.lightning(dim=11, weights_of=0)], [H.lightning(), H.attention(weights_of=0)],
                   [H.attention(), H.attention(conv=2, weights_of=0)], [H.lightning(weights_of=1), H.lightning(weights_of=0)],
                   [H.attention(scaling=dict(factor=2.0))]):
        with pytest.raises(ValueError):
            ModelConfig.from_dict(H.config(layers))
    for streams in (-1, 9):
        with pytest.raises(ValueError):
            ModelConfig.from_dict(H.config([H.lightning()], streams=streams))


@pytest.mark.parametrize("dims,base,scaling", [(8, 50.0, H.YARN), (16, 10000.0, dict(factor=4.0, original=4096, fast=20.0, slow=2.0)),
                                               (64, 500000.0, dict(factor=1.0, original=128, fast=32.0, slow=1.0)),
                                               (2, 10.0, dict(factor=8.0, original=1024, fast=8.0, slow=4.0)), (6, 7.0, None), (0, 7.0, None)])
def test_rotation_table(dims, base, scaling):
    from mlx_vlm_amd.models.zivitar.config import rotation

    rot = dict(base=base, dims=dims)
    if scaling:
        rot["scaling"] = scaling
    n, f, amp = rotation(rot)
    assert n == dims
    if not dims:
        assert f is None and amp == 1.0
        return
    want, wamp = O.rotation_table(rot)
    assert f.dtype == np.float32 and np.allclose(f, want.numpy(), rtol=1e-6, atol=0) and abs(amp - wamp) < 1e-12
    if scaling and dims == 8:                # slow pairs are stretched, fast ones kept
        plain = [base ** (-2 * i / dims) for i in range(dims // 2)]
        assert f[0] < plain[0] * 1.0001 and abs(f[-1] - plain[-1] / 3.0) < 1e-6 and abs(amp - (1 + 0.1 * math.log(3.0))) < 1e-12


def test_registry_finds_the_package_by_architecture():
    from mlx_vlm_amd.utils import get_model_and_args

    arch, name = get_model_and_args({"architecture": "Zivitar"})
    assert name == "zivitar" and hasattr(arch, "Model") and hasattr(arch, "ModelConfig") and "diff_attn" in arch.HIP_SOURCES


def test_weights_load_on_the_cpu_device_with_shape_checks_and_state_per_layer():
    from mlx_vlm_amd.models.cache import PAGE
    from mlx_vlm_amd.models.zivitar import LanguageModel, ModelConfig

    cfg = H.mixed_config()
    W = H.weights(cfg, seed=3)
    for dtype, T in (("bfloat16", torch.bfloat16), ("float32", torch.float32)):
        lm = LanguageModel(ModelConfig.from_dict(copy.deepcopy(cfg)), device="cpu", dtype=dtype, kv_pool_tokens=5 * PAGE, max_seqs=3)
        lm.load_weights(dict(W, unused=torch.zeros(3)))                           # a tensor nobody asks for is left alone
        pool = lm.pool
        assert sorted(pool.rows) == sorted((r, n) for r in (1, 2, 4, 5, 6) for n in "kv")
        # keys: two maps per head, fp32 or two bf16 planes padded to 8
        split = T == torch.bfloat16
        assert pool.rows[(1, "k")].dtype == T and pool.rows[(1, "v")].dtype == T
        assert pool.rows[(1, "k")].shape == (5, PAGE, 2 * 2 * (2 * 16 if split else 12)) and pool.rows[(6, "k")].shape == (5, PAGE, 2 * 2 * 8 if split else 12)
        assert pool.rows[(4, "v")].shape == (5, PAGE, 2 * 20)
        assert sorted(pool.state) == [0, 3, 7] and pool.state[0].shape == (3, 3, 10, 14) and all(t.dtype == torch.float32 for t in pool.state.values())
        # packed projection rows: 4 * 2 * 12 | 2 * 2 * 12 | 2 * 20 ; carried: taps - 1 of them per sequence (none for one tap)
        assert sorted(pool.aux) == [(1, "conv"), (2, "conv"), (4, "conv")] and pool.aux[(1, "conv")].shape == (3, 2, 96 + 48 + 40)
        L0, L1, L3, L4, L5 = (lm._L[i] for i in (0, 1, 3, 4, 5))
        assert L3.wproj is L0.wproj and L3.decay.tolist() != L0.decay.tolist() and L4.wproj is L1.wproj and (L4.window, L4.keep) == (5, 0)
        assert L5.wproj is lm._L[6].wproj and L5.window == 0 and L5.inv_freq is None and lm._L[6].rot_dims == 2
        assert torch.equal(L1.wproj[L1.off["k"]: L1.off["k"] + 48], W["l1.mix.k"].to(T)) and torch.equal(L1.conv[L1.off["v"]: L1.off["v"] + 40], W["l1.mix.v.conv"].to(T))
        w = H.as_f64(W)
        lam = O.lambda_of(*(w["l1.mix." + n] for n in ("lq1", "lk1", "lq2", "lk2")), 0.4)
        assert abs(L1.lam - lam) < 1e-9 and abs(L4.lam - (lam + 0.3)) < 1e-9
        assert L0.hc1.mix.dtype == torch.float32 and torch.equal(L0.hc1.mix, W["l0.hc1.mix"].float())
        assert len(lm.make_cache()) == 8 and not lm.make_cache()[1].is_trimmable()
    short = dict(W)
    short["l1.mix.k.conv"] = short["l1.mix.k.conv"][:, :-1]
    with pytest.raises(ValueError):
        LanguageModel(ModelConfig.from_dict(copy.deepcopy(cfg)), device="cpu").load_weights(short)
    missing = {k: v for k, v in W.items() if k != "l0.hc2.mix"}
    with pytest.raises(KeyError):
        LanguageModel(ModelConfig.from_dict(copy.deepcopy(cfg)), device="cpu").load_weights(missing)


def test_oracle_is_causal_windowed_and_keeps_the_first_tokens_in_view():
    cfg = H.mixed_config()
    W = H.as_f64(H.weights(cfg, seed=9))
    ids = np.arange(60) % cfg["vocab"]
    a, _ = O.forward(cfg, W, ids)
    ids2 = ids.copy()
    ids2[40:] = (ids2[40:] + 7) % cfg["vocab"]
    b, _ = O.forward(cfg, W, ids2)
    assert torch.allclose(a[:40], b[:40], rtol=0, atol=1e-11) and not torch.allclose(a[40:], b[40:])
    # one attention layer, window 4, two kept tokens, 3 taps: token 10 reaches the keys of 10..12, seen by rows up to 15; token 1
    # reaches the key of the kept token 1 (and of 2, 3, which are not kept), so every later row knows it
    one = H.config([H.attention(size=4, keep=2, mlp=None)])
    W1 = H.as_f64(H.weights(one, seed=2))
    x, _ = O.forward(one, W1, ids)
    for tok, rows in ((10, list(range(10, 16))), (1, list(range(1, 60))), (2, [2, 3, 4, 5, 6, 7])):
        ids3 = ids.copy()
        ids3[tok] = (ids3[tok] + 1) % one["vocab"]
        y, _ = O.forward(one, W1, ids3)
        assert [t for t in range(60) if not torch.allclose(x[t], y[t], rtol=0, atol=1e-11)] == rows, tok
    seen = O.visible(12, 3, 2)
    assert seen[9].nonzero().flatten().tolist() == [0, 1, 7, 8, 9] and seen[1].nonzero().flatten().tolist() == [0, 1]
    # rotation: the pair of dimension i is i + dims / 2; the rest passes
    v = torch.zeros(3, 1, 6, dtype=F64)
    v[..., 0], v[..., 5] = 1.0, 2.0
    r = O.rotate_half(v, dict(dims=4, base=100.0))[:, 0]
    ang = torch.tensor([0.0, 1.0, 2.0], dtype=F64)
    assert torch.allclose(r[:, 0], torch.cos(ang)) and torch.allclose(r[:, 2], torch.sin(ang)) and torch.equal(r[:, 4:], v[:, 0, 4:]) and torch.all(r[:, 1] == 0)
    # the streams: mix is indexed [from, to]
    X = torch.tensor([[[1.0]], [[10.0]]], dtype=F64)
    n = O.hyper_write(X, torch.tensor([[100.0]], dtype=F64), torch.tensor([[1.0, 2.0], [3.0, 4.0]], dtype=F64), torch.tensor([1.0, 0.0], dtype=F64))
    assert n.flatten().tolist() == [131.0, 42.0] and float(O.hyper_read(X, torch.tensor([2.0, 0.5], dtype=F64))) == 7.0
    g, u = torch.tensor([5.0, -4.0], dtype=F64), torch.tensor([-9.0, 0.5], dtype=F64)
    c = O.clamped_glu(g, u, 2.0)                                      # the gate is cut from above only, the linear part on both sides
    assert torch.allclose(c, torch.stack([2.0 * torch.sigmoid(torch.tensor(3.404, dtype=F64)) * -1.0, -4.0 * torch.sigmoid(torch.tensor(-6.808, dtype=F64)) * 1.5]))
