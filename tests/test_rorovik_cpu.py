"""Host side of the Rorovik model package (no GPU): config parsing, its defaults and refusals, the registry lookup by config.json, weight
loading with its shape checks and the per-layer caches on the CPU device, and the plain oracle against itself (causality, the window's
reach, the distance bias, the sink, the mixed values, the rotation, the router)."""
import copy
import math

import numpy as np
import pytest
import torch

from tests import rorovik_helpers as H
from tests import rorovik_oracle as O

F64 = torch.float64


def test_config_reads_every_size_and_refuses_what_the_design_does_not_have():
    from mlx_vlm_amd.models.rorovik import ModelConfig

    mc = ModelConfig.from_dict(H.mixed_config(vocab=123, width=56, eps=3e-4, mult=0.45, side=7))
    assert (mc.vocab, mc.width, mc.norm_eps, mc.residual_mult, mc.side_dim, mc.v_first, len(mc.layers)) == (123, 56, 3e-4, 0.45, 7, 2, 8)
    assert [L.window for L in mc.layers] == [5, 0, 9, 0, 70, 0, 12, 0] and [L.v_mix for L in mc.layers] == [False, False, True, False, True, False, True, False]
    assert [L.moe for L in mc.layers] == [False, True, True, False, False, True, False, False] and [L.ff for L in mc.layers] == [40, 16, 16, 40, 40, 16, 0, 0]
    assert mc.layers[1].router == (5, 1, 2) and mc.layers[2].router == (3, 2, 3) and mc.layers[5].router == (4, 0, 4)
    assert mc.layers[1].limit == 1.2 and mc.layers[5].limit == math.inf
    plain = H.config([H.attention(window=0, every=None, v_mix=False, mlp=dict(ff=16)), H.latent(scaling=None)], side=0)
    del plain["residual_mult"], plain["layers"][0]["mixer"]["kv_heads"], plain["layers"][0]["mixer"]["vdim"], plain["layers"][1]["mixer"]["rot"]["dims"]
    mp = ModelConfig.from_dict(plain)                                             # what a config leaves out
    assert (mp.residual_mult, mp.side_dim, mp.v_first) == (1.0, 0, None) and mp.layers[0].mixer["kv_heads"] == 4 and mp.layers[0].mixer["vdim"] == 12
    assert not mp.layers[0].moe and mp.layers[1].mixer["rot"]["dims"] == 8
    ModelConfig.from_dict(H.config([dict(H.latent(mlp=None), mlp=None)]))
    no_scale = H.attention()
    del no_scale["mixer"]["scale"]
    for layers in ([dict(H.latent(), type="lightning")], [H.attention(heads=5, kv_heads=2)], [H.attention(window=-3)], [H.attention(every=-1)], [H.attention(vdim=300)], [H.attention(dim=800)],
                   [no_scale], [H.latent(rot_dim=5)], [dict(H.latent(), mixer=dict(H.latent()["mixer"], rot=dict(base=5.0, dims=4)))],
                   [dict(H.latent(), mixer={k: v for k, v in H.latent()["mixer"].items() if k != "rot"})], [H.latent(scaling=dict(factor=2.0))],
                   [H.latent(kv_rank=1100)], [H.latent(q_rank=0)], [H.latent(mlp=H.moe(experts=2, identity=1, top=4))], [H.latent(mlp=H.moe(experts=0, identity=3))],
                   [H.latent(mlp=H.moe(experts=250, identity=7))], [H.latent(mlp=H.moe(limit=-1.0))], [H.latent(mlp=dict(kind="glu", ff=8))],
                   [H.latent(mlp=dict(kind="dense"))], [H.attention(vdim=20), H.attention(vdim=16)], [H.attention(kv_heads=2), H.attention(kv_heads=4)]):
        with pytest.raises(ValueError):
            ModelConfig.from_dict(H.config(layers))


def test_registry_finds_the_package_by_architecture():
    from mlx_vlm_amd.utils import get_model_and_args

    arch, name = get_model_and_args({"architecture": "Rorovik"})
    assert name == "rorovik" and hasattr(arch, "Model") and hasattr(arch, "ModelConfig") and "grouped_attn" in arch.HIP_SOURCES


def test_weights_load_on_the_cpu_device_with_shape_checks_and_caches_per_layer():
    from mlx_vlm_amd.models.cache import PAGE
    from mlx_vlm_amd.models.rorovik import LanguageModel, ModelConfig

    cfg = H.mixed_config()
    W = H.weights(cfg, seed=3)
    make = lambda dtype="bfloat16": LanguageModel(ModelConfig.from_dict(copy.deepcopy(cfg)), device="cpu", dtype=dtype, kv_pool_tokens=5 * PAGE, max_seqs=3)  # noqa: E731
    for dtype, T in (("bfloat16", torch.bfloat16), ("float32", torch.float32)):
        lm = make(dtype)
        lm.load_weights(dict(W, unused=torch.zeros(3)))                           # a tensor nobody asks for is left alone
        pool = lm.pool
        assert sorted(pool.rows, key=str) == sorted([(i, n) for i in (0, 2, 4, 5, 6) for n in "kv"] + [(i, "c") for i in (1, 3, 7)], key=str)
        split = T == torch.bfloat16
        assert pool.rows[(2, "k")].shape == (5, PAGE, 2 * 2 * 16 if split else 2 * 12) and pool.rows[(2, "v")].shape == (5, PAGE, 40)
        assert pool.rows[(1, "c")].shape == (5, PAGE, 48) and pool.rows[(1, "c")].dtype == T and not pool.state and not pool.aux
        L1, L2, L4 = lm._L[1], lm._L[2], lm._L[4]
        assert L2.vother is None and L4.vother == 2 and L4.mix == float(W["l4.mix.vmix"].float()) and lm._L[5].vother is None
        assert L2.slope.tolist() == [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8] and L2.sink.dtype == torch.float32
        assert torch.equal(L2.wproj[L2.off["k"]: L2.off["k"] + 24], W["l2.mix.k"].to(T)) and torch.equal(L1.wproj[L1.off["dkv"]: L1.off["dkv"] + 48], W["l1.mix.dkv"].to(T))
        assert torch.equal(L1.wff[2 * 16: 3 * 16], W["l1.mlp.e1.gate"].to(T)) and torch.equal(L1.down[:, 16:32], W["l1.mlp.e1.down"].to(T))
        assert torch.equal(L1.corr, W["l1.mlp.correction"].float()) and abs(L1.amp - (1 + 0.1 * math.log(3.0))) < 1e-12 and lm._L[3].amp == 1.0
        assert len(lm.make_cache()) == 8 and lm.make_cache()[1].is_trimmable() and not lm.STATEFUL
    for name in ("l0.norm1b", "l2.mix.vmix", "l4.mix.vmix", "l1.mlp.correction", "l0.mlp.down.b", "l3.side.norm", "side.embed", "embed.norm"):
        if name == "l2.mix.vmix":                                                 # the first mixing layer's weight is not used
            make().load_weights({k: v for k, v in W.items() if k != name})
            continue
        with pytest.raises(KeyError):
            make().load_weights({k: v for k, v in W.items() if k != name})
    for name in ("l1.mix.uq", "l2.mix.q.norm", "l1.mlp.router", "side.embed"):
        with pytest.raises(ValueError):
            make().load_weights(dict(W, **{name: W[name][:-1]}))


def test_oracle_is_causal_and_windowed_and_its_mechanisms_do_what_they_say():
    cfg = H.mixed_config()
    orc = O.Oracle(cfg, H.weights(cfg, seed=9), F64)
    ids = np.arange(60) % cfg["vocab"]
    a = orc.forward(ids)
    ids2 = ids.copy()
    ids2[40:] = (ids2[40:] + 7) % cfg["vocab"]
    b = orc.forward(ids2)
    assert torch.allclose(a[:40], b[:40], rtol=0, atol=1e-11) and not torch.allclose(a[40:], b[40:])
    one = H.config([H.attention(window=4, mlp=None)])
    o1 = O.Oracle(one, H.weights(one, seed=2), F64)
    x = o1.forward(ids)
    ids3 = ids.copy()
    ids3[10] = 77
    y = o1.forward(ids3)
    assert [t for t in range(60) if not torch.allclose(x[t], y[t], rtol=0, atol=1e-11)] == [10, 11, 12, 13]
    # a sink takes its share once; a bias by distance is not the same as one by the key's position once there is a sink
    s = torch.tensor([[[0.0, 0.0], [1.0, 2.0]]], dtype=F64)
    w = O.sink_softmax(s, O.visible(2), torch.tensor([0.5], dtype=F64))[0]
    assert abs(float(w[0, 0]) - 1 / (1 + math.exp(0.5))) < 1e-12 and w[0, 1] == 0
    assert abs(float(w[1, 1]) - math.exp(2) / (math.exp(0.5) + math.exp(1) + math.exp(2))) < 1e-12
    assert O.slopes(4, F64).tolist() == [0.25, 0.0625, 0.015625, 0.00390625] and abs(float(O.slopes(6, F64)[0]) - 2 ** (-8 / 6)) < 1e-15
    t = O.temperature(12, dict(coef=0.5, every=4), F64)
    assert t[:3].tolist() == [1.0] * 3 and abs(float(t[3]) - (1 + 0.5 * math.log(2))) < 1e-12 and abs(float(t[11]) - (1 + 0.5 * math.log(4))) < 1e-12
    # neighbours are paired; both components grow by the factor
    v = torch.zeros(3, 1, 4, dtype=F64)
    v[..., 0], v[..., 3] = 1.0, 2.0
    r = O.rotate_pairs(v, dict(dims=4, base=100.0))[:, 0]
    ang = torch.tensor([0.0, 1.0, 2.0], dtype=F64)
    assert torch.allclose(r[:, 0], torch.cos(ang)) and torch.allclose(r[:, 1], torch.sin(ang)) and torch.allclose(r[:, 3], 2 * torch.cos(0.1 * ang))
    f, amp = O.frequencies(dict(dims=8, base=50.0, scaling=H.YARN))
    assert abs(amp - (1 + 0.1 * math.log(3.0))) < 1e-12 and abs(f[-1] - 50.0 ** -0.75 / 3.0) < 1e-12
    # the correction enters the choice alone
    z = torch.tensor([[2.0, 1.0, 0.0]], dtype=F64)
    p = torch.softmax(z, -1)
    assert torch.allclose(O.route(z, 1, torch.tensor([0.0, 0.0, 0.9], dtype=F64)), torch.tensor([[0.0, 0.0, float(p[0, 2])]], dtype=F64))
    g, u = torch.tensor([5.0, -4.0], dtype=F64), torch.tensor([-9.0, 0.5], dtype=F64)
    c = O.clamped_glu(g, u, 2.0)
    assert torch.allclose(c, torch.stack([2.0 * torch.sigmoid(torch.tensor(3.404, dtype=F64)) * -1.0, -4.0 * torch.sigmoid(torch.tensor(-6.808, dtype=F64)) * 1.5]))


@pytest.mark.parametrize("dims,base,scaling", [(8, 50.0, H.YARN), (16, 10000.0, dict(factor=4.0, original=4096, fast=20.0, slow=2.0)),
                                               (64, 500000.0, dict(factor=1.0, original=128, fast=32.0, slow=1.0)), (2, 10.0, None)])
def test_rotation_table_agrees_with_the_oracle(dims, base, scaling):
    from mlx_vlm_amd.models.ragged import rotation

    rot = dict(base=base, dims=dims, **(dict(scaling=scaling) if scaling else {}))
    n, f, amp = rotation(rot)
    want, wamp = O.frequencies(rot)
    assert n == dims and np.allclose(f, want, rtol=1e-6, atol=0) and abs(amp - wamp) < 1e-12
