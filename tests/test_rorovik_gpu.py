"""Rorovik on MI355X against the plain restatement in tests/rorovik_oracle.py (float64 on the CPU, dense masks).

Small random checkpoints with unequal sizes (tests/rorovik_helpers.py) are written to disk and loaded through `utils.load_model`
(registry by config.json, safetensors reader, weight packing).  float32 serving is compared tightly, bfloat16 within the rounding of a
16-bit projection chain.  Covered: every mechanism alone (operator level and as a one-layer model); whole prompts against portions of
several sizes (down to two tokens and one) and against token-by-token decoding; batches of unequal requests against each alone; pages and
slots freed and used again; keys at page, tile and window borders, just inside and just outside the window, and far back among
hundreds, in prompts and decoding, with one score made to stand out; sinks that decide; mixed values; the first tokens; long decoding; sizes
that are equal or 1 elsewhere; greedy generation through generate_step and the continuous batch generator; replay of a scheduled trace, also
through the command line program; captured decode steps."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from tests import rorovik_helpers as H
from tests import rorovik_oracle as O

pytestmark = pytest.mark.gpu
F64 = torch.float64
TOL = {"float32": 4e-5, "bfloat16": 4e-2}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _close(got, want, dtype):
    """float32: every row within TOL.  bfloat16: the median row within TOL and eight rows in ten within twice that (an expert choice inside
    the rounding of a 16-bit activation moves that row)"""
    if dtype == "float32":
        return H.rel_rms(got, want) < TOL[dtype]
    return H.rel_rms(got, want, 0.5) < TOL[dtype] and H.rel_rms(got, want, 0.8) < 2 * TOL[dtype]


def _load(tmp_path, cfg, W, dtype, tokens=4096, seqs=6, name="m"):
    from mlx_vlm_amd.utils import load_model

    return load_model(H.write_checkpoint(str(tmp_path / name), cfg, W), dtype=dtype, kv_pool_tokens=tokens, max_seqs=seqs)


def _ids(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).numpy().astype(np.int32)


def _oracle(cfg, W, ids, layers=None):
    return O.Oracle(cfg, W, F64).forward(ids, layers)


def _portions(lm, ids, sizes):
    """the prompt in portions of the given sizes (cycled), every row's logits"""
    c, out, o, j = lm.make_cache(), [], 0, 0
    while o < len(ids):
        n = min(sizes[j % len(sizes)], len(ids) - o)
        out.append(lm.step([(c[0]._seq, ids[o:o + n])], want="all").cpu())
        o, j = o + n, j + 1
    c[0]._seq.release()
    return torch.cat(out)


def _whole(lm, ids):
    return _portions(lm, ids, [len(ids)])


def _split_rows(k, heads, D):
    """fp32 key rows [.., heads * D] as a bf16 pool keeps them: per head hi = bf16(k) and lo = bf16(k - hi), each padded to 8 columns"""
    D8 = (D + 7) & ~7
    v = k.view(*k.shape[:-1], heads, D)
    hi = v.to(torch.bfloat16)
    out = torch.zeros(*k.shape[:-1], heads, 2, D8, dtype=torch.bfloat16)
    out[..., 0, :D], out[..., 1, :D] = hi, (v - hi.float()).to(torch.bfloat16)
    return out.reshape(*k.shape[:-1], heads * 2 * D8)


def _joined_rows(pool, heads, D):
    """what such a pool holds, in float64"""
    if pool.dtype == torch.float32:
        return pool.double()
    v = pool.double().view(*pool.shape[:-1], heads, 2, (D + 7) & ~7)
    return (v[..., 0, :D] + v[..., 1, :D]).reshape(*pool.shape[:-1], heads * D)


# ------------------------------------------------------------------------------------------------ operators
@pytest.mark.parametrize("D", [52, 51, 640, 1540, 5000])
@pytest.mark.parametrize("T", [torch.float32, torch.bfloat16])
def test_sandwich_step_norms_the_result_adds_it_and_forms_the_next_input(T, D):
    from mlx_vlm_amd import ops

    g = torch.Generator().manual_seed(D)
    r = lambda *s: torch.randn(*s, generator=g)                                     # noqa: E731
    x, y, src = r(7, D), r(7, D + 4).to(T), r(7, D + 8).to(T)
    bias, wy, w = (0.5 * r(D)).to(T), (1 + 0.3 * r(D)).to(T), (1 + 0.3 * r(D)).to(T)
    pw = torch.rand(7, generator=g)
    pw[2] = 0.0
    d = lambda t: t.double()                                                        # noqa: E731
    tol = 3e-5 if T == torch.float32 else 3e-2
    for b, p in ((None, None), (bias, None), (None, pw), (bias, pw)):
        z = d(y)[:, :D] + (d(b) if b is not None else 0) + (d(p).view(-1, 1) * d(src)[:, :D] if p is not None else 0)
        new = d(x) + 0.7 * O.norm(z, d(wy), 1e-3)
        for kw, want in ((dict(w=w.cuda()), O.norm(new, d(w), 1e-3)), (dict(cast=True), new), ({}, None)):
            xd = x.cuda()
            h = ops.sandwich_step(xd, y.cuda()[:, :D], wy.cuda(), 0.7, eps=1e-3, bias=None if b is None else b.cuda(), pass_=None if p is None else p.cuda(),
                                  src=None if p is None else src.cuda()[:, :D], **kw)
            assert (xd.cpu().double() - new).abs().max() < 3e-5
            assert h is None if want is None else (h.dtype == T and (h.cpu().double() - want).abs().max() < tol * want.abs().max())
    table, ids = r(11, D).to(T), torch.tensor([3, 0, 10, 3, 7, 1, 5], dtype=torch.int32)
    xd = torch.full((7, D), float("nan")).cuda()
    h = ops.sandwich_step(xd, table.cuda(), wy.cuda(), ids=ids.cuda(), init=True, w=w.cuda(), eps=1e-3)
    new = O.norm(d(table)[ids.long()], d(wy), 1e-3)
    assert (xd.cpu().double() - new).abs().max() < 3e-5 and (h.cpu().double() - O.norm(new, d(w), 1e-3)).abs().max() < 4 * tol


@pytest.mark.parametrize("D,E,identity,top", [(48, 6, 1, 2), (56, 3, 2, 3), (57, 14, 0, 4), (1536, 13, 3, 2), (64, 1, 1, 1), (64, 40, 3, 7), (128, 200, 56, 9),
                                              (64, 90, 0, 90), (3584, 64, 8, 6)])
@pytest.mark.parametrize("T", [torch.float32, torch.bfloat16])
def test_router_scores_correction_and_identity_experts(T, D, E, identity, top):
    from mlx_vlm_amd import ops

    g = torch.Generator().manual_seed(D + E)
    C = E + identity
    for rows in (1, 5, 37):
        h, w = torch.randn(rows, D + 8, generator=g).to(T), (torch.randn(C, D, generator=g) * 2.0 / D ** 0.5).to(T)
        corr = torch.randn(C, generator=g) * 0.2
        z = h.double()[:, :D] @ w.double().T
        for c in (corr, None):
            want = O.route(z, top, c.double() if c is not None else torch.zeros(C, dtype=F64))
            sel = torch.softmax(z, -1) + (c.double() if c is not None else 0)
            top_c = torch.sort(sel, descending=True).values
            clear = (top_c[:, top - 1] - top_c[:, top] > 1e-6) if top < C else torch.ones(rows, dtype=torch.bool)
            gate, ident = ops.moe_router_softmax(h.cuda()[:, :D], w.cuda(), top, identity, None if c is None else c.cuda())
            assert gate.shape == (rows, E) and (ident is None) == (identity == 0)
            assert ((gate.cpu().double() - want[:, :E]).abs()[clear] < 1e-5).all() and clear.float().mean() > 0.9
            assert ((gate.cpu() != 0) == (want[:, :E] != 0))[clear].all()
            if identity:
                assert ((ident.cpu().double() - want[:, E:].sum(-1)).abs()[clear] < 1e-5).all()
    # ties: the lowest index wins; a correction lifts an expert into the choice and enters nothing else
    h = torch.zeros(2, D).to(T).cuda()
    gate, ident = ops.moe_router_softmax(h, w.cuda(), 1, identity)
    assert torch.allclose(gate[:, 0].cpu(), torch.full((2,), 1.0 / C), rtol=1e-6) and (gate[:, 1:] == 0).all()
    lift = torch.zeros(C)
    lift[C - 1] = 5.0
    gate, ident = ops.moe_router_softmax(h, w.cuda(), 1, identity, lift.cuda())
    got = ident if identity else gate[:, C - 1]
    assert torch.allclose(got.cpu(), torch.full((2,), 1.0 / C), rtol=1e-6) and (gate[:, : min(E, C - 1)] == 0).all()


@pytest.mark.parametrize("ff,E", [(16, 3), (13, 4)])
@pytest.mark.parametrize("T", [torch.float32, torch.bfloat16])
def test_gated_units_with_biases_and_with_a_route_table(T, ff, E):
    from mlx_vlm_amd import ops

    g = torch.Generator().manual_seed(ff)
    gu = (2 * torch.randn(9, 2 * E * ff + 8, generator=g)).to(T)
    tol = 1e-5 if T == torch.float32 else 3e-2
    gb, ub = (torch.randn(ff, generator=g).to(T) for _ in range(2))
    pad = (ff + 7) // 8 * 8
    for a, b in ((gb, ub), (None, None), (gb, None)):
        out = torch.zeros(9, pad, dtype=T, device="cuda")
        ops.glu_rows(gu.cuda(), gu.cuda()[:, pad:], ops.GLU_RELU, out=out[:, :ff], gbias=None if a is None else a.cuda(), ubias=None if b is None else b.cuda())
        z, u = gu.double()[:, :ff] + (a.double() if a is not None else 0), gu.double()[:, pad: pad + ff] + (b.double() if b is not None else 0)
        want = z.clamp(min=0) * u
        assert (out[:, :ff].cpu().double() - want).abs().max() < tol * want.abs().max() and (out[:, ff:] == 0).all()
    route = torch.rand(9, E, generator=g)
    route[torch.rand(9, E, generator=g) < 0.4] = 0.0
    for limit in (0.7, float("inf")):
        out = torch.full((9, (E * ff + 7) // 8 * 8), float("nan"), dtype=T, device="cuda")[:, : E * ff]
        ops.glu_rows(gu.cuda(), gu.cuda()[:, ff:], ops.GLU_CLAMPED, out=out, route=route.cuda(), E=E, ff=ff, estride=2 * ff, limit=limit)
        v = gu.double()[:, : 2 * E * ff].view(9, E, 2, ff)
        want = (O.clamped_glu(v[:, :, 0], v[:, :, 1], None if limit == float("inf") else limit) * route.double().view(9, E, 1)).reshape(9, E * ff)
        assert (out.cpu().double() - want).abs().max() < tol * want.abs().max()
        assert (out.cpu()[(route == 0).repeat_interleave(ff, 1)] == 0).all()


@pytest.mark.parametrize("T,K,E,top,ff,N", [(300, 128, 5, 2, 64, 72), (70, 64, 3, 3, 128, 64), (64, 192, 40, 4, 64, 320), (513, 64, 1, 1, 64, 8), (257, 64, 6, 2, 192, 128)])
@pytest.mark.parametrize("act", [0, 1, 3])
def test_experts_evaluated_pair_by_pair(T, K, E, top, ff, N, act):
    """the chosen pairs sorted by expert (unequal counts, an expert without tokens, tokens with fewer pairs than `top` and with none), gathered
    products, and their sum in the residual step"""
    from mlx_vlm_amd import ops

    g = torch.Generator().manual_seed(T + E)
    bf = torch.bfloat16
    h, wup, wdown = torch.randn(T, K + 8, generator=g).to(bf), (torch.randn(E * 2 * ff, K, generator=g) / K ** 0.5).to(bf), (torch.randn(N, E * ff, generator=g) / ff ** 0.5).to(bf)
    gate = torch.zeros(T, E)
    for t in range(T):
        n = int(torch.randint(0, top + 1, (1,), generator=g)) if t % 3 == 0 else top
        pick = torch.randperm(E, generator=g)[:n]
        if E > 2:
            pick = pick[pick != 1]                                                  # expert 1 stays without tokens
        gate[t, pick] = torch.rand(len(pick), generator=g) + 0.1
    tok, tile_expert, ntiles, slots = (x.cpu() for x in ops.moe_plan(gate.cuda(), top))
    n = int(ntiles)
    assert n == sum(-(-int((gate[:, e] != 0).sum()) // 128) for e in range(E))
    at = 0
    for e in range(E):
        mine = torch.nonzero(gate[:, e]).view(-1)
        tiles = -(-len(mine) // 128)
        assert (tile_expert[at: at + tiles] == e).all()
        seg = tok[at * 128: (at + tiles) * 128]
        assert torch.equal(seg[: len(mine)].long(), mine) and (seg[len(mine):] == -1).all()
        at += tiles
    for t in range(T):
        s = [int(i) for i in slots[t] if i >= 0]
        assert [int(tile_expert[i // 128]) for i in s] == torch.nonzero(gate[t]).view(-1).tolist() and all(int(tok[i]) == t for i in s)
    limit = 0.9
    out, slots = ops.moe_grouped_rows(h.cuda()[:, :K], wup.cuda(), wdown.cuda(), gate.cuda(), top, act, limit)
    hd, want = h.double()[:, :K], torch.zeros(T, N, dtype=F64)
    for e in range(E):
        a, u = hd @ wup.double()[e * 2 * ff: e * 2 * ff + ff].T, hd @ wup.double()[e * 2 * ff + ff: (e + 1) * 2 * ff].T
        m = O.clamped_glu(a, u, limit) if act == 3 else (O.gelu_tanh(a) if act == 0 else a * torch.sigmoid(a)) * u
        want += gate[:, e:e + 1].double() * (m @ wdown.double()[:, e * ff: (e + 1) * ff].T)
    x = torch.zeros(T, N).cuda()
    got = torch.zeros(T, N, dtype=F64)
    o, sl = out.cpu().double(), slots.cpu()
    for k in range(top):
        ok = sl[:, k] >= 0
        got[ok] += o[sl[ok, k].long()]
    assert (got - want).abs().max() < 2e-2 * want.abs().max()
    ops.sandwich_step(x, out, torch.ones(N, dtype=bf).cuda(), eps=1e-3, slots=slots, init=True)
    assert (x.cpu().double() - O.rms(got, 1e-3)).abs().max() < 1e-4


@pytest.mark.parametrize("HQ,HK,D,Dv", [(4, 2, 12, 20), (3, 3, 7, 5), (12, 2, 128, 128), (1, 1, 1, 1)])
@pytest.mark.parametrize("T", [torch.float32, torch.bfloat16])
def test_projection_rows_norm_over_all_heads_multiplier_and_mixed_values(T, HQ, HK, D, Dv):
    from mlx_vlm_amd import ops
    from mlx_vlm_amd.models.cache import PAGE

    g = torch.Generator().manual_seed(HQ * D)
    r = lambda *s: torch.randn(*s, generator=g)                                     # noqa: E731
    nq, nk, nv = HQ * D, HK * D, HK * Dv
    offs = (0, nq + 3, nq + nk + 3)
    n = 9
    x = r(n, nq + nk + nv + 5).to(T)
    qb, kb, vb = (0.5 * r(m) for m in (nq, nk, nv))
    qb, kb, vb, qw, kw = qb.to(T), kb.to(T), vb.to(T), (1 + 0.3 * r(nq)).to(T), (1 + 0.3 * r(nk)).to(T)
    pos = torch.tensor([0, 1, 5, 62, 63, 64, 65, 700, 3], dtype=torch.int32)
    seq = torch.tensor([1] * 8 + [0], dtype=torch.int32)
    bt = torch.zeros(2, 12, dtype=torch.int32)
    bt[1] = torch.randperm(12, generator=g).to(torch.int32) + 1
    other = r(13, PAGE, nv).to(T)
    row = lambda p, t: p[int(bt[int(seq[t]), int(pos[t]) // PAGE]), int(pos[t]) % PAGE]              # noqa: E731
    for temp, mix in (((0.3, 6), None), (None, 0.37), ((0.5, 1), 1.0)):
        kpool = torch.zeros(13, PAGE, ops.diff_key_width(HK, D, T == torch.bfloat16), dtype=T).cuda()
        vpool = torch.zeros(13, PAGE, nv, dtype=T).cuda()
        q = torch.full((n, nq), float("nan")).cuda()
        ops.qkv_rownorm_rows(x.cuda(), offs, HQ, HK, D, nv, qw.cuda(), kw.cuda(), 1e-4, seq.cuda(), pos.cuda(), bt.cuda(), q, kpool, vpool, qbias=qb.cuda(),
                             kbias=kb.cuda(), vbias=vb.cuda(), temp=temp, vother=None if mix is None else other.cuda(), mix=mix or 0.0)
        xd = x.double()
        wq = O.norm(xd[:, :nq] + qb.double(), qw.double(), 1e-4)
        if temp:
            wq = wq * O.temperature(701, dict(coef=temp[0], every=temp[1]), F64)[pos.long()].view(-1, 1)
        wk = O.norm(xd[:, offs[1]: offs[1] + nk] + kb.double(), kw.double(), 1e-4)
        wv = xd[:, offs[2]: offs[2] + nv] + vb.double()
        kp = _joined_rows(kpool.cpu(), HK, D)
        assert (q.cpu().double() - wq).abs().max() < 3e-5
        for t in range(n):
            v = wv[t] if mix is None else (1 - mix) * wv[t] + mix * row(other, t).double()
            assert ((row(kp, t) - wk[t]).abs() <= 2e-5 + 2.0 ** -16 * wk[t].abs()).all(), t
            assert ((row(vpool, t).cpu().double() - v).abs() <= (2e-6 if T == torch.float32 else 5e-3) * (1 + v.abs())).all(), t
        assert int((vpool != 0).any(-1).sum()) <= n                                 # nothing else was written


def _pool_case(g, deep=1890):
    """two sequences at different offsets on scattered pages, one `deep` tokens deep"""
    bt = torch.zeros(3, 32, dtype=torch.int32)
    bt[1, :31] = torch.randperm(31, generator=g).to(torch.int32) + 1
    tok_seq = torch.tensor([1] * 37 + [2] * 5, dtype=torch.int32)
    tok_pos = torch.tensor(list(range(deep, deep + 37)) + list(range(5)), dtype=torch.int32)
    qb = [torch.tensor(t, dtype=torch.int32).cuda() for t in ([0, 16, 32, 37], [16, 16, 5, 5])]
    return bt, tok_seq, tok_pos, qb


@pytest.mark.parametrize("D,Dv,Hh,G", [(12, 20, 6, 2), (16, 16, 2, 2), (6, 33, 3, 1), (40, 72, 20, 1), (64, 128, 6, 2), (128, 128, 12, 2), (1, 1, 1, 1),
                                       (18, 256, 2, 1), (256, 256, 1, 1), (72, 136, 4, 2), (768, 24, 7, 1)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_grouped_attention_bias_window_sink_and_gate_against_a_dense_softmax(dtype, D, Dv, Hh, G):
    from mlx_vlm_amd import ops
    from mlx_vlm_amd.models.cache import PAGE

    g = torch.Generator().manual_seed(D + Dv)
    bt, tok_seq, tok_pos, qb = _pool_case(g)
    kpool = torch.randn(32, PAGE, G * D, generator=g) * 0.7
    vpool = torch.randn(32, PAGE, G * Dv, generator=g).to(dtype)
    q = torch.randn(42, Hh * D, generator=g)
    pool = kpool if dtype == torch.float32 else _split_rows(kpool, G, D)
    kpool = _joined_rows(pool, G, D)
    rows = {sq: (kpool[bt[sq].long()].reshape(-1, G, D).double(), vpool[bt[sq].long()].reshape(-1, G, Dv).double()) for sq in (1, 2)}
    qd = q.double().view(42, Hh, D)
    gate = torch.randn(42, Hh + 3, generator=g).to(dtype)
    slopes = O.slopes(Hh, F64).float()
    sinks = torch.randn(Hh, generator=g) * 3
    for window, scale, slope, sink, gt in ((0, 1.0, slopes, sinks, gate), (17, 2.0, None, sinks + 4, None), (1025, 0.5, slopes * 0.01, None, gate),
                                           (1, 1.0, slopes, sinks, gate), (64, 4.0, slopes * 0.1, sinks - 8, None), (0, 1.0, None, None, None),
                                           (0, 1.0, slopes, sinks + 60, None)):
        scale = scale / max(D, 4) ** 0.5
        want = torch.zeros(42, Hh, Dv, dtype=F64)
        for t in range(42):
            sq, pos = int(tok_seq[t]), int(tok_pos[t])
            lo = max(0, pos - window + 1) if window else 0
            kh = torch.arange(Hh) // (Hh // G)
            s = torch.einsum("hd,jhd->hj", qd[t], rows[sq][0][lo:pos + 1][:, kh]) * scale
            if slope is not None:
                s = s - slope.double().view(Hh, 1) * (pos - torch.arange(lo, pos + 1)).double()
            if sink is None:
                w = torch.softmax(s, -1)
            else:
                w = torch.softmax(torch.cat([s, sink.double().view(Hh, 1)], 1), -1)[:, :-1]
            want[t] = torch.einsum("hj,jhd->hd", w, rows[sq][1][lo:pos + 1][:, kh])
            if gt is not None:
                want[t] *= torch.sigmoid(gt[t, :Hh].double()).view(Hh, 1)
        args = (tok_seq.cuda(), tok_pos.cuda(), bt.cuda(), Hh, G, D, Dv, scale)
        dev = lambda t: None if t is None else t.cuda()                             # noqa: E731
        kw = dict(window=window, slope=dev(slope), sink=dev(sink), gate=dev(gt))
        a, b = (torch.full((42, Hh * Dv + 8), float("nan"), dtype=dtype, device="cuda")[:, : Hh * Dv] for _ in range(2))
        ops.grouped_attn_blocks(q.cuda(), pool.cuda(), vpool.cuda(), *qb, *args, b, **kw)
        tol = 2e-5 if dtype == torch.float32 else 1e-2
        assert (b.cpu().double().view(42, Hh, Dv) - want).abs().max() < tol, window
        for nsplit in (None, 1, 2, 7, 64):                                          # workgroups that share a column group's keys
            ops.grouped_attn_rows(q.cuda(), pool.cuda(), vpool.cuda(), *args, a, nsplit=nsplit, **kw)
            assert (a.cpu().double().view(42, Hh, Dv) - want).abs().max() < tol, (window, nsplit)


@pytest.mark.parametrize("R,Dr,Hh", [(40, 8, 3), (21, 4, 2), (512, 64, 12), (136, 24, 10), (264, 2, 2), (96, 32, 20), (24, 0, 1), (520, 8, 2), (16, 16, 33)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_latent_attention_with_sinks_every_form_against_a_dense_softmax(dtype, R, Dr, Hh):
    from mlx_vlm_amd import ops
    from mlx_vlm_amd.models.cache import PAGE

    g = torch.Generator().manual_seed(R + Dr)
    bt, tok_seq, tok_pos, qb = _pool_case(g)
    pool = (torch.randn(32, PAGE, R + Dr, generator=g) * 0.7).to(dtype)
    rows = {sq: pool[bt[sq].long()].reshape(-1, R + Dr).double() for sq in (1, 2)}
    q = torch.randn(42, Hh, R + Dr, generator=g).to(dtype).float()                  # (the matrix-core forms take bf16 queries)
    sinks = torch.randn(Hh, generator=g) * 3
    for sink, scale in ((sinks, 1.0), (None, 2.0), (sinks + 7, 4.0)):
        scale = scale / (R + Dr) ** 0.5
        want = torch.zeros(42, Hh, R, dtype=F64)
        for t in range(42):
            sq, pos = int(tok_seq[t]), int(tok_pos[t])
            s = q[t].double() @ rows[sq][: pos + 1].T * scale
            if sink is not None:
                s = torch.cat([s, sink.double().view(Hh, 1)], 1)
            want[t] = torch.softmax(s, -1)[:, : pos + 1] @ rows[sq][: pos + 1, :R]
        args = (tok_seq.cuda(), tok_pos.cuda(), bt.cuda(), Hh, R, Dr, scale)
        dsink = None if sink is None else sink.cuda()
        tol = 2e-5 if dtype == torch.float32 else 1e-2                              # (a bf16 read-out is rounded once)
        for name, got in _latent_forms(ops, q.cuda(), pool.cuda(), qb, args, dsink):
            assert (got.cpu().double() - want).abs().max() < tol, name


def _latent_forms(ops, q, pool, qb, args, sink):
    R = args[4]
    yield "rows", ops.latent_attn(q, pool, *args, sink=sink)
    if R <= 512:
        yield "blocks", ops.latent_attn_blocks(q, pool, *qb, *args, sink=sink)
    if ops.latent_mfma_fits(pool, R, args[5]):
        yield "matrix-core blocks", ops.latent_attn_mfma(q.bfloat16(), pool, *args, sink=sink, blocks=qb).float()
        for nsplit in (None, 1, 2, 7, 64):
            yield f"matrix-core rows, {nsplit} splits", ops.latent_attn_mfma(q.bfloat16(), pool, *args, sink=sink, nsplit=nsplit).float()


@pytest.mark.parametrize("R,Dr,Rq", [(40, 8, 24), (21, 4, 9), (512, 64, 1536), (16, 0, 1), (300, 2, 7)])
@pytest.mark.parametrize("T", [torch.float32, torch.bfloat16])
def test_latent_rows_query_latent_and_scaled_interleaved_rotation(T, R, Dr, Rq):
    from mlx_vlm_amd import ops
    from mlx_vlm_amd.models.cache import PAGE
    from mlx_vlm_amd.models.ragged import rotation

    g = torch.Generator().manual_seed(R)
    n, Hh, D = 9, 3, 5
    pos = torch.tensor([0, 1, 5, 62, 63, 64, 65, 700, 3], dtype=torch.int32)
    seq = torch.tensor([1] * 8 + [0], dtype=torch.int32)
    bt = torch.zeros(2, 12, dtype=torch.int32)
    bt[1] = torch.randperm(12, generator=g).to(torch.int32) + 1
    x = torch.randn(n, R + Dr + Rq + 3, generator=g).to(T)
    w, wq = (1 + 0.3 * torch.randn(R, generator=g)).to(T), (1 + 0.3 * torch.randn(Rq, generator=g)).to(T)
    q = torch.randn(n, Hh * (D + Dr), generator=g).to(T)
    tol = 3e-5 if T == torch.float32 else 3e-2
    for scaling in (H.YARN, None) if Dr else (None,):
        rot = dict(base=500.0, dims=Dr, **(dict(scaling=scaling) if scaling else {}))
        _, f, amp = rotation(rot if Dr else None)
        inv = torch.from_numpy(f).cuda() if Dr else None
        pool = torch.zeros(13, PAGE, R + Dr, dtype=T).cuda()
        xd = x.cuda()
        cq = ops.latent_prep_rows(xd[:, : R + Dr], w.cuda(), R, Dr, inv, seq.cuda(), pos.cuda(), bt.cuda(), pool, 1e-4, amp=amp, dq=xd[:, R + Dr + 3:], wq=wq.cuda())
        assert (cq.cpu().double() - O.norm(x.double()[:, R + Dr + 3:], wq.double(), 1e-4)).abs().max() < tol
        want = torch.cat([O.norm(x.double()[:, :R], w.double(), 1e-4), x.double()[:, R: R + Dr]], 1)
        qabs = torch.zeros(n, Hh, R + Dr).cuda()
        if Dr:
            ops.rope_pairs_rows(q.cuda()[:, D:], D + Dr, Hh, Dr, inv, pos.cuda(), qabs.view(n, -1)[:, R:], R + Dr, amp=amp)

            def turned(y):               # [n, .., Dr] at the rows' own positions
                full = torch.zeros(701, *y.shape[1:], dtype=F64)
                out = torch.empty_like(y)
                for t in range(n):
                    full[int(pos[t])] = y[t]
                    out[t] = O.rotate_pairs(full, rot)[int(pos[t])]
                return out
            want[:, R:] = turned(want[:, R:])
            wq_rot = turned(q.double().view(n, Hh, D + Dr)[..., D:])
            assert (qabs[:, :, R:].cpu().double() - wq_rot).abs().max() < 2e-4
            if T == torch.bfloat16:
                half = torch.zeros(n, Hh, R + Dr, dtype=T).cuda()
                ops.rope_pairs_rows(q.cuda()[:, D:], D + Dr, Hh, Dr, inv, pos.cuda(), half.view(n, -1)[:, R:], R + Dr, amp=amp)
                assert (half[:, :, R:].cpu().double() - wq_rot).abs().max() < 3e-2
        for t in range(n):
            got = pool[int(bt[int(seq[t]), int(pos[t]) // PAGE]), int(pos[t]) % PAGE].cpu().double()
            assert (got - want[t]).abs().max() < max(tol, 2e-4), t


# ------------------------------------------------------------------------------------------------ one-layer models
ONE = {"attention": [H.attention()], "attention_equal_heads": [H.attention(heads=3, kv_heads=3, window=64, mlp=H.moe())],
       "attention_one_kv_head_no_window": [H.attention(heads=5, kv_heads=1, dim=12, vdim=12, window=0, every=1)],
       "attention_window_1": [H.attention(heads=1, kv_heads=1, dim=2, vdim=1, window=1, every=None, v_mix=False, mlp=None)],
       "attention_wide": [H.attention(heads=2, kv_heads=1, dim=64, vdim=136, scale=0.12, window=100, every=64)],
       "latent": [H.latent()], "latent_one_head_no_scaling": [H.latent(heads=1, dim=24, rot_dim=4, vdim=3, scaling=None, mlp=None)],
       "latent_no_rotation": [H.latent(rot_dim=0, mlp="dense")],
       "latent_wide": [H.latent(heads=4, dim=64, rot_dim=32, vdim=48, kv_rank=264, q_rank=100, base=10000.0)],
       "latent_rank_520": [H.latent(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=520, q_rank=16, mlp=None)],
       "latent_odd_sizes": [H.latent(heads=3, dim=7, rot_dim=2, vdim=9, kv_rank=21, q_rank=11, mlp=H.dense(19))],
       "moe_pair_by_pair": [H.attention(mlp=H.moe(experts=6, identity=2, top=3, ff=64)), H.latent(mlp=H.moe(experts=4, identity=0, top=2, ff=128, limit=None))],
       "moe_all_chosen": [H.latent(mlp=H.moe(experts=3, identity=2, top=5))], "moe_top_1": [H.latent(mlp=H.moe(experts=7, identity=3, top=1, ff=9, limit=0.4))],
       "moe_mostly_identity": [H.attention(mlp=H.moe(experts=1, identity=6, top=3))]}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", sorted(ONE))
def test_each_mixer_and_feed_forward_alone(tmp_path, kind, dtype):
    cfg = H.config(ONE[kind], width=128 if "pair" in kind else 56, side=0 if "equal" in kind else 12, mult=1.0 if "wide" in kind else 0.6)
    W = H.weights(cfg, seed=3)
    ids = _ids(150, cfg["vocab"], 5)
    lm = _load(tmp_path, cfg, W, dtype, tokens=512).language_model
    want = _oracle(cfg, W, ids)
    assert _close(_whole(lm, ids), want, dtype)
    assert _close(_portions(lm, ids, [70, 1, 2, 30]), want, dtype)
    if "pair" in kind and dtype == "bfloat16":
        assert lm.GROUPED_ROWS <= 70


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layers_match_layer_by_layer(tmp_path, dtype):
    cfg = H.mixed_config()
    W = H.weights(cfg, seed=11)
    ids = _ids(90, cfg["vocab"], 6)
    lm = _load(tmp_path, cfg, W, dtype, tokens=512).language_model
    lm._trace = []
    c = lm.make_cache()
    lm.step([(c[0]._seq, ids)], want="all")
    ref = []
    _oracle(cfg, W, ids, ref)
    assert len(lm._trace) == len(ref) == 8 and len(c) == 8
    for i, (a, b) in enumerate(zip(lm._trace, ref)):
        assert _close(a.cpu(), b, dtype), i
    lm._trace = None
    c[0]._seq.release()


# ------------------------------------------------------------------------------------------------ schedules
@pytest.fixture(scope="module")
def mixed32(tmp_path_factory):
    cfg = H.mixed_config()
    W = H.weights(cfg, seed=21)
    model = _load(tmp_path_factory.mktemp("mixed32"), cfg, W, "float32", tokens=1024, seqs=4)
    return cfg, W, model.language_model


def test_portions_and_token_by_token_equal_the_whole_prompt(mixed32):
    cfg, W, lm = mixed32
    ids = _ids(200, cfg["vocab"], 7)
    want = _oracle(cfg, W, ids)
    assert H.rel_rms(_whole(lm, ids), want) < TOL["float32"]
    for sizes in ([1], [2], [3, 1, 2], [37], [61, 2, 1], [63], [64], [65, 1, 1, 1, 2], [9, 70]):
        assert H.rel_rms(_portions(lm, ids, sizes), want) < TOL["float32"], sizes


def test_bf16_portions_and_decode(tmp_path):
    cfg = H.mixed_config()
    W = H.weights(cfg, seed=22)
    lm = _load(tmp_path, cfg, W, "bfloat16", tokens=1024).language_model
    ids = _ids(140, cfg["vocab"], 8)
    want = _oracle(cfg, W, ids)
    for sizes in ([140], [1], [2], [5, 1, 1, 40], [64, 3]):
        assert _close(_portions(lm, ids, sizes), want, "bfloat16"), sizes


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_batch_equals_each_alone_and_pages_and_slots_are_reused(tmp_path, dtype):
    cfg = H.mixed_config()
    W = H.weights(cfg, seed=21)
    lm = _load(tmp_path, cfg, W, dtype, tokens=1024, seqs=4).language_model
    rng = np.random.default_rng(3)
    reqs = [_ids(n, cfg["vocab"], 30 + n) for n in (130, 2, 75, 1, 64, 199, 33)]
    alone = [_oracle(cfg, W, r) for r in reqs]
    free0 = lm.pool.free_pages
    live, waiting, got = {}, list(range(len(reqs))), {i: [] for i in range(len(reqs))}
    used_slots, used_pages = [], []
    while waiting or live:
        while waiting and len(live) < 4:
            i = waiting.pop(0)
            live[i] = [lm.make_cache(), 0]
            used_slots.append(live[i][0][0]._seq.seq)
        entries, who = [], []
        for i, (c, o) in live.items():
            if rng.random() < 0.25 and len(live) > 1:
                continue                                                     # left out of this step
            n = min(int(rng.choice([1, 1, 2, 3, 17, 64, 70])), len(reqs[i]) - o)
            entries.append((c[0]._seq, reqs[i][o:o + n]))
            who.append((i, n))
        if not entries:
            continue
        lg = lm.step(entries, want="all").cpu()
        o = 0
        for i, n in who:
            got[i].append(lg[o:o + n])
            o += n
            live[i][1] += n
            if live[i][1] == len(reqs[i]):
                c = live.pop(i)[0]
                used_pages += list(c[0]._seq.pages)
                c[0]._seq.release()
    assert _close(torch.cat([torch.cat(got[i]) for i in range(len(reqs))]), torch.cat(alone), dtype)
    assert lm.pool.free_pages == free0 and len(set(used_slots)) < len(used_slots) and len(set(used_pages)) < len(used_pages)


def test_wanted_rows_are_a_subset_or_none(mixed32):
    cfg, W, lm = mixed32
    a, b = _ids(50, cfg["vocab"], 1), _ids(20, cfg["vocab"], 2)
    wa, wb = _oracle(cfg, W, a), _oracle(cfg, W, b)
    ca, cb = lm.make_cache(), lm.make_cache()
    assert lm.step([(ca[0]._seq, a[:30])], want=[[]]) is None
    lg = lm.step([(cb[0]._seq, b), (ca[0]._seq, a[30:])], want=[[3, 19], [0, 7, 19]]).cpu()
    assert H.rel_rms(lg, torch.cat([wb[[3, 19]], wa[[30, 37, 49]]])) < TOL["float32"]
    ca[0]._seq.release(), cb[0]._seq.release()


def test_pool_exhaustion_is_an_error_not_a_fault(tmp_path):
    cfg = H.config([H.latent(), H.attention()])
    lm = _load(tmp_path, cfg, H.weights(cfg, seed=1), "float32", tokens=128, seqs=2).language_model
    c = lm.make_cache()
    lm.step([(c[0]._seq, _ids(128, cfg["vocab"], 1))])
    with pytest.raises(RuntimeError):
        lm.step([(c[0]._seq, _ids(1, cfg["vocab"], 2))])
    c[0]._seq.release()
    c = lm.make_cache()
    lm.step([(c[0]._seq, _ids(100, cfg["vocab"], 3))])
    c[0]._seq.release()


def test_a_step_is_taken_back_by_trimming_the_cache(tmp_path):
    """row caches only: after a trim the same positions are written again and nothing of the dropped tokens is seen"""
    cfg = H.mixed_config()
    W = H.weights(cfg, seed=33)
    lm = _load(tmp_path, cfg, W, "float32", tokens=512).language_model
    a, b = _ids(90, cfg["vocab"], 4), _ids(30, cfg["vocab"], 5)
    want = _oracle(cfg, W, np.concatenate([a[:60], b]))
    c = lm.make_cache()
    lm.step([(c[0]._seq, a)])
    assert all(x.is_trimmable() for x in c) and max(x.trim(30) for x in c) == 30 and c[0].offset == 60
    got = lm.step([(c[0]._seq, b)], want="all").cpu()
    assert H.rel_rms(got, want[60:]) < TOL["float32"]
    c[0]._seq.release()


# ------------------------------------------------------------------------------------------------ edges made visible
def _marked_embedding(W):
    """token 1 (`mark`) lives on stream direction 0 alone, token 2 (the asking token) on direction 1 alone; no other token has a component
    along either"""
    emb = W["embed"].float()
    emb[:, :2] = 0
    emb[1], emb[2] = 0, 0
    emb[1, 0], emb[2, 1] = 4.0, 4.0
    W["embed"] = emb.to(torch.bfloat16)


def _mark_attention(W, p="l0.mix."):
    """the key of `mark` and the query of the asking token point along the all-ones direction; every other key leans to a direction
    orthogonal to it"""
    _marked_embedding(W)
    k, q = 0.3 * W[p + "k"].float(), W[p + "q"].float()
    k[:, :2], q[:, :2] = 0, 0
    k[:, 0], q[:, 1] = 3.0, 3.0
    W[p + "k"], W[p + "q"] = k.to(torch.bfloat16), q.to(torch.bfloat16)
    W[p + "k.b"] = (torch.tensor([1.0, -1.0] * (k.shape[0] // 2))).to(torch.bfloat16)
    W[p + "q.b"] = torch.zeros(q.shape[0]).to(torch.bfloat16)


def _mark_latent(W, R, p="l0.mix."):
    """latent coordinate 0 belongs to `mark`, query-latent coordinate 0 to the asking token; the unrotated key of coordinate 0 and the query of
    that latent are all ones"""
    _marked_embedding(W)
    dkv, dq, uk, uq = (W[p + n].float() for n in ("dkv", "dq", "uk", "uq"))
    dkv[:, :2], dq[:, :2] = 0, 0
    dkv[0], dq[0] = 0, 0
    dkv[0, 0], dq[0, 1] = 3.0, 3.0
    uk, uq = 0.3 * uk, 0.3 * uq
    uk[:, 0], uq[:, 0] = 1.0, 1.0
    for n, t in (("dkv", dkv), ("dq", dq), ("uk", uk), ("uq", uq)):
        W[p + n] = t.to(torch.bfloat16)


def _check_probe(lm, cfg, W, dtype, n, ask, at, seen, portions):
    ids = 3 + _ids(n, cfg["vocab"] - 3, 40 + ask + at)
    ids[at], ids[ask] = 1, 2
    want = _oracle(cfg, W, ids)
    other = ids.copy()
    other[at] = 5
    moved = H.rel_rms(_oracle(cfg, W, other)[ask:ask + 1], want[ask:ask + 1])
    if seen:                                              # the probe is sharp: with and without `mark` in view differ widely
        assert moved > 0.05, (ask, at, moved)
    else:
        assert moved < 1e-9, (ask, at, moved)             # out of view: the asked row does not know the token at all
    for sizes in portions:
        sizes = [s for s in sizes if s > 0]
        got = _portions(lm, ids, sizes)
        assert H.rel_rms(got[ask:ask + 1], want[ask:ask + 1]) < (2.5 if dtype == "bfloat16" else 1) * TOL[dtype], (ask, at, sizes)
        assert _close(got, want, dtype), (ask, at, sizes)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("window", [1, 2, 16, 17, 33, 64, 65, 130])
def test_window_edge_in_prompt_and_decoding(tmp_path, window, dtype):
    """token `mark` appears once, at distance window - 1 (just inside) or window (just outside) of the asked position, and its key towers over
    all others.  Whole prompt, portions cut at the edge and at the asked token, and decoding token by token must agree with the oracle."""
    cfg = H.config([H.attention(heads=2, kv_heads=1, dim=8, vdim=12, scale=3.0, window=window, coef=0.1, every=64, mlp=None)], width=48, vocab=64)
    W = H.weights(cfg, seed=5)
    _mark_attention(W)
    lm = _load(tmp_path, cfg, W, dtype, tokens=1024).language_model
    n = 2 * window + 70
    for ask in (window + 3, n - 1):
        for at in {ask - window + 1, ask - window}:
            if not 0 <= at < ask:
                continue
            _check_probe(lm, cfg, W, dtype, n, ask, at, ask - at < window, ([n], [at + 1, 1000], [ask, 1], [ask - 1, 2], [at, 1, 1000], [3, 1]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["attention", "latent"])
def test_far_key_among_hundreds_and_at_page_borders(tmp_path, kind, dtype):
    """no window: one key whose score towers over all others, at the first positions, around page borders and hundreds of tokens back; seen
    from its own position's successor and from far away, in a prompt, at a portion's first token and decoded"""
    layer = (H.attention(heads=2, kv_heads=1, dim=16, vdim=16, scale=2.0, window=0, coef=0.1, every=64, mlp=None) if kind == "attention" else
             H.latent(heads=2, dim=16, rot_dim=4, vdim=16, kv_rank=24, q_rank=16, scale=0.5, mlp=None))
    cfg = H.config([layer], width=48, vocab=64)
    W = H.weights(cfg, seed=5)
    _mark_attention(W) if kind == "attention" else _mark_latent(W, 24)
    lm = _load(tmp_path, cfg, W, dtype, tokens=1024).language_model
    n = 700
    for at in (0, 1, 63, 64, 65, 255, 256, 511, 640):
        for ask in sorted({at + 1, min(at + 130, n - 1), n - 1}):
            _check_probe(lm, cfg, W, dtype, n, ask, at, True, ([n], [at + 1, 1000], [ask, 1], [ask - 1, 2]) + (([at, 1, 1000],) if at else ()))


@pytest.mark.parametrize("kind", ["attention", "latent"])
def test_sinks_count_once_and_are_neither_scaled_nor_biased(tmp_path, kind):
    """sinks as large as the scores: leaving them out, scaling them or biasing them by a distance moves the logits"""
    cfg = H.config([H.attention(window=40, mlp=None) if kind == "attention" else H.latent(mlp=None)])
    W = H.weights(cfg, seed=45)
    W["l0.mix.sink"] = torch.linspace(1.0, 3.0, W["l0.mix.sink"].numel()).to(torch.bfloat16)
    ids = _ids(120, cfg["vocab"], 43)
    want = _oracle(cfg, W, ids)
    for change in (-100.0, 0.3, 1.0):
        W2 = dict(W)
        W2["l0.mix.sink"] = (W["l0.mix.sink"].float() * 0.3 if change == 0.3 else W["l0.mix.sink"].float() + change).to(torch.bfloat16)
        assert H.rel_rms(_oracle(cfg, W2, ids), want) > 1e-3
    for dtype in ("float32", "bfloat16"):
        lm = _load(tmp_path, cfg, W, dtype, tokens=256, name=dtype).language_model
        assert _close(_whole(lm, ids), want, dtype) and _close(_portions(lm, ids, [7, 1, 30, 2]), want, dtype), dtype


def test_values_are_mixed_with_those_of_the_first_mixing_layer(tmp_path):
    """the first layer that mixes is not the first attention layer; its own mixing weight is unused, a later layer's decides"""
    layers = [H.attention(heads=2, v_mix=False), H.attention(heads=4, window=30), H.latent(mlp="dense"), H.attention(heads=2, dim=10, mlp=None), H.attention(heads=6, window=0)]
    cfg = H.config(layers)
    W = H.weights(cfg, seed=47)
    ids = _ids(130, cfg["vocab"], 48)
    want = _oracle(cfg, W, ids)
    for i, moves in ((1, False), (3, True), (4, True)):
        W2 = dict(W)
        W2[f"l{i}.mix.vmix"] = torch.tensor(0.95).to(torch.bfloat16)
        assert (H.rel_rms(_oracle(cfg, W2, ids), want) > 1e-2) == moves
    for dtype in ("float32", "bfloat16"):
        lm = _load(tmp_path, cfg, W, dtype, tokens=256, name=dtype).language_model
        assert [ns.vother if ns.type == "attention" else None for ns in lm._L] == [None, None, None, 1, 1]
        for sizes in ([130], [7, 1, 30, 2], [64, 3]):
            assert _close(_portions(lm, ids, sizes), want, dtype), (dtype, sizes)


def test_first_tokens_and_a_one_token_request(mixed32):
    cfg, W, lm = mixed32
    for n in (1, 2, 3, 4, 5):
        ids = _ids(n, cfg["vocab"], 90 + n)
        want = _oracle(cfg, W, ids)
        assert H.rel_rms(_whole(lm, ids), want) < TOL["float32"]
        assert H.rel_rms(_portions(lm, ids, [1]), want) < TOL["float32"]


def test_long_decoding_crosses_pages_windows_and_multiplier_steps(tmp_path):
    cfg = H.config([H.attention(window=70, every=50), H.latent(mlp="dense"), H.attention(window=0, mlp=None), H.latent(heads=2, dim=8, rot_dim=2, vdim=8)])
    W = H.weights(cfg, seed=17)
    ids = _ids(400, cfg["vocab"], 19)
    want = _oracle(cfg, W, ids)
    for dtype in ("float32", "bfloat16"):
        lm = _load(tmp_path, cfg, W, dtype, tokens=1024, name=dtype).language_model
        got = _portions(lm, ids, [20] + [1] * 380)
        assert _close(got, want, dtype)
        assert H.rel_rms(got[-1:], want[-1:]) < 2.5 * TOL[dtype]


def test_other_sizes(tmp_path):
    """widths, head sizes and feed-forward sizes that are not multiples of 8, an odd vocabulary, more than sixteen heads on one key head, a window
    beyond the prompt, a token input of one column, a multiplier of one"""
    layers = [H.attention(heads=18, kv_heads=1, dim=5, vdim=7, scale=0.7, window=1000, mlp=H.dense(37)),
              H.latent(heads=19, dim=5, rot_dim=6, vdim=3, kv_rank=13, q_rank=7, mlp=H.moe(experts=2, identity=1, top=1, ff=11)),
              H.attention(heads=5, kv_heads=5, dim=6, vdim=9, window=3, v_mix=False, mlp=H.moe(experts=17, identity=1, top=6, ff=5, limit=100.0)),
              H.latent(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, q_rank=1, mlp=None)]
    for side in (1, 17):
        cfg = H.config(layers, vocab=301, width=61, eps=3e-4, mult=1.0, side=side)
        W = H.weights(cfg, seed=23)
        ids = _ids(100, cfg["vocab"], 29)
        want = _oracle(cfg, W, ids)
        for dtype in ("float32", "bfloat16"):
            lm = _load(tmp_path, cfg, W, dtype, tokens=256, name=f"{dtype}{side}").language_model
            assert _close(_whole(lm, ids), want, dtype), dtype
            assert _close(_portions(lm, ids, [50, 1, 2]), want, dtype), dtype


# ------------------------------------------------------------------------------------------------ generation
def _greedy_oracle(cfg, W, prompt, n):
    ids, toks, margins = list(prompt), [], []
    for _ in range(n):
        lg = _oracle(cfg, W, np.asarray(ids))[-1]
        top = torch.topk(lg, 2).values
        toks.append(int(lg.argmax()))
        margins.append(float((top[0] - top[1]) / lg.std()))
        ids.append(toks[-1])
    return toks, margins


def test_greedy_generation_through_generate_step_and_the_batch_generator(tmp_path):
    from mlx_vlm_amd.batch import BatchGenerator
    from mlx_vlm_amd.generate import generate_step

    cfg = H.config(H.mixed_layers()[:5])
    W = H.weights(cfg, seed=51)
    model = _load(tmp_path, cfg, W, "float32", tokens=2048, seqs=8)
    prompts = [_ids(n, cfg["vocab"], 60 + n) for n in (9, 70, 33)]
    refs = [_greedy_oracle(cfg, W, p, 12) for p in prompts]

    def agree(got, ref):
        toks, margins = ref
        for a, b, m in zip(got, toks, margins):
            if a != b:
                assert m < 0.05, (got, toks, margins)            # a tie within the bf16 rounding of the sampler's logits
                return
    for p, ref in zip(prompts, refs):
        for lookahead in (0, 4):                                 # steps enqueued ahead of the token asked for are taken back at the end
            got = [t for t, _ in generate_step(p[None], model, None, None, max_tokens=12, temperature=0.0, lookahead=lookahead)]
            assert len(got) == 12
            agree(got, ref)
    gen = BatchGenerator(model, None, max_tokens=12, completion_batch_size=2, prefill_batch_size=2, compute_logprobs=True)
    uids = gen.insert([p for p in prompts])
    out = {u: [] for u in uids}
    while gen.has_work:
        _, rs = gen.next()
        for r in rs:
            out[r.uid].append(r.token)
    gen.close()
    for u, ref in zip(uids, refs):
        assert len(out[u]) == 12
        agree(out[u], ref)
    assert len(model.language_model.pool._free_seqs) >= 7         # rows gave their slots back (the scratch row keeps one)


def test_trace_session_replays_mixed_steps(tmp_path):
    from mlx_vlm_amd.batch import TraceSession

    cfg = H.config(H.mixed_layers()[:5])
    W = H.weights(cfg, seed=61)
    model = _load(tmp_path, cfg, W, "float32", tokens=256, seqs=4)
    a, b = _ids(100, cfg["vocab"], 1), _ids(30, cfg["vocab"], 2)
    wa, wb = _oracle(cfg, W, a), _oracle(cfg, W, b)
    s = TraceSession(model)
    assert s.step([("a", a[:64].tolist(), [])]) is None
    lg = s.step([("a", a[64:99].tolist(), [0, 34]), ("b", b[:29].tolist(), [28])])
    assert H.rel_rms(lg, torch.stack([wa[64], wa[98], wb[28]])) < TOL["float32"]
    lg = s.step([("b", b[29:].tolist(), [0]), ("a", a[99:].tolist(), [0])], end=["a", "b"])
    assert H.rel_rms(lg, torch.stack([wb[29], wa[99]])) < TOL["float32"]
    assert model.language_model.pool.free_pages == 4


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_program_writes_the_asked_logits(tmp_path, dtype):
    """bin/trace_run as a child process: steps on its standard input, `done <step>` lines and logits files back"""
    cfg = H.config([H.attention(), H.latent(mlp="dense"), H.attention(heads=2, mlp=None)])
    W = H.weights(cfg, seed=63)
    folder = H.write_checkpoint(str(tmp_path / "m"), cfg, W)
    a, b = _ids(70, cfg["vocab"], 1), _ids(9, cfg["vocab"], 2)
    wa, wb = _oracle(cfg, W, a), _oracle(cfg, W, b)
    steps = [dict(step=0, entries=[dict(id="a", tokens=a[:66].tolist(), want=[0, 65])], end=[]),
             dict(step=1, entries=[dict(id="a", tokens=a[66:67].tolist(), want=[]), dict(id="b", tokens=b[:2].tolist(), want=[1])], end=[]),
             dict(step=2, entries=[dict(id="b", tokens=b[2:].tolist(), want=[6]), dict(id="a", tokens=a[67:].tolist(), want=[0, 2])], end=["a", "b"]),
             dict(step=3, entries=[dict(id="c", tokens=b.tolist(), want=[8])], end=["c"])]
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out),
                        "--max-tokens", "192"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    want = {0: wa[[0, 65]], 1: wb[[1]], 2: torch.cat([wb[[8]], wa[[67, 69]]]), 3: wb[[8]]}
    for n, w in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, cfg["vocab"]))
        assert got.shape == w.shape and H.rel_rms(got, w) < 2.5 * TOL[dtype], n


@pytest.mark.parametrize("rows", [1, 3, 12, 64])
def test_captured_decode_steps_equal_eager_ones(tmp_path, rows):
    """a captured decode step is replayed many times, with eager work (another request's prompt, a release, synchronisations)
    between the replays; every replay's logits and token must equal the eager step's.  12 and 64 rows: the prompt forms of the attentions
    and the experts pair by pair inside a captured step."""
    from mlx_vlm_amd.sample_utils import make_sampler

    pairs = [H.attention(window=70, mlp=H.moe(experts=6, identity=2, top=3, ff=64)), H.latent(mlp=H.moe(experts=4, identity=0, top=2, ff=64)), H.attention(heads=2)]
    cfg = H.mixed_config() if rows < 64 else H.config(pairs, width=64)
    W = H.weights(cfg, seed=71)
    lm = _load(tmp_path, cfg, W, "bfloat16", tokens=16384, seqs=rows + 3).language_model
    sargs = make_sampler().engine_args()
    prompts = [_ids(n, cfg["vocab"], 80 + n) for n in ([40, 7, 66] * 22)[:rows]]
    steps = 70 if rows < 64 else 20

    def run(use_graph):
        caches = lm.make_cache_batch(rows)
        lg = lm.prefill(torch.cat([torch.as_tensor(p) for p in prompts]).cuda().reshape(-1, 1), None, caches, [len(p) for p in prompts])
        st = lm.decode_begin(caches, lg.argmax(-1), np.zeros((rows, 1)), max_new_tokens=80)
        out = []
        for i in range(steps):                                       # crosses a page border and the windows in every row
            lm.decode_run(st, 1, sargs, use_graph=use_graph)
            out.append((st.tok.cpu().clone(), st.logits.float().cpu().clone()))
            if i % 9 == 4:                                           # eager work between replays
                other = lm.make_cache()
                lm.step([(other[0]._seq, _ids(30 + i, cfg["vocab"], i))])
                torch.cuda.synchronize()
                other[0]._seq.release()
        for c in caches:
            c[0]._seq.release()
        return out
    eager, graph = run(False), run(True)
    assert any(isinstance(v, tuple) for v in lm._graphs.values())            # a graph was captured and used
    for i, ((t0, l0), (t1, l1)) in enumerate(zip(eager, graph)):
        assert torch.equal(t0, t1) and torch.equal(l0, l1), i


def test_sampled_generation_uses_the_device_sampler_and_refuses_what_is_not_built(tmp_path):
    from mlx_vlm_amd.generate import generate_step

    cfg = H.config(H.mixed_layers()[:3])
    model = _load(tmp_path, cfg, H.weights(cfg, seed=91), "bfloat16", tokens=1024, seqs=4)
    p = _ids(20, cfg["vocab"], 5)
    runs = [[t for t, _ in generate_step(p[None], model, None, None, max_tokens=16, temperature=0.8, top_p=0.9, seed=7)] for _ in range(2)]
    assert runs[0] == runs[1] and len(runs[0]) == 16 and all(0 <= t < cfg["vocab"] for t in runs[0])
    with pytest.raises(NotImplementedError):
        list(generate_step(p[None], model, None, None, max_tokens=4, repetition_penalty=1.3))
    assert len(model.language_model.pool._free_seqs) == 4           # every generation gave its slot back
