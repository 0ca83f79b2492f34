"""Zivitar on MI355X against the plain restatement in tests/zivitar_oracle.py (float64 on the CPU, dense masks, token loops).

Small random checkpoints with unequal sizes (tests/zivitar_helpers.py) are written to disk and loaded through
`utils.load_model` (registry by config.json, safetensors reader, weight packing).  float32 serving is compared tightly,
bfloat16 within the rounding of a 16-bit projection chain.  Covered: every mechanism alone (operator level and as a one-layer
model); borrowed tensors; whole prompts against portions of several sizes (down to two tokens and one) and against token-by-token
decoding; batches of unequal requests against each alone; pages, state slots and carried convolution inputs freed and used
again; keys at page, tile and window borders, just inside and just outside the window, the kept first tokens and the next ones, and
far back among hundreds, in prompts and decoding, with one score made to stand out; recurrent states that remember hundreds of
tokens; the first tokens; long decoding; sizes that are equal or 1 elsewhere; greedy generation through generate_step and the
continuous batch generator; replay of a scheduled trace, also through the command line program; captured decode steps."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from tests import zivitar_helpers as H
from tests import zivitar_oracle as O

pytestmark = pytest.mark.gpu
F64 = torch.float64
TOL = {"float32": 4e-5, "bfloat16": 4e-2}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _close(got, want, dtype):
    """float32: every row within TOL.  bfloat16: the median row within TOL and nine rows in ten within twice that (the difference of
    two maps and its norm amplify a 16-bit rounding where the maps nearly agree)"""
    if dtype == "float32":
        return H.rel_rms(got, want) < TOL[dtype]
    return H.rel_rms(got, want, 0.5) < TOL[dtype] and H.rel_rms(got, want, 0.9) < 2 * TOL[dtype]


def _load(tmp_path, cfg, W, dtype, tokens=4096, seqs=6, name="m"):
    from mlx_vlm_amd.utils import load_model

    return load_model(H.write_checkpoint(str(tmp_path / name), cfg, W), dtype=dtype, kv_pool_tokens=tokens, max_seqs=seqs)


def _ids(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).numpy().astype(np.int32)


def _oracle(cfg, W, ids, streams=False):
    lg, st = O.forward(cfg, H.as_f64(W), ids)
    return (lg, st) if streams else lg


def _whole(lm, ids):
    c = lm.make_cache()
    lg = lm.step([(c[0]._seq, ids)], want="all").cpu()
    c[0]._seq.release()
    return lg


def _portions(lm, ids, sizes):
    """the prompt in portions of the given sizes (cycled), every row's logits"""
    c, out, o, j = lm.make_cache(), [], 0, 0
    while o < len(ids):
        n = min(sizes[j % len(sizes)], len(ids) - o)
        out.append(lm.step([(c[0]._seq, ids[o:o + n])], want="all").cpu())
        o, j = o + n, j + 1
    c[0]._seq.release()
    return torch.cat(out)


def _segments(lens, slots, pos0):
    """the tables of a ragged step"""
    i32 = torch.int32
    cu = torch.tensor([0] + list(np.cumsum(lens)), dtype=i32).cuda()
    tok_seq = torch.cat([torch.full((n,), s, dtype=i32) for n, s in zip(lens, slots)]).cuda()
    tok_pos = torch.cat([torch.arange(p, p + n, dtype=i32) for n, p in zip(lens, pos0)]).cuda()
    return tok_seq, tok_pos, cu, torch.tensor(slots, dtype=i32).cuda(), torch.tensor(pos0, dtype=i32).cuda()


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
@pytest.mark.parametrize("S", [1, 2, 3, 5, 8])
@pytest.mark.parametrize("D", [52, 51, 1280])
def test_hyper_step_writes_all_streams_from_the_old_ones_and_norms_the_read(S, D):
    from mlx_vlm_amd import ops

    g = torch.Generator().manual_seed(S * D)
    for T in (torch.float32, torch.bfloat16):
        X, y = torch.randn(7, S, D, generator=g), torch.randn(7, D + 4, generator=g).to(T)
        mix, out, inn = torch.randn(S, S, generator=g), torch.randn(S, generator=g), torch.randn(S, generator=g)
        w = (1 + 0.3 * torch.randn(D, generator=g)).to(T)
        new = O.hyper_write(X.double().transpose(0, 1), y.double()[:, :D], mix.double(), out.double())
        h_want = O.rms(O.hyper_read(new, inn.double()), 1e-3) * w.double()
        kw = dict(y=y.cuda()[:, :D], mix=mix.cuda(), out=out.cuda(), w_in=inn.cuda(), w=w.cuda(), eps=1e-3)
        tol = 3e-5 if T == torch.float32 else 4e-2
        Xd = X.cuda()
        h = ops.hyper_step(Xd, S, **kw)                                              # in place
        assert h.dtype == T and (h.cpu().double() - h_want).abs().max() < tol
        assert (Xd.cpu().double() - new.transpose(0, 1)).abs().max() < 3e-5
        # one row that stands for all streams, then the same written out
        row = X[:, 0].contiguous()
        new1 = O.hyper_write(row.double()[None].repeat(S, 1, 1), y.double()[:, :D], mix.double(), out.double())
        Xo = torch.full((7, S, D), float("nan")).cuda()
        h = ops.hyper_step(row.cuda(), S, xout=Xo, **kw)
        assert (Xo.cpu().double() - new1.transpose(0, 1)).abs().max() < 3e-5
        assert (h.cpu().double() - O.rms(O.hyper_read(new1, inn.double()), 1e-3) * w.double()).abs().max() < tol
        # read only (streams untouched), the plain sum, write only
        before = Xo.clone()
        h = ops.hyper_step(Xo, S, w=w.cuda(), eps=1e-3)
        assert torch.equal(Xo, before) and (h.cpu().double() - O.rms(new1.sum(0), 1e-3) * w.double()).abs().max() < tol
        assert ops.hyper_step(Xo, S, y=y.cuda()[:, :D], mix=mix.cuda(), out=out.cuda()) is None
        assert (Xo.cpu().double() - O.hyper_write(before.cpu().double().transpose(0, 1), y.double()[:, :D], mix.double(), out.double())
                .transpose(0, 1)).abs().max() < 1e-4


@pytest.mark.parametrize("taps", [0, 1, 3, 7])
@pytest.mark.parametrize("T", [torch.float32, torch.bfloat16])
def test_convolved_rotated_rows_across_portions_pages_and_reused_slots(T, taps):
    """three sequences in portions down to one token, two of them side by side in one launch, positions beyond a page; then a new
    sequence in a slot whose carry still holds the old one's inputs"""
    from mlx_vlm_amd import ops
    from mlx_vlm_amd.models.cache import PAGE
    from mlx_vlm_amd.models.zivitar.config import rotation

    g = torch.Generator().manual_seed(taps)
    HQ, HK, D, NV = 6, 2, 10, 14
    offs = (0, 64, 88)
    C = 104
    for rot in (dict(base=50.0, dims=6, scaling=H.YARN), dict(base=30.0, dims=10), None):
        dims, f, amp = rotation(rot)
        inv = torch.from_numpy(f).cuda() if f is not None else None
        w = (0.5 * torch.randn(C, taps, generator=g)).to(T) if taps else None
        seqs = {s: torch.randn(n, C + 8, generator=g).to(T) for s, n in ((0, 99), (2, 71), (1, 5))}
        carry = torch.full((3, taps - 1, C), float("nan")).cuda() if taps > 1 else None
        bt = (torch.randperm(6, generator=g).to(torch.int32) + 1).view(3, 2).contiguous()
        kpool = torch.zeros(7, PAGE, ops.diff_key_width(HK, D, T == torch.bfloat16), dtype=T).cuda()
        vpool = torch.zeros(7, PAGE, NV, dtype=T).cuda()

        def reference(x):
            y = O.causal_conv(x.double()[:, :C], w.double()) if taps else x.double()[:, :C]
            n = y.shape[0]
            turn = lambda z, h: O.rotate_half(z.reshape(n, h, D), rot).reshape(n, h * D)          # noqa: E731
            return turn(y[:, : HQ * D], HQ), turn(y[:, 64: 64 + HK * D], HK), y[:, 88: 88 + NV]
        want = {s: reference(x) for s, x in seqs.items()}
        got, at = {s: [] for s in seqs}, {s: 0 for s in seqs}

        def launch(step, src):
            lens, slots, pos0 = [n for _, n in step], [s for s, _ in step], [at[s] for s, _ in step]
            rows = torch.cat([src[s][at[s]: at[s] + n] for s, n in step]).cuda()
            q = torch.empty(rows.shape[0], HQ * D).cuda()
            ops.conv_qkv_rows(rows[:, :C], None if w is None else w.cuda(), carry, offs, HQ, HK, D, NV, *_segments(lens, slots, pos0), bt.cuda(),
                              q, kpool, vpool, rot_dims=dims, inv_freq=inv, amp=amp)
            o = 0
            for s, n in step:
                got[s].append(q[o:o + n].cpu())
                o, at[s] = o + n, at[s] + n
        for step in ([(0, 5)], [(0, 1), (2, 3)], [(2, 1), (0, 1)], [(0, 2), (2, 7)], [(0, 90), (1, 5)], [(2, 60)]):
            launch(step, seqs)
        tol = 2e-5 if T == torch.float32 else 5e-3
        for s, x in seqs.items():
            q, k, v = want[s]
            kp = _joined_rows(kpool[bt[s].long()].cpu(), HK, D).reshape(-1, HK * D)[: len(x)]
            vp = vpool[bt[s].long()].reshape(-1, NV)[: len(x)].cpu().double()
            assert (torch.cat(got[s]).double() - q).abs().max() < 2e-5, s          # fp32 from the projected row on, whatever T is
            assert ((kp - k).abs() <= 2e-5 + 2.0 ** -16 * k.abs()).all() and ((vp - v).abs() <= tol * (1e-2 + v.abs())).all(), s
        got[0], at[0] = [], 0                                                       # slot 0 again, from position 0
        launch([(0, 4)], {0: seqs[2]})
        assert (torch.cat(got[0]).double() - want[2][0][:4]).abs().max() < 2e-5


@pytest.mark.parametrize("D,Dv,Hh,G", [(12, 20, 6, 2), (16, 16, 2, 2), (6, 33, 3, 1), (40, 72, 20, 1), (64, 128, 6, 2), (72, 136, 4, 2), (1, 1, 1, 1),
                                       (18, 256, 2, 1), (256, 256, 1, 1), (320, 24, 2, 1)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_differential_attention_against_dense_maps(dtype, D, Dv, Hh, G):
    """two sequences at different offsets on scattered pages (one 1890 tokens deep), windows with and without kept tokens, both forms"""
    from mlx_vlm_amd import ops
    from mlx_vlm_amd.models.cache import PAGE

    g = torch.Generator().manual_seed(D + Dv)
    bt = torch.zeros(3, 32, dtype=torch.int32)
    bt[1, :31] = torch.randperm(31, generator=g).to(torch.int32) + 1
    kpool = torch.randn(32, PAGE, G * 2 * D, generator=g) * 0.7
    vpool = torch.randn(32, PAGE, G * Dv, generator=g).to(dtype)
    tok_seq = torch.tensor([1] * 37 + [2] * 5, dtype=torch.int32)
    tok_pos = torch.tensor(list(range(1890, 1927)) + list(range(5)), dtype=torch.int32)
    q = torch.randn(42, Hh * 2 * D, generator=g)
    qb_start = torch.tensor([0, 16, 32, 37], dtype=torch.int32).cuda()
    qb_count = torch.tensor([16, 16, 5, 5], dtype=torch.int32).cuda()
    pool = kpool if dtype == torch.float32 else _split_rows(kpool, G * 2, D)
    kpool = _joined_rows(pool, G * 2, D)
    rows = {sq: (kpool[bt[sq].long()].reshape(-1, G, 2, D).double(), vpool[bt[sq].long()].reshape(-1, G, Dv).double()) for sq in (1, 2)}
    qd = q.double().view(42, Hh, 2, D)
    for window, keep, scale, lam, diff in ((0, 0, 1.0, 0.7, 0.6), (17, 0, 1.0, 0.3, 0.2), (17, 4, 2.0, 0.9, 0.5), (1025, 70, 0.5, 1.2, 0.8),
                                           (1, 1, 1.0, -0.4, 0.0), (900, 1888, 1.0, 0.5, 0.3), (64, 16, 1.0, 0.0, 0.4)):
        scale = scale / max(D, 4) ** 0.5
        want = torch.zeros(42, Hh, Dv, dtype=F64)
        for t in range(42):
            sq, pos = int(tok_seq[t]), int(tok_pos[t])
            seen = O.visible(pos + 1, window if window > 0 else None, keep)[pos].nonzero().flatten()
            for h in range(Hh):
                kh = h // (Hh // G)
                a = [torch.softmax(rows[sq][0][seen, kh, m] @ qd[t, h, m] * scale, dim=0) @ rows[sq][1][seen, kh] for m in (0, 1)]
                want[t, h] = O.rms(a[0] - lam * a[1], 1e-5) * (1.0 - diff)
        args = (tok_seq.cuda(), tok_pos.cuda(), bt.cuda(), Hh, G, D, Dv, scale, lam, 1.0 - diff, 1e-5)
        a, b = (torch.full((42, Hh * Dv + 8), float("nan"), dtype=dtype, device="cuda")[:, : Hh * Dv] for _ in range(2))
        ops.diff_attn_blocks(q.cuda(), pool.cuda(), vpool.cuda(), qb_start, qb_count, *args, b, window=window, keep=keep)
        tol = 1e-4 if dtype == torch.float32 else 2e-2                              # (the norm magnifies what the difference cancels)
        for nsplit in (None, 1, 2, 7, 64):                                          # workgroups that share a column group's keys
            ops.diff_attn_rows(q.cuda(), pool.cuda(), vpool.cuda(), *args, a, window=window, keep=keep, nsplit=nsplit)
            assert (a.cpu().double().view(42, Hh, Dv) - want).abs().max() < tol, (window, keep, nsplit)
        assert (b.cpu().double().view(42, Hh, Dv) - want).abs().max() < tol, (window, keep)


@pytest.mark.parametrize("Hh,D,Dv", [(3, 10, 14), (1, 72, 136), (2, 33, 5), (7, 1, 1), (2, 128, 128), (2, 64, 32), (3, 64, 64), (1, 160, 48)])
@pytest.mark.parametrize("T", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("room", [0, 1, 3, 100])
def test_fixed_decay_recurrence_in_portions_and_reused_slots(T, Hh, D, Dv, room):
    """room: chunks the workspace of the chunk-parallel form holds (0: token by token; fewer than the step has: windows of chunks)"""
    from mlx_vlm_amd import _lib, ops

    g = torch.Generator().manual_seed(D + Dv)
    n = 333
    qkvg = {c: torch.randn(n, Hh * k + 3, generator=g).to(T) for c, k in (("q", D), ("k", D), ("v", Dv), ("g", Dv))}
    decay = torch.tensor([(0.05, 0.999, 0.9, 1.0, 0.5, 0.99, 0.0)[h] for h in range(Hh)])
    w = (1 + 0.3 * torch.randn(Hh * Dv, generator=g)).to(T)
    val = {c: t.double()[:, : Hh * k].reshape(n, Hh, k) for (c, t), k in zip(qkvg.items(), (D, D, Dv, Dv))}
    raw_want = O.fixed_decay_recurrence(O.silu(val["q"]), O.silu(val["k"]), O.silu(val["v"]), decay.double())
    want = O.rms(raw_want.reshape(n, Hh * Dv), 1e-4) * w.double() * torch.sigmoid(val["g"].reshape(n, -1))
    state = torch.full((3, Hh, D, Dv), float("nan")).cuda()

    def run(parts):
        """parts: [(slot, lo, hi)] side by side in one launch"""
        rows = {c: torch.cat([t[lo:hi] for _, lo, hi in parts]).cuda() for c, t in qkvg.items()}
        ntok = rows["q"].shape[0]
        out, raw = torch.empty(ntok, Hh * Dv, dtype=T, device="cuda"), torch.empty(ntok, Hh, Dv, device="cuda")
        keep = [decay.cuda(), w.cuda()]
        _, _, cu, sl, p0 = _segments([hi - lo for _, lo, hi in parts], [s for s, _, _ in parts], [lo for _, lo, _ in parts])
        a = _lib.RecurrenceArgs()
        a.q, a.k, a.v, a.g = (rows[c].data_ptr() for c in "qkvg")
        a.ldq, a.ldk, a.ldv, a.ldg = (rows[c].stride(0) for c in "qkvg")
        a.gated, a.q_act, a.k_act, a.v_act, a.qscale, a.kscale = 0, 1, 1, 1, 1.0, 1.0
        a.decay, a.normw, a.gate_act, a.row_norm, a.eps = keep[0].data_ptr(), keep[1].data_ptr(), 1, 1, 1e-4
        a.seg_start, a.seg_slot, a.seg_pos0 = cu.data_ptr(), sl.data_ptr(), p0.data_ptr()
        a.state, a.raw, a.out, a.ldo = state.data_ptr(), raw.data_ptr(), out.data_ptr(), out.stride(0)
        a.H, a.D, a.Dv = Hh, D, Dv
        ws = torch.full((max(room, 1) * Hh * D * Dv,), float("nan"), device="cuda")
        if room:
            a.ws, a.ws_floats = ws.data_ptr(), ws.numel()
        ops.linear_recurrence(a, len(parts), ntok, T == torch.float32)
        torch.cuda.synchronize()
        return out.float().cpu()
    scale = want.abs().max()
    tol = (3e-5 if T == torch.float32 else 1e-2) * scale
    whole = run([(1, 0, n)])
    assert (whole.double() - want).abs().max() < tol
    cuts = [0, 1, 3, 17, 18, 20, 84, 148, 213, 300, n]
    parts = torch.cat([run([(2, a, b)]) for a, b in zip(cuts, cuts[1:])])
    assert (parts.double() - want).abs().max() < tol
    assert torch.equal(run([(2, 0, n)]), whole)                         # a used slot, from position 0
    # three sequences side by side: a decoded token next to portions, all from the same tokens at different depths
    run([(0, 0, 150)]), run([(1, 0, 40)]), run([(2, 0, 299)])
    both = run([(0, 150, 290), (1, 40, 41), (2, 299, n)])
    assert (both.double() - torch.cat([want[150:290], want[40:41], want[299:n]])).abs().max() < tol
    S = torch.zeros(Hh, D, Dv, dtype=F64)
    for t in range(n):
        S = decay.double()[:, None, None] * S + O.silu(val["k"][t])[:, :, None] * O.silu(val["v"][t])[:, None, :]
    assert (state[2].cpu().double() - S).abs().max() < 3e-5 * S.abs().max().clamp_min(1.0)


@pytest.mark.parametrize("dim", [24, 23])
def test_clamped_gated_unit_and_capped_logits(dim):
    from mlx_vlm_amd import ops

    g = torch.Generator().manual_seed(5)
    for T in (torch.float32, torch.bfloat16):
        gu = (3 * torch.randn(9, 64, generator=g)).to(T)
        for limit in (0.5, 2.0, float("inf")):
            out = torch.zeros(9, 32, dtype=T, device="cuda")
            ops.glu_rows(gu.cuda(), gu.cuda()[:, 32:], ops.GLU_CLAMPED, out=out[:, :dim], limit=limit)
            want = O.clamped_glu(gu.double()[:, :dim], gu.double()[:, 32: 32 + dim], limit)
            assert (out[:, :dim].cpu().double() - want).abs().max() < (1e-5 if T == torch.float32 else 3e-2) * want.abs().max() and torch.all(out[:, dim:] == 0)
        x = gu[:, :dim].clone()
        for cap in (0.0, 2.5):
            want = 0.3 * x.double() if not cap else cap * torch.tanh(0.3 * x.double() / cap)
            o = torch.zeros(9, dim, device="cuda")
            ops.logit_cap_rows(x.cuda(), 0.3, cap, out=o)
            assert (o.cpu().double() - want).abs().max() < 1e-5
            y = x.cuda()
            ops.logit_cap_rows(y, 0.3, cap)
            assert (y.cpu().double() - want).abs().max() < (1e-5 if T == torch.float32 else 2e-2)


# ------------------------------------------------------------------------------------------------ one-layer models
ONE = {"lightning": [H.lightning()], "lightning_one_wide_head_no_ff": [H.lightning(heads=1, dim=72, vdim=136, mlp=None)],
       "lightning_many_small_heads": [H.lightning(heads=7, dim=3, vdim=5, mlp=H.dense(8, 0.3))],
       "lightning_wide": [H.lightning(heads=2, dim=128, vdim=64, mlp=H.dense(96, 7.0))],
       "attention": [H.attention()], "attention_equal_heads_no_rotation": [H.attention(heads=3, kv_heads=3, rot_dims=0, mlp=None)],
       "attention_one_kv_head_full_rotation": [H.attention(heads=5, kv_heads=1, dim=12, vdim=12, rot_dims=12, size=64, keep=64)],
       "attention_no_window_no_scaling": [H.attention(size=0, scaling=None, conv=5)],
       "attention_window_1_one_tap": [H.attention(size=1, keep=1, conv=1, heads=1, kv_heads=1, dim=2, vdim=1, rot_dims=2)],
       "attention_no_convolution": [H.attention(conv=0, diff=0.0)],
       "attention_wide": [H.attention(heads=2, kv_heads=1, dim=64, vdim=128, rot_dims=32, base=10000.0, size=100, keep=5)]}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", sorted(ONE))
def test_each_mixer_alone(tmp_path, kind, dtype):
    cfg = H.config(ONE[kind], streams=1 if "one_tap" in kind else (4 if "wide" in kind else 2), cap=0.0 if "equal" in kind else 5.0,
                   logit_scale=1.0 if "equal" in kind else 0.7)
    W = H.weights(cfg, seed=3)
    ids = _ids(150, cfg["vocab"], 5)
    lm = _load(tmp_path, cfg, W, dtype, tokens=512).language_model
    want = _oracle(cfg, W, ids)
    assert _close(_whole(lm, ids), want, dtype)
    assert _close(_portions(lm, ids, [70, 1, 2, 30]), want, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layers_match_layer_by_layer_with_borrowed_tensors(tmp_path, dtype):
    cfg = H.mixed_config()
    W = H.weights(cfg, seed=11)
    ids = _ids(90, cfg["vocab"], 6)
    lm = _load(tmp_path, cfg, W, dtype, tokens=512).language_model
    lm._trace = []
    c = lm.make_cache()
    lm.step([(c[0]._seq, ids)], want="all")
    _, ref = _oracle(cfg, W, ids, streams=True)
    assert len(lm._trace) == len(ref) == 8 and len(c) == 8
    for i, (a, b) in enumerate(zip(lm._trace, ref)):
        assert _close(a.cpu(), b, dtype), i
    lm._trace = None
    c[0]._seq.release()


def test_without_streams_the_residual_is_a_plain_sum(tmp_path):
    """a config that names no streams: the same logits as one stream whose weights are all one"""
    cfg = H.config([H.lightning(), H.attention()], streams=1)
    W = H.weights(cfg, seed=4)
    for k in list(W):
        if ".hc" in k:
            W[k] = torch.ones_like(W[k])
    ids = _ids(40, cfg["vocab"], 2)
    want = _oracle(cfg, W, ids)
    plain = {k: v for k, v in cfg.items() if k != "streams"}
    lm = _load(tmp_path, plain, {k: v for k, v in W.items() if ".hc" not in k}, "float32", tokens=256).language_model
    assert _close(_whole(lm, ids), want, "float32")


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


def test_unequal_batch_equals_each_alone_and_pages_and_slots_are_reused(mixed32):
    cfg, W, lm = mixed32
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
    for i in range(len(reqs)):
        assert H.rel_rms(torch.cat(got[i]), alone[i]) < TOL["float32"], i
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
    cfg = H.config([H.lightning(), H.attention()])
    lm = _load(tmp_path, cfg, H.weights(cfg, seed=1), "float32", tokens=128, seqs=2).language_model
    c = lm.make_cache()
    lm.step([(c[0]._seq, _ids(128, cfg["vocab"], 1))])
    with pytest.raises(RuntimeError):
        lm.step([(c[0]._seq, _ids(1, cfg["vocab"], 2))])
    c[0]._seq.release()
    c = lm.make_cache()
    lm.step([(c[0]._seq, _ids(100, cfg["vocab"], 3))])
    c[0]._seq.release()


# ------------------------------------------------------------------------------------------------ edges made visible
def _marked(W, G, D):
    """token 1 (`mark`) lives on stream direction 0 alone, token 2 (the asking token) on direction 1 alone; no other token has
    a component along either.  The convolution passes the current token only (the kernel still runs and carries).  The key of
    `mark` and the query of the asking token point along one direction of map 1; every other key leans away from it."""
    emb = W["embed"].float()
    emb[:, :2] = 0
    emb[1], emb[2] = 0, 0
    emb[1, 0], emb[2, 1] = 4.0, 4.0
    W["embed"] = emb.to(torch.bfloat16)
    p = "l0.mix."
    for n in "qkv":
        w = torch.zeros_like(W[p + n + ".conv"])
        w[:, -1] = 1.0
        W[p + n + ".conv"] = w
    k, q = W[p + "k"].float().view(G, 2, D, -1), W[p + "q"].float().view(-1, 2, D, W[p + "q"].shape[1])
    k[:, 0] *= 0.3
    q[:, 0, :, 1], k[:, 0, :, 0] = 0.0, 0.0
    q[:, 0, -1, 1], k[:, 0, -1, 0] = 3.0, 3.0              # the last dimension of map 1: not rotated
    W[p + "k"], W[p + "q"] = k.reshape(W[p + "k"].shape).to(torch.bfloat16), q.reshape(W[p + "q"].shape).to(torch.bfloat16)


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
@pytest.mark.parametrize("window,keep", [(1, 0), (2, 3), (16, 1), (17, 16), (64, 4), (65, 17), (130, 64)])
def test_window_edge_and_kept_tokens_in_prompt_and_decoding(tmp_path, window, keep, dtype):
    """token `mark` appears once: at distance window - 1 (just inside) or window (just outside) of the asked position, or as the last
    kept token (in view from anywhere) or the one after it, and its key towers over all others.  Whole prompt, portions cut at
    the edge and at the asked token, and decoding token by token must agree with the oracle."""
    cfg = H.config([H.attention(heads=2, kv_heads=1, dim=8, vdim=12, scale=1.0, size=window, keep=keep, rot_dims=4, mlp=None)], width=48, vocab=64,
                   streams=2)
    W = H.weights(cfg, seed=5)
    _marked(W, 1, 8)
    lm = _load(tmp_path, cfg, W, dtype, tokens=1024).language_model
    n = 2 * window + keep + 70
    for ask in (window + keep + 3, n - 1):
        for at in sorted({ask - window + 1, ask - window, 0, keep - 1, keep}):
            if not 0 <= at < ask:
                continue
            _check_probe(lm, cfg, W, dtype, n, ask, at, ask - at < window or at < keep,
                         ([n], [at + 1, 1000], [ask, 1], [ask - 1, 2], [at, 1, 1000], [3, 1]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_far_key_among_hundreds_and_at_page_borders(tmp_path, dtype):
    """causal attention: one key whose score towers over all others, at the first positions, around page borders and hundreds of
    tokens back; seen from its own position's successor and from far away, in a prompt, at a portion's first token and decoded"""
    cfg = H.config([H.attention(heads=2, kv_heads=1, dim=16, vdim=16, scale=1.5, size=0, rot_dims=2, mlp=None)], width=48, vocab=64)
    W = H.weights(cfg, seed=5)
    _marked(W, 1, 16)
    lm = _load(tmp_path, cfg, W, dtype, tokens=1024).language_model
    n = 700
    for at in (0, 1, 63, 64, 65, 255, 256, 511, 640):
        for ask in sorted({at + 1, min(at + 130, n - 1), n - 1}):
            _check_probe(lm, cfg, W, dtype, n, ask, at, True, ([n], [at + 1, 1000], [ask, 1], [ask - 1, 2]) + (([at, 1, 1000],) if at else ()))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_recurrent_states_remember_hundreds_of_tokens(tmp_path, dtype):
    """decays near one: tokens 40..43 still move the logits 300 and 650 tokens later - whole, in portions, and decoded from a state
    that crossed many steps"""
    cfg = H.config([H.lightning(heads=2, dim=8, vdim=8, decay=[0.9995, 1.0], mlp=None), H.lightning(heads=3, dim=8, vdim=4, decay=[0.999, 0.5, 0.9999], mlp=None)],
                   width=48, vocab=64)
    W = H.weights(cfg, seed=7)
    n = 700
    ids = _ids(n, cfg["vocab"], 3)
    want = _oracle(cfg, W, ids)
    other = ids.copy()
    other[40:44] = (other[40:44] + 9) % cfg["vocab"]
    moved = _oracle(cfg, W, other)
    for ask in (340, 699):
        assert H.rel_rms(moved[ask:ask + 1], want[ask:ask + 1]) > 2e-3, ask
    lm = _load(tmp_path, cfg, W, dtype, tokens=1024).language_model
    for sizes in ([n], [44, 1000], [41, 2, 300, 1], [64], [600] + [1] * 100):
        got = _portions(lm, ids, sizes)
        assert H.rel_rms(got, want) < 1e-4 if dtype == "float32" else _close(got, want, dtype), sizes
        assert H.rel_rms(got[[340, 699]], want[[340, 699]]) < 2.5 * TOL[dtype], sizes


def test_first_tokens_and_a_one_token_request(mixed32):
    cfg, W, lm = mixed32
    for n in (1, 2, 3, 4, 5):                                       # shorter than the windows and the convolutions
        ids = _ids(n, cfg["vocab"], 90 + n)
        want = _oracle(cfg, W, ids)
        assert H.rel_rms(_whole(lm, ids), want) < TOL["float32"]
        assert H.rel_rms(_portions(lm, ids, [1]), want) < TOL["float32"]


def test_long_decoding_crosses_pages_and_windows(tmp_path):
    cfg = H.config([H.attention(size=70, keep=3), H.lightning(), H.attention(size=0, mlp=None), H.attention(size=5, keep=20, weights_of=0)])
    W = H.weights(cfg, seed=17)
    ids = _ids(400, cfg["vocab"], 19)
    want = _oracle(cfg, W, ids)
    for dtype in ("float32", "bfloat16"):
        lm = _load(tmp_path, cfg, W, dtype, tokens=1024, name=dtype).language_model
        got = _portions(lm, ids, [20] + [1] * 380)
        assert _close(got, want, dtype)
        assert H.rel_rms(got[-1:], want[-1:]) < 2.5 * TOL[dtype]


def test_other_sizes(tmp_path):
    """widths, head sizes and feed-forward sizes that are not multiples of 8, an odd vocabulary, one stream and five, more than sixteen
    heads on one key head, a window beyond the prompt, everything kept, one rotated pair, a limit so wide that nothing is cut"""
    layers = [H.attention(heads=18, kv_heads=1, dim=5, vdim=7, scale=0.7, size=1000, keep=3, rot_dims=2, base=7.0, conv=2, mlp=H.dense(37, 100.0)),
              H.lightning(heads=5, dim=9, vdim=11, mlp=H.dense(19, 0.1)),
              H.attention(heads=5, kv_heads=5, dim=6, vdim=9, size=3, keep=1000, rot_dims=6, conv=6, mlp=H.dense(11, 1.0)),
              H.lightning(heads=1, dim=1, vdim=1, mlp=None)]
    for streams in (1, 5):
        cfg = H.config(layers, vocab=301, width=61, eps=3e-4, streams=streams, logit_scale=2.0, cap=3.0)
        W = H.weights(cfg, seed=23)
        ids = _ids(100, cfg["vocab"], 29)
        want = _oracle(cfg, W, ids)
        for dtype in ("float32", "bfloat16"):
            lm = _load(tmp_path, cfg, W, dtype, tokens=256, name=f"{dtype}{streams}").language_model
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

    cfg = H.config(H.mixed_layers()[:5], cap=40.0)                  # a wide cap: greedy choices survive bf16 logits
    W = H.weights(cfg, seed=51)
    W["head"] = (W["head"].float() * 3).to(torch.bfloat16)
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
        got = [t for t, _ in generate_step(p[None], model, None, None, max_tokens=12, temperature=0.0)]
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
    cfg = H.config(H.mixed_layers()[:4])
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


def test_captured_decode_steps_equal_eager_ones(tmp_path):
    """a captured decode step is replayed many times, with eager work (another request's prompt, a release, synchronisations)
    between the replays; every replay's logits and token must equal the eager step's"""
    from mlx_vlm_amd.sample_utils import make_sampler

    cfg = H.mixed_config()
    W = H.weights(cfg, seed=71)
    lm = _load(tmp_path, cfg, W, "bfloat16", tokens=2048, seqs=6).language_model
    sargs = make_sampler().engine_args()
    prompts = [_ids(n, cfg["vocab"], 80 + n) for n in (40, 7, 66)]

    def run(use_graph):
        caches = lm.make_cache_batch(3)
        lg = lm.prefill(torch.cat([torch.as_tensor(p) for p in prompts]).cuda().reshape(-1, 1), None, caches, [len(p) for p in prompts])
        st = lm.decode_begin(caches, lg.argmax(-1), np.zeros((3, 1)), max_new_tokens=80)
        out = []
        for i in range(70):                                          # crosses a page border and the windows in every row
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
