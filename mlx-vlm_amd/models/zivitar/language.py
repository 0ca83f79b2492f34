"""Zivitar language model on the HIP operator library (the ragged step of models/ragged.py).

The residual is S fp32 streams per token, [T, S, width].  A sublayer boundary is ONE kernel: the previous sublayer's result y is
written back (new stream t = sum_s mix[s, t] x_s + out[t] y), the next sublayer's input sum_s in[s] x_s is formed and RMS-normed into
the serving dtype.  The embedding rows stand for all S streams until the first write.
    proj = h @ [mixer projections]^T                                     one GEMM (rows packed at load)
    lightning : fixed-decay matrix-state recurrence on silu(q), silu(k), silu(v), state fp32 per sequence; RMS norm over all heads of a
                token with a weight, times sigmoid(g); W_o
    attention : short causal convolution over the packed [q | k | v] columns (projected values carried per sequence), rotate-half
                positions on the first rot dims of every map, keys (fp32 precision) and values into the paged caches - one kernel; differential
                softmax attention inside a window that keeps the first tokens in view, difference normed per head - one kernel; W_o
    dense     : [gate | up] in one GEMM, clamped gated activation, W_down
Final norm of the summed streams at the wanted rows, logits = cap tanh(scale (rows @ head^T) / cap).  A layer with `weights_of` uses
another layer's tensors with a cache / state of its own.
"""
from __future__ import annotations

from types import SimpleNamespace
from typing import Dict

import torch

from ... import _lib, ops
from ..cache import HybridPool, PagedSequence, RecurrentCache
from ..ragged import RaggedLanguageModel, _al8, pack_rows
from .config import ModelConfig, rotation


class LanguageModel(RaggedLanguageModel):
    NAME = "Zivitar"
    ROWS_FORM = 8          # steps of up to this many tokens run the decode form of the attention

    def __init__(self, config: ModelConfig, **kwargs):
        super().__init__(config, **kwargs)

    # ------------------------------------------------------------------ weights
    def load_weights(self, W: Dict[str, torch.Tensor]):
        cfg, dev, T = self.config, self.device, self.dtype
        f32 = torch.float32
        Wd, eps = cfg.width, cfg.norm_eps
        S = self._S = max(1, cfg.streams)

        def g(name, shape, dtype=None):
            if name not in W:
                raise KeyError(f"Zivitar checkpoint: tensor {name!r} missing")
            t = W[name]
            if tuple(t.shape) != tuple(shape):
                raise ValueError(f"Zivitar checkpoint: {name} is {tuple(t.shape)}, the config says {tuple(shape)}")
            return t.to(device=dev, dtype=dtype or T).contiguous()

        def hyper(p):            # stream weights of a sublayer; without streams the plain residual step
            if not cfg.streams:
                one = torch.ones(1, dtype=f32, device=dev)
                return SimpleNamespace(inn=one, out=one, mix=one.view(1, 1))
            return SimpleNamespace(inn=g(p + "in", (S,), f32), out=g(p + "out", (S,), f32), mix=g(p + "mix", (S, S), f32))

        self._w = dict(embed=g("embed", (cfg.vocab, Wd)), final_norm=g("final.norm", (Wd,)), head=g("head", (cfg.vocab, Wd)))
        owners = {}
        for i, L in enumerate(cfg.layers):
            if L.weights_of is not None:
                continue
            p, m = f"l{i}.", L.mixer
            H, D, Dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
            ns = dict(norm1=g(p + "norm1", (Wd,)), hc1=hyper(p + "hc1."), wo=g(p + "mix.o", (Wd, H * Dv)))
            if L.type == "lightning":
                parts = [("q", g(p + "mix.q", (H * D, Wd))), ("k", g(p + "mix.k", (H * D, Wd))), ("v", g(p + "mix.v", (H * Dv, Wd))),
                         ("g", g(p + "mix.g", (H * Dv, Wd)))]
                ns["normw"] = g(p + "mix.norm", (H * Dv,))
            else:
                G, taps = int(m["kv_heads"]), L.taps
                rows = (("q", H * 2 * D), ("k", G * 2 * D), ("v", G * Dv))
                parts = [(n, g(p + "mix." + n, (r, Wd))) for n, r in rows]
                # one filter per packed projection row (padding rows: zeros)
                ns["conv"] = pack_rows([(n, g(p + f"mix.{n}.conv", (r, taps))) for n, r in rows], T, dev)[0] if taps else None
                lq1, lk1, lq2, lk2 = (g(p + "mix." + n, (D,), torch.float64).cpu() for n in ("lq1", "lk1", "lq2", "lk2"))
                ns["lam0"] = float(torch.exp((lq1 * lk1).sum()) - torch.exp((lq2 * lk2).sum()))
            ns["wproj"], ns["off"] = pack_rows(parts, T, dev)
            if L.mlp is not None:
                ns.update(norm2=g(p + "norm2", (Wd,)), hc2=hyper(p + "hc2."))
                ns["wff"], ns["foff"] = pack_rows([(n, g(p + "mlp." + n, (L.ff, Wd))) for n in ("gate", "up")], T, dev)
                ns["down"] = g(p + "mlp.down", (Wd, L.ff))
            owners[i] = ns
        self._L, rows, states, aux = [], {}, {}, {}
        for i, L in enumerate(cfg.layers):
            ns, m = SimpleNamespace(type=L.type, **owners[i if L.weights_of is None else L.weights_of]), L.mixer
            ns.H, ns.D, ns.Dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
            ns.ff, ns.limit = L.ff, L.limit
            if L.type == "lightning":
                ns.decay = torch.tensor([float(x) for x in m["decay"]], dtype=f32, device=dev)
                states[i] = (ns.H, ns.D, ns.Dv, False)
            else:
                ns.G, ns.scale, ns.diff, ns.taps = int(m["kv_heads"]), float(m["scale"]), float(m["diff"]), L.taps
                ns.lam = ns.lam0 + ns.diff
                ns.window, ns.keep = L.window
                ns.rot_dims, f, ns.amp = rotation(m.get("rot"))
                ns.inv_freq = torch.from_numpy(f).to(dev) if f is not None else None
                # rotated keys: fp32, or two bf16 values per coordinate (the same bytes)
                rows[(i, "k")] = (ops.diff_key_width(ns.G * 2, ns.D, T == torch.bfloat16), T)
                rows[(i, "v")] = (ns.G * ns.Dv, T)
                if ns.taps > 1:
                    aux[(i, "conv")] = (ns.taps - 1, ns.wproj.shape[0])
            self._L.append(ns)
        self.pool = HybridPool(len(self._L), rows, states, self._kv_pool_tokens, self._max_seqs, device=dev, dtype=T, aux_layers=aux)
        return self

    # ------------------------------------------------------------------ cache
    def make_cache(self):
        seq = PagedSequence(self.pool)
        # (attention layers carry convolution inputs beside their rows: neither kind of layer can forget its last tokens)
        return [RecurrentCache(seq, i) for i in range(len(self._L))]

    def make_cache_batch(self, n: int):
        return [self.make_cache() for _ in range(n)]

    # ------------------------------------------------------------------ mixers
    def _attention(self, i, ns, proj, pl, keep):
        """-> [tokens, heads * vdim] in the serving dtype: normed differences of the two maps"""
        Tn, H, G, D, Dv, dev, pool = pl.Tn, ns.H, ns.G, ns.D, ns.Dv, self.device, self.pool
        kpool, vpool = pool.rows[(i, "k")], pool.rows[(i, "v")]
        q = torch.empty(Tn, H * 2 * D, dtype=torch.float32, device=dev)
        ops.conv_qkv_rows(proj, ns.conv, pool.aux.get((i, "conv")), (ns.off["q"], ns.off["k"], ns.off["v"]), 2 * H, 2 * G, D, G * Dv,
                          pl.tok_seq, pl.tok_pos, pl.cu, pl.slot, pl.pos0, pool.block_table, q, kpool, vpool, rot_dims=ns.rot_dims,
                          inv_freq=ns.inv_freq, amp=ns.amp)
        out = torch.empty(Tn, _al8(H * Dv), dtype=self.dtype, device=dev)[:, : H * Dv]
        args = (pl.tok_seq, pl.tok_pos, pool.block_table, H, G, D, Dv, ns.scale, ns.lam, 1.0 - ns.diff, self.config.norm_eps, out)
        if Tn <= self.ROWS_FORM:
            ops.diff_attn_rows(q, kpool, vpool, *args, window=ns.window, keep=ns.keep)
        else:
            ops.diff_attn_blocks(q, kpool, vpool, pl.qb_start, pl.qb_count, *args, window=ns.window, keep=ns.keep)
        keep.append(q)
        return out

    def _lightning(self, i, ns, proj, pl, keep):
        """-> [tokens, heads * vdim] in the serving dtype: normed, gated read-outs"""
        Tn, H, D, Dv, dev = pl.Tn, ns.H, ns.D, ns.Dv, self.device
        col = lambda name: proj[:, ns.off[name]:].data_ptr()          # noqa: E731
        raw = torch.empty(Tn, H, Dv, dtype=torch.float32, device=dev)
        out = torch.empty(Tn, _al8(H * Dv), dtype=self.dtype, device=dev)[:, : H * Dv]
        a = _lib.RecurrenceArgs()
        a.q, a.k, a.v, a.g = col("q"), col("k"), col("v"), col("g")
        a.ldq = a.ldk = a.ldv = a.ldg = proj.stride(0)
        a.gated, a.q_act, a.k_act, a.v_act, a.qscale, a.kscale = 0, 1, 1, 1, 1.0, 1.0
        a.decay, a.normw, a.gate_act, a.row_norm, a.eps = ns.decay.data_ptr(), ns.normw.data_ptr(), 1, 1, self.config.norm_eps
        a.seg_start, a.seg_slot, a.seg_pos0 = pl.cu.data_ptr(), pl.slot.data_ptr(), pl.pos0.data_ptr()
        a.state, a.raw, a.out, a.ldo = self.pool.state[i].data_ptr(), raw.data_ptr(), out.data_ptr(), out.stride(0)
        a.H, a.D, a.Dv = H, D, Dv
        ws = self._workspace(pl, H * D * Dv)
        if ws is not None:
            a.ws, a.ws_floats = ws.data_ptr(), ws.numel()
        ops.linear_recurrence(a, pl.nseg, Tn, self.dtype == torch.float32)
        keep += [raw, ws]
        return out

    def _workspace(self, pl, entries):
        """room for the chunk-parallel recurrence of a step with prompt portions: `entries` fp32 values per chunk, up to 256 MB (longer
        prompts run in windows of chunks)"""
        if pl.Tn - pl.nseg < 16:                              # decode rows and short portions only
            return None
        chunks = pl.Tn // 64 + pl.nseg
        return torch.empty(min(chunks, max(1, (64 << 20) // entries)) * entries, dtype=torch.float32, device=self.device)

    # ------------------------------------------------------------------ the device side of a step
    def _run(self, pl, logits_dtype=torch.float32):
        """Nothing here looks at host data that changes between two steps of the same shape, so a decode step can be
        captured once and replayed."""
        cfg, dev, T = self.config, self.device, self.dtype
        eps, Tn, f32, S = cfg.norm_eps, pl.Tn, torch.float32, self._S
        emb = ops.embed_scale_f32(pl.ids, self._w["embed"], 1.0)
        X = torch.empty(Tn, S, cfg.width, dtype=f32, device=dev)
        x = emb                  # what stands for the streams: the embedding rows until the first write, then X
        keep = [pl.md, pl.ids, emb, X]
        pending = None           # (y, stream weights) of a sublayer whose result the next boundary writes back

        def boundary(w_in=None, w=None):
            nonlocal pending, x
            y, hc = pending or (None, None)
            h = ops.hyper_step(x, S, y=y, mix=hc.mix if hc else None, out=hc.out if hc else None, w_in=w_in, w=w, eps=eps,
                               xout=X if hc else None)
            if hc:
                x = X
            pending = None
            return h

        for i, ns in enumerate(self._L):
            h = boundary(ns.hc1.inn, ns.norm1)
            proj = self._linear(h, ns.wproj)
            o = self._lightning(i, ns, proj, pl, keep) if ns.type == "lightning" else self._attention(i, ns, proj, pl, keep)
            pending = (self._linear(o, ns.wo), ns.hc1)
            keep += [h, proj, o, pending]
            if ns.ff:
                h2 = boundary(ns.hc2.inn, ns.norm2)
                gu = self._linear(h2, ns.wff)
                act = torch.empty(Tn, _al8(ns.ff), dtype=T, device=dev)[:, : ns.ff]
                ops.glu_rows(gu, gu[:, ns.foff["up"]:], ops.GLU_CLAMPED, out=act, limit=ns.limit)
                pending = (self._linear(act, ns.down), ns.hc2)
                keep += [h2, gu, act, pending]
            if self._trace is not None:
                boundary()
                self._trace.append(X.sum(dim=1))
        self._keep = keep
        if pl.rows.size == 0:
            if pending:
                boundary()
            return None
        if not pl.all_rows:      # the last write and the head only where logits are wanted
            idx = pl.rows_d.long()
            x = x.index_select(0, idx)
            if pending:
                pending = (pending[0].index_select(0, idx), pending[1])
            X = torch.empty(idx.numel(), S, cfg.width, dtype=f32, device=dev)
        hn = boundary(None, self._w["final_norm"])
        # rows at a pitch of vocab rounded up to 8: 16-byte aligned bf16 rows for the samplers, whatever the vocabulary
        out = torch.empty(hn.shape[0], _al8(cfg.vocab), dtype=logits_dtype, device=dev)[:, : cfg.vocab]
        self._linear(hn, self._w["head"], out=out)
        if cfg.logit_scale != 1.0 or cfg.logit_softcap:
            ops.logit_cap_rows(out, cfg.logit_scale, cfg.logit_softcap)
        return out
