"""Rorovik language model on the HIP operator library (the ragged step of models/ragged.py).

The residual stream x is fp32.  A sublayer is normed before and after, x += m * norm_b(f(norm_a(x))); the step that adds a result also forms
the next reader's input, one kernel:
    x = norm(embed[token])      and the first layer's norm1, one kernel
    attention        : proj = h @ [q | k | v | g]^T (rows packed at load); ONE kernel adds the biases, norms q and k over all their heads, multiplies
                       q by 1 + coef ln(floor((p + 1) / every) + 1), mixes v with the first mixing layer's cached values of the token
                       and writes k and v into the paged caches; grouped softmax attention with distance bias, window, sink and
                       gate - one kernel; W_o
    latent_attention : proj = h @ [dq | dkv]^T; ONE kernel norms the query's latent, and norms / rotates / caches the shared row; W_uq;
                       absorbed form q' = U_k^T q per head straight over the cached rows, sink softmax, U_v per head; W_o
    x += m * norm1b(.)          and norm2 (or the next reader), one kernel
    dense ff  : h2 @ [gate | up]^T, relu(gate + b) * (up + b), W_down (its bias enters in the residual step)
    moe ff    : router logits, softmax scores and choice in one kernel; bf16 prompts: the chosen pairs sorted by expert, gathered [gate | up] products
                with the clamped gate * weight, W_down per pair, summed in the residual step; other steps: ONE GEMM over every expert's
                [gate | up] rows, clamped gate * weight (exact zeros for the experts a token did not choose), ONE GEMM over the
                stacked W_down - the sum over experts is its k loop; identity experts add weight * h2 in the residual step
    x += m * norm2b(.)          and x in the serving dtype, one kernel
    token input: gelu_tanh(x @ side.gate^T) * side.embed[token, layer slice], side.proj
    x += m * rms(.) * side.norm and the next layer's norm1, one kernel
Final norm of the wanted rows, logits = rows @ head^T.
"""
from __future__ import annotations

from types import SimpleNamespace
from typing import Dict

import torch

from ... import ops
from ..cache import HybridPool, PagedSequence, RowCache
from ..ragged import RaggedLanguageModel, _al8, pack_cols, pack_rows, rotation
from .config import ModelConfig


class LanguageModel(RaggedLanguageModel):
    NAME = "Rorovik"
    STATEFUL = False       # row caches only: a step that ran is taken back by moving the cache offset
    ROWS_FORM = 8          # steps of up to this many tokens run the decode form of the attentions
    GROUPED_ROWS = 64      # bf16 steps of at least this many tokens evaluate only the chosen (token, expert) pairs

    def __init__(self, config: ModelConfig, **kwargs):
        super().__init__(config, **kwargs)

    # ------------------------------------------------------------------ weights
    def load_weights(self, W: Dict[str, torch.Tensor]):
        cfg, dev, T = self.config, self.device, self.dtype
        f32 = torch.float32

        def g(name, shape, dtype=None):
            if name not in W:
                raise KeyError(f"Rorovik checkpoint: tensor {name!r} missing")
            t = W[name]
            if tuple(t.shape) != tuple(shape):
                raise ValueError(f"Rorovik checkpoint: {name} is {tuple(t.shape)}, the config says {tuple(shape)}")
            return t.to(device=dev, dtype=dtype or T).contiguous()

        Wd, side = cfg.width, cfg.side_dim
        self._w = dict(embed=g("embed", (cfg.vocab, Wd)), embed_norm=g("embed.norm", (Wd,)), final_norm=g("final.norm", (Wd,)),
                       head=g("head", (cfg.vocab, Wd)))
        if side:
            self._w["side_embed"] = g("side.embed", (cfg.vocab, side * len(cfg.layers)))
        rows = {}
        self._L = []
        for i, L in enumerate(cfg.layers):
            p, m = f"l{i}.", L.mixer
            ns = SimpleNamespace(type=L.type, norm1=g(p + "norm1", (Wd,)), norm1b=g(p + "norm1b", (Wd,)), window=L.window, scale=float(m["scale"]))
            H = ns.H = int(m["heads"])
            ns.D, ns.Dv = D, Dv = int(m["dim"]), int(m["vdim"])
            ns.sink = g(p + "mix.sink", (H,), f32)
            if L.type == "attention":
                G = ns.G = int(m["kv_heads"])
                qt = m.get("q_temp")
                ns.q_temp = (float(qt["coef"]), int(qt["every"])) if qt is not None else None
                ns.slope = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], dtype=f32, device=dev)
                parts = [(n, g(p + "mix." + n, (r, Wd))) for n, r in (("q", H * D), ("k", G * D), ("v", G * Dv), ("g", H))]
                ns.qb, ns.kb, ns.vb = g(p + "mix.q.b", (H * D,)), g(p + "mix.k.b", (G * D,)), g(p + "mix.v.b", (G * Dv,))
                ns.qn, ns.kn = g(p + "mix.q.norm", (H * D,)), g(p + "mix.k.norm", (G * D,))
                ns.vother = cfg.v_first if L.v_mix and i != cfg.v_first else None
                ns.mix = float(g(p + "mix.vmix", (), f32)) if ns.vother is not None else 0.0
                # normed keys: fp32, or two bf16 values per coordinate (the same bytes)
                rows[(i, "k")] = (ops.diff_key_width(G, D, T == torch.bfloat16), T)
                rows[(i, "v")] = (G * Dv, T)
            else:
                Dr, R, Rq = int(m["rot_dim"]), int(m["kv_rank"]), int(m["q_rank"])
                ns.Dr, ns.R, ns.Rq = Dr, R, Rq
                _, f, ns.amp = rotation(m["rot"] if Dr else None)
                ns.inv_freq = torch.from_numpy(f).to(dev) if f is not None else None
                parts = [("dq", g(p + "mix.dq", (Rq, Wd))), ("dkv", g(p + "mix.dkv", (R + Dr, Wd)))]
                ns.dq_norm, ns.dkv_norm = g(p + "mix.dq.norm", (Rq,)), g(p + "mix.dkv.norm", (R,))
                ns.wuq, _ = pack_rows([("uq", g(p + "mix.uq", (H * (D + Dr), Rq)))], T, dev)
                # per-head maps of the latent, moved to the query side (transposed) and the output side
                ns.uk_t = g(p + "mix.uk", (H * D, R)).view(H, D, R).transpose(1, 2).contiguous()          # [H, R, D]
                ns.uv = g(p + "mix.uv", (H * Dv, R)).view(H, Dv, R).contiguous()                           # [H, Dv, R]
                rows[(i, "c")] = R + Dr
            ns.wproj, ns.off = pack_rows(parts, T, dev)
            ns.wo = g(p + "mix.o", (Wd, H * Dv))
            ns.ff, ns.moe = L.ff, L.moe
            if L.mlp is not None:
                ns.norm2, ns.norm2b = g(p + "norm2", (Wd,)), g(p + "norm2b", (Wd,))
                ns.down_b = None
                if ns.moe:
                    ns.E, ns.identity, ns.top = L.router
                    ns.limit = L.limit
                    ns.router, ns.corr = g(p + "mlp.router", (ns.E + ns.identity, Wd)), g(p + "mlp.correction", (ns.E + ns.identity,), f32)
                    # expert e's rows: [gate_e | up_e], 2 ff rows side by side, so that a step of few rows can skip whole experts
                    ns.wff = torch.cat([g(p + f"mlp.e{e}.{n}", (ns.ff, Wd)) for e in range(ns.E) for n in ("gate", "up")], dim=0)
                    ns.wff, _ = pack_rows([("experts", ns.wff)], T, dev)
                    ns.down = torch.cat([g(p + f"mlp.e{e}.down", (Wd, ns.ff)) for e in range(ns.E)], dim=1).contiguous()
                else:
                    ns.wff, ns.foff = pack_rows([(n, g(p + "mlp." + n, (ns.ff, Wd))) for n in ("gate", "up")], T, dev)
                    ns.gate_b, ns.up_b, ns.down_b = (g(p + f"mlp.{n}.b", (r,)) for n, r in (("gate", ns.ff), ("up", ns.ff), ("down", Wd)))
                    ns.down = g(p + "mlp.down", (Wd, ns.ff))
            if side:
                ns.side_gate, _ = pack_rows([("gate", g(p + "side.gate", (side, Wd)))], T, dev)
                ns.side_proj, _ = pack_cols([("proj", g(p + "side.proj", (Wd, side)))], T, dev)
                ns.side_norm = g(p + "side.norm", (Wd,))
            self._L.append(ns)
        self.pool = HybridPool(len(cfg.layers), rows, {}, self._kv_pool_tokens, self._max_seqs, device=dev, dtype=T)
        return self

    # ------------------------------------------------------------------ cache
    def make_cache(self):
        seq = PagedSequence(self.pool)
        return [RowCache(seq, (i, "k" if ns.type == "attention" else "c")) for i, ns in enumerate(self._L)]

    def make_cache_batch(self, n: int):
        return [self.make_cache() for _ in range(n)]

    # ------------------------------------------------------------------ mixers
    def _attention(self, ns, proj, pl, i, keep):
        """-> [tokens, heads * vdim] in the serving dtype: gated attention read-outs"""
        Tn, H, G, D, Dv, dev, pool = pl.Tn, ns.H, ns.G, ns.D, ns.Dv, self.device, self.pool
        kpool, vpool = pool.rows[(i, "k")], pool.rows[(i, "v")]
        q = torch.empty(Tn, H * D, dtype=torch.float32, device=dev)
        ops.qkv_rownorm_rows(proj, (ns.off["q"], ns.off["k"], ns.off["v"]), H, G, D, G * Dv, ns.qn, ns.kn, self.config.norm_eps, pl.tok_seq,
                             pl.tok_pos, pool.block_table, q, kpool, vpool, qbias=ns.qb, kbias=ns.kb, vbias=ns.vb, temp=ns.q_temp,
                             vother=None if ns.vother is None else pool.rows[(ns.vother, "v")], mix=ns.mix)
        out = torch.empty(Tn, _al8(H * Dv), dtype=self.dtype, device=dev)[:, : H * Dv]
        args = (pl.tok_seq, pl.tok_pos, pool.block_table, H, G, D, Dv, ns.scale, out)
        kw = dict(window=ns.window, slope=ns.slope, sink=ns.sink, gate=proj[:, ns.off["g"]:])
        if Tn <= self.ROWS_FORM:
            ops.grouped_attn_rows(q, kpool, vpool, *args, **kw)
        else:
            ops.grouped_attn_blocks(q, kpool, vpool, pl.qb_start, pl.qb_count, *args, **kw)
        keep.append(q)
        return out

    def _latent_attention(self, ns, proj, pl, i, keep):
        """-> [tokens, heads * vdim] in the serving dtype"""
        Tn, H, D, Dr, Dv, R, dev = pl.Tn, ns.H, ns.D, ns.Dr, ns.Dv, ns.R, self.device
        bt, cpool = self.pool.block_table, self.pool.rows[(i, "c")]
        cq = ops.latent_prep_rows(proj[:, ns.off["dkv"]:], ns.dkv_norm, R, Dr, ns.inv_freq, pl.tok_seq, pl.tok_pos, bt, cpool,
                                  self.config.norm_eps, amp=ns.amp, dq=proj[:, ns.off["dq"]:], wq=ns.dq_norm)
        q = self._linear(cq, ns.wuq)
        mfma = ops.latent_mfma_fits(cpool, R, Dr)
        qabs = torch.empty(Tn, H * (R + Dr), dtype=torch.bfloat16 if mfma else torch.float32, device=dev)
        # absorbed keys: q'_h = U_k,h^T q_h for every head (batch = heads, strides inside the packed rows)
        ops.linear_any(q, ns.uk_t.view(H * R, D), out=qabs, M=Tn, N=R, K=D, batch=H, stride_a=D + Dr, stride_w=R * D, stride_c=R + Dr)
        if Dr:
            ops.rope_pairs_rows(q[:, D:], D + Dr, H, Dr, ns.inv_freq, pl.tok_pos, qabs[:, R:], R + Dr, amp=ns.amp)
        qv = qabs.view(Tn, H, R + Dr)
        if mfma:
            ol = ops.latent_attn_mfma(qv, cpool, pl.tok_seq, pl.tok_pos, bt, H, R, Dr, ns.scale, sink=ns.sink,
                                      blocks=None if Tn <= self.ROWS_FORM else (pl.qb_start, pl.qb_count))
        elif (self.dtype == torch.float32 or Tn > self.ROWS_FORM) and R <= 512 and (32 * _al8(R + Dr) + 512) * 4 <= 150 * 1024:
            ol = ops.latent_attn_blocks(qv, cpool, pl.qb_start, pl.qb_count, pl.tok_seq, pl.tok_pos, bt, H, R, Dr, ns.scale, sink=ns.sink)
        else:
            ol = ops.latent_attn(qv, cpool, pl.tok_seq, pl.tok_pos, bt, H, R, Dr, ns.scale, sink=ns.sink)
        out = torch.empty(Tn, _al8(H * Dv), dtype=self.dtype, device=dev)[:, : H * Dv]
        ops.linear_any(ol.view(Tn, H * R), ns.uv.view(H * Dv, R), out=out, M=Tn, N=Dv, K=R, batch=H, stride_a=R, stride_w=Dv * R, stride_c=Dv)
        keep += [cq, q, qabs, ol]
        return out

    # ------------------------------------------------------------------ feed-forwards
    def _feed_forward(self, ns, h, keep):
        """-> what the residual step adds up: the result rows, and of experts the weight of the input rows handed on and, where the chosen pairs
        were evaluated one by one, each token's rows"""
        Tn, T, dev, ff = h.shape[0], self.dtype, self.device, ns.ff
        if ns.moe:
            few = Tn <= self.STREAM_ROWS and T != torch.float32       # decode rows over bf16 weights: weight-streaming projections
            route, ident = ops.moe_router_softmax(h, ns.router, ns.top, ns.identity, ns.corr)
            step = dict(pass_=ident, src=h) if ident is not None else {}
            if Tn >= self.GROUPED_ROWS and ops.moe_grouped_fits(h, ns.wff, ns.down, ff):
                y, slots = ops.moe_grouped_rows(h, ns.wff, ns.down, route, ns.top, ops.GLU_CLAMPED, ns.limit)
                keep += [route, y, step]
                return y, dict(step, slots=slots)
            gu = self._linear(h, ns.wff, skip=dict(skip_gate=route, skip_col0=0, E=ns.E, ff=2 * ff) if few else None)
            act = torch.empty(Tn, _al8(ns.E * ff), dtype=T, device=dev)[:, : ns.E * ff]
            ops.glu_rows(gu, gu[:, ff:], ops.GLU_CLAMPED, out=act, route=route, E=ns.E, ff=ff, estride=2 * ff, limit=ns.limit)
            keep.append(route)
        else:
            step = dict(bias=ns.down_b)
            gu = self._linear(h, ns.wff)
            act = torch.empty(Tn, _al8(ff), dtype=T, device=dev)[:, :ff]
            ops.glu_rows(gu[:, ns.foff["gate"]: ns.foff["gate"] + ff], gu[:, ns.foff["up"]:], ops.GLU_RELU, out=act, gbias=ns.gate_b, ubias=ns.up_b)
        y = self._linear(act, ns.down)
        keep += [gu, act, y, step]
        return y, step

    # ------------------------------------------------------------------ the device side of a step
    def _run(self, pl, logits_dtype=torch.float32):
        """Nothing here looks at host data that changes between two steps of the same shape, so a decode step can be
        captured once and replayed."""
        cfg, dev, T = self.config, self.device, self.dtype
        eps, mult, Tn, side = cfg.norm_eps, cfg.residual_mult, pl.Tn, cfg.side_dim
        norms1 = [ns.norm1 for ns in self._L] + [None]
        x = torch.empty(Tn, cfg.width, dtype=torch.float32, device=dev)
        h = ops.sandwich_step(x, self._w["embed"], self._w["embed_norm"], ids=pl.ids, init=True, w=norms1[0], eps=eps)
        keep = [pl.md, pl.ids, x]
        for i, ns in enumerate(self._L):
            # what the layer's last sublayer hands on: the stream itself to the token input, else the next layer's normed input
            last = dict(cast=True) if side else dict(w=norms1[i + 1])
            proj = self._linear(h, ns.wproj)
            o = (self._attention if ns.type == "attention" else self._latent_attention)(ns, proj, pl, i, keep)
            y = self._linear(o, ns.wo)
            keep += [h, proj, o, y]
            h = ops.sandwich_step(x, y, ns.norm1b, mult, eps=eps, **(dict(w=ns.norm2) if ns.ff else last))
            if ns.ff:
                h2 = h
                y, step = self._feed_forward(ns, h2, keep)
                h = ops.sandwich_step(x, y, ns.norm2b, mult, eps=eps, **step, **last)
                keep.append(h2)
            if side:
                gt = self._linear(h, ns.side_gate)
                e = torch.empty(Tn, _al8(side), dtype=T, device=dev)
                if e.shape[1] != side:
                    e[:, side:].zero_()
                ops.gelu_tanh_gate_rows(gt[:, :side], self._w["side_embed"], pl.ids, i * side, out=e[:, :side])
                y = self._linear(e, ns.side_proj)
                keep += [h, gt, e, y]
                h = ops.sandwich_step(x, y, ns.side_norm, mult, w=norms1[i + 1], eps=eps)
            if self._trace is not None:
                self._trace.append(x.clone())
        keep.append(h)
        self._keep = keep
        if pl.rows.size == 0:
            return None
        xl = x if pl.all_rows else x.index_select(0, pl.rows_d.long())
        hn = ops.rms_rows(xl, self._w["final_norm"], eps)
        # rows at a pitch of vocab rounded up to 8: 16-byte aligned bf16 rows for the samplers, whatever the vocabulary
        out = torch.empty(hn.shape[0], _al8(cfg.vocab), dtype=logits_dtype, device=dev)[:, : cfg.vocab]
        return self._linear(hn, self._w["head"], out=out)
