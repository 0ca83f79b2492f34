"""`bench.py --workload zivitar-compare`: prefill and decode throughput of the Zivitar design (three hyper-connected fp32 residual
streams, a fixed-decay recurrence with one norm over all heads, differential attention on convolved q / k / v inside a window that
keeps the first tokens, dense clamped gated feed-forwards) next to the framework's closest model, Luvapel (matrix-state recurrences,
windowed attention and dense feed-forwards on the same ragged step), at the same width, depth, head count, key rows per head and
feed-forward weights - random weights, synthetic token ids, bf16.  Not the headline metric: one JSON line of its own."""
from __future__ import annotations

import torch

from benchlib.garesun import SIZES, _measure
from benchlib.luvapel import luvapel_cfg, luvapel_weights


def zivitar_cfg(s, window=1024):
    H, hd = s["heads"], s["hd"]
    # the comparison model's feed-forward has two matrices of 3/4 of the dense intermediate, this one three: the same weights
    mlp = dict(kind="dense", ff=s["inter"] // 2 // 64 * 64, limit=7.0)
    light = dict(type="lightning", mixer=dict(heads=H, dim=hd, vdim=hd, decay=[1 - 2.0 ** -(5 + h % 4) for h in range(H)]), mlp=mlp)
    # two maps of half a head's size each: as many query and key rows as an attention head of that size has
    att = dict(type="attention", mlp=mlp,
               mixer=dict(heads=H, kv_heads=s["kv_heads"], dim=hd // 2, vdim=hd, scale=(hd // 2) ** -0.5, diff=0.5, conv=4,
                          mask=dict(size=window, keep_first=8),
                          rot=dict(base=500000.0, dims=hd // 4, scaling=dict(factor=8.0, original=4096, fast=24.0, slow=2.0))))
    layers = [dict(att if i % 3 == 1 else light) for i in range(s["layers"])]
    return dict(architecture="Zivitar", vocab=s["vocab"], width=s["width"], layers=layers, norm=dict(eps=1e-6), streams=3, logit_scale=1.0,
                logit_softcap=30.0)


def zivitar_weights(cfg, dev, seed=0):
    g = torch.Generator(device=dev).manual_seed(seed)
    W, width, S = {}, cfg["width"], cfg["streams"]

    def lin(name, o, i, s=1.0):
        W[name] = (torch.randn(o, i, generator=g, device=dev, dtype=torch.float32) * (s * i ** -0.5)).to(torch.bfloat16)

    def const(name, n, v=1.0):
        W[name] = torch.full((n,), v, dtype=torch.bfloat16, device=dev)

    lin("embed", cfg["vocab"], width, width ** 0.5)
    lin("head", cfg["vocab"], width)
    const("final.norm", width)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        for q in "12":
            const(p + "norm" + q, width)
            const(p + f"hc{q}.in", S, 1.0 / S)
            const(p + f"hc{q}.out", S, 0.5)
            W[p + f"hc{q}.mix"] = (torch.eye(S, device=dev) + 0.05).to(torch.bfloat16)
        if L["type"] == "lightning":
            for n, r in (("q", H * D), ("k", H * D), ("v", H * Dv), ("g", H * Dv)):
                lin(p + "mix." + n, r, width)
            const(p + "mix.norm", H * Dv)
        else:
            for n, r in (("q", H * 2 * D), ("k", m["kv_heads"] * 2 * D), ("v", m["kv_heads"] * Dv)):
                lin(p + "mix." + n, r, width)
                lin(p + f"mix.{n}.conv", r, m["conv"])
            for n in ("lq1", "lk1", "lq2", "lk2"):
                const(p + "mix." + n, D, 0.05)
        lin(p + "mix.o", width, H * Dv)
        ff = L["mlp"]["ff"]
        lin(p + "mlp.gate", ff, width)
        lin(p + "mlp.up", ff, width)
        lin(p + "mlp.down", width, ff)
    return W


def workload_zivitar_compare(args):
    from mlx_vlm_amd.models import luvapel, zivitar

    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    prompt_lens, rows, ctx, steps = (512, 2048), (1, 8), 512, max(8, int(args.steps) * 8)
    ids_in = lambda ids: (torch.as_tensor(ids, dtype=torch.int32, device=dev).reshape(-1, 1), None)      # noqa: E731
    res = {}
    for name, s in SIZES.items():
        r = {}
        for model, arch, cfg_of, weights_of in (("zivitar", zivitar, zivitar_cfg, zivitar_weights), ("luvapel", luvapel, luvapel_cfg, luvapel_weights)):
            cfg = cfg_of(s)
            m = arch.Model(arch.ModelConfig.from_dict(cfg), device=dev, dtype="bfloat16", kv_pool_tokens=16384, max_seqs=12)
            m.load_weights(weights_of(cfg, dev))
            r[model] = _measure(m.language_model, ids_in, s["vocab"], prompt_lens, rows, ctx, steps)
            del m
            torch.cuda.empty_cache()
        r["ratio_zivitar_over_luvapel"] = {f"{ph}_{k}": round(r["zivitar"][ph][k]["tokens_per_s"] / r["luvapel"][ph][k]["tokens_per_s"], 3)
                                           for ph in ("prefill", "decode") for k in r["luvapel"][ph]}
        res[name] = dict(sizes=s, **r)
    return {"metric": "zivitar_vs_luvapel", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic", "n_gpus": 1,
            "config": {"layers": "6 per model: (lightning, differential attention, lightning) x 2 on 3 residual streams, dense clamped gated "
                                 "feed-forward of half the dense intermediate (3 matrices) | (general_delta, parallel[window attention | gated "
                                 "delta], general_delta) x 2, dense relu^2 feed-forward of 3/4 of it (2 matrices)",
                       "window": 1024, "prompt_lens": list(prompt_lens), "decode_rows": list(rows), "decode_context": ctx},
            "results": res}
