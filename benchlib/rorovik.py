"""`bench.py --workload rorovik-compare`: prefill and decode throughput of the Rorovik design (sublayers normed before and after on an fp32
stream; latent attention with a query latent, scaled rotary positions and sinks; grouped attention with distance bias, window, sinks and mixed
values; dense biased relu-gated and clamped expert feed-forwards with identity experts; a token input per layer) next to the framework's
closest model, Tilalorn (latent and grouped attention, dense gated feed-forwards and mixtures of experts on the same ragged step), at the
same width, depth, head counts and sizes, latent ranks and feed-forward work per token - random weights, synthetic token ids, bf16.  Not the
headline metric: one JSON line of its own."""
from __future__ import annotations

import torch

from benchlib.garesun import SIZES, _measure
from benchlib.tilalorn import tilalorn_cfg, tilalorn_weights


def rorovik_cfg(s, window=1024):
    H, hd, W = s["heads"], s["hd"], s["width"]
    # the comparison model's sizes: a dense layer of half the dense intermediate, or 2 of 8 experts of a quarter of it (here two identity
    # experts compete with them: at most the same work per token)
    dense = dict(kind="dense", ff=s["inter"] // 2 // 8 * 8)
    moe = dict(kind="moe", expert=dict(ff=s["inter"] // 4 // 8 * 8, limit=7.0), router=dict(experts=8, identity=2, top=2))
    att = dict(heads=H, kv_heads=s["kv_heads"], dim=hd, vdim=hd, scale=hd ** -0.5, q_temp=dict(coef=0.1, every=1024), mask=dict(size=window), v_mix=True)
    lat = dict(heads=H, dim=hd, rot_dim=64, vdim=hd, kv_rank=512, q_rank=W // 2, scale=(hd + 64) ** -0.5,
               rot=dict(base=500000.0, dims=64, scaling=dict(factor=4.0, original=4096, fast=32.0, slow=1.0)))
    pattern = [("attention", att, dense), ("latent_attention", lat, moe), ("latent_attention", lat, dense), ("attention", att, moe), ("attention", att, dense),
               ("latent_attention", lat, moe)]
    layers = [dict(type=t, mixer=dict(m), mlp=ml) for t, m, ml in (pattern[i % 6] for i in range(s["layers"]))]
    return dict(architecture="Rorovik", vocab=s["vocab"], width=W, layers=layers, norm=dict(eps=1e-6), residual_mult=0.5, token_side=dict(dim=64))


def rorovik_weights(cfg, dev, seed=0):
    g = torch.Generator(device=dev).manual_seed(seed)
    W, width, side = {}, cfg["width"], cfg["token_side"]["dim"]

    def lin(name, o, i):
        W[name] = (torch.randn(o, i, generator=g, device=dev, dtype=torch.float32) * i ** -0.5).to(torch.bfloat16)

    def const(name, n, v=0.0):
        W[name] = torch.full((n,), v, dtype=torch.bfloat16, device=dev)

    lin("embed", cfg["vocab"], width)
    lin("head", cfg["vocab"], width)
    lin("side.embed", cfg["vocab"], side * len(cfg["layers"]))
    for n in ("embed.norm", "final.norm"):
        const(n, width, 1.0)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        for n in ("norm1", "norm1b", "norm2", "norm2b", "side.norm"):
            const(p + n, width, 1.0)
        const(p + "mix.sink", H)
        if L["type"] == "attention":
            for n, r in (("q", H * D), ("k", m["kv_heads"] * D), ("v", m["kv_heads"] * Dv)):
                lin(p + "mix." + n, r, width)
                const(p + f"mix.{n}.b", r)
            const(p + "mix.q.norm", H * D, 1.0)
            const(p + "mix.k.norm", m["kv_heads"] * D, 1.0)
            lin(p + "mix.g", H, width)
            W[p + "mix.vmix"] = torch.tensor(0.5, dtype=torch.bfloat16, device=dev)
        else:
            Dr, R, Rq = m["rot_dim"], m["kv_rank"], m["q_rank"]
            for n, o, k in (("dq", Rq, width), ("uq", H * (D + Dr), Rq), ("dkv", R + Dr, width), ("uk", H * D, R), ("uv", H * Dv, R)):
                lin(p + "mix." + n, o, k)
            const(p + "mix.dq.norm", Rq, 1.0)
            const(p + "mix.dkv.norm", R, 1.0)
        lin(p + "mix.o", width, H * Dv)
        ml = L["mlp"]
        if ml["kind"] == "moe":
            E, I = ml["router"]["experts"], ml["router"]["identity"]
            lin(p + "mlp.router", E + I, width)
            const(p + "mlp.correction", E + I)
            for e in range(E):
                for n in ("gate", "up"):
                    lin(p + f"mlp.e{e}.{n}", ml["expert"]["ff"], width)
                lin(p + f"mlp.e{e}.down", width, ml["expert"]["ff"])
        else:
            for n, o, k in (("gate", ml["ff"], width), ("up", ml["ff"], width), ("down", width, ml["ff"])):
                lin(p + "mlp." + n, o, k)
                const(p + f"mlp.{n}.b", o)
        lin(p + "side.gate", side, width)
        lin(p + "side.proj", width, side)
    return W


def workload_rorovik_compare(args):
    from mlx_vlm_amd.models import rorovik, tilalorn

    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    prompt_lens, rows, ctx, steps = (512, 2048), (1, 8), 512, max(8, int(args.steps) * 8)
    ids_in = lambda ids: (torch.as_tensor(ids, dtype=torch.int32, device=dev).reshape(-1, 1), None)      # noqa: E731
    res = {}
    for name, s in SIZES.items():
        r = {}
        for model, arch, cfg_of, weights_of in (("rorovik", rorovik, rorovik_cfg, rorovik_weights), ("tilalorn", tilalorn, tilalorn_cfg, tilalorn_weights)):
            cfg = cfg_of(s)
            m = arch.Model(arch.ModelConfig.from_dict(cfg), device=dev, dtype="bfloat16", kv_pool_tokens=16384, max_seqs=12)
            m.load_weights(weights_of(cfg, dev))
            r[model] = _measure(m.language_model, ids_in, s["vocab"], prompt_lens, rows, ctx, steps)
            del m
            torch.cuda.empty_cache()
        r["ratio_rorovik_over_tilalorn"] = {f"{ph}_{k}": round(r["rorovik"][ph][k]["tokens_per_s"] / r["tilalorn"][ph][k]["tokens_per_s"], 3)
                                            for ph in ("prefill", "decode") for k in r["tilalorn"][ph]}
        res[name] = dict(sizes=s, **r)
    return {"metric": "rorovik_vs_tilalorn", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic", "n_gpus": 1,
            "config": {"layers": "6 per model, (attention, latent_attention, latent_attention, attention, attention, latent_attention), feed-forwards "
                                 "alternately dense of half the dense intermediate and 8 experts of a quarter, top 2 (| 2 identity experts "
                                 "more); attention window 1024 on the grouped | on the latent layers",
                       "window": 1024, "prompt_lens": list(prompt_lens), "decode_rows": list(rows), "decode_context": ctx},
            "results": res}
