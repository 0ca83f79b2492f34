"""Plain restatement of the Rorovik decoder for the tests: one function per mechanism, whole prompts, dense masks, per-head keys and
values written out (no absorbed maps, no cache, no pages), in the dtype it is given (float64 in the tests).  It shares no code with
the product path.

Notation: x [T, W] the residual stream, p the positions 0..T-1, eps the norm constant, m the residual multiplier,
rms(y) = y / sqrt(mean(y^2) + eps), norm(y, w) = rms(y) * w.
    x            = norm(E[token], w_e)
    layer        : x <- x + m norm(mixer(norm(x, w1)), w1b);   x <- x + m norm(ff(norm(x, w2)), w2b)   (the second step only with a
                   feed-forward);   x <- x + m norm(P (gelu_tanh(G x) * E2[token, layer slice]), w_s)
    logits       = norm(x, w_f) W_head^T
"""
from __future__ import annotations

import math

import torch


def rms(y, eps):
    return y / torch.sqrt(y.pow(2).mean(-1, keepdim=True) + eps)


def norm(y, w, eps):
    return rms(y, eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def frequencies(rot):
    """(frequency per pair, factor on cos and sin) of a rotation over `dims` dimensions, with the scaled form where the entry has one"""
    n, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def index(turns):           # pair index (real number) whose angle makes `turns` full turns over the original length
        return n * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(index(sc["fast"])), 0), min(math.ceil(index(sc["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * r + fi * (1.0 - r))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate_pairs(y, rot):
    """y [T, ..., dims]: the neighbours (2 i, 2 i + 1) turn by position * frequency_i"""
    f, amp = frequencies(rot)
    T = y.shape[0]
    a = torch.arange(T, dtype=y.dtype).view(T, *([1] * (y.dim() - 2)), 1) * torch.tensor(f, dtype=y.dtype)
    u, v = y[..., 0::2], y[..., 1::2]
    out = torch.empty_like(y)
    out[..., 0::2] = amp * (u * torch.cos(a) - v * torch.sin(a))
    out[..., 1::2] = amp * (v * torch.cos(a) + u * torch.sin(a))
    return out


def visible(T, window=None):
    """[T, T] bool: query i sees key j when 0 <= i - j (< window when there is one)"""
    d = torch.arange(T).view(-1, 1) - torch.arange(T).view(1, -1)
    return (d >= 0) & ((d < window) if window else torch.ones_like(d, dtype=torch.bool))


def sink_softmax(scores, vis, sink):
    """scores [H, T, T], sink [H]: exp(s) / (exp(sink_h) + sum over the visible keys of exp(s))"""
    s = scores.masked_fill(~vis, float("-inf"))
    top = torch.maximum(s.max(-1, keepdim=True).values, sink.view(-1, 1, 1))
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink.view(-1, 1, 1) - top))


def temperature(T, qt, dtype):
    steps = (torch.arange(T) + 1) // qt["every"]
    return 1.0 + qt["coef"] * torch.log(steps.to(dtype) + 1.0)


def slopes(H, dtype):
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], dtype=dtype)


def attention_mixer(W, p, m, h, eps, v_first=None):
    """-> (output, values before any mixing when this layer takes part in it and is the first).  v_first: the first layer's values"""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m.get("vdim", m["dim"])
    q = norm(h @ W[p + "q"].T + W[p + "q.b"], W[p + "q.norm"], eps).view(T, H, D)
    k = norm(h @ W[p + "k"].T + W[p + "k.b"], W[p + "k.norm"], eps).view(T, G, D)
    v = (h @ W[p + "v"].T + W[p + "v.b"]).view(T, G, Dv)
    if m.get("v_mix"):
        if v_first is None:
            v_first = v
        else:
            lam = W[p + "vmix"]
            v = (1.0 - lam) * v + lam * v_first
    if m.get("q_temp"):
        q = q * temperature(T, m["q_temp"], h.dtype).view(T, 1, 1)
    k, v = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1)
    s = torch.einsum("ihd,jhd->hij", q, k) * m["scale"]
    dist = (torch.arange(T).view(-1, 1) - torch.arange(T).view(1, -1)).to(h.dtype)
    s = s - slopes(H, h.dtype).view(H, 1, 1) * dist
    w = sink_softmax(s, visible(T, (m.get("mask") or {}).get("size")), W[p + "sink"])
    o = torch.einsum("hij,jhd->ihd", w, v) * torch.sigmoid(h @ W[p + "g"].T).view(T, H, 1)
    return o.reshape(T, H * Dv) @ W[p + "o"].T, v_first


def latent_mixer(W, p, m, h, eps):
    T = h.shape[0]
    H, D, Dr, Dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (norm(h @ W[p + "dq"].T, W[p + "dq.norm"], eps) @ W[p + "uq"].T).view(T, H, D + Dr)
    d = h @ W[p + "dkv"].T
    c = norm(d[:, :R], W[p + "dkv.norm"], eps)
    k = (c @ W[p + "uk"].T).view(T, H, D)
    v = (c @ W[p + "uv"].T).view(T, H, Dv)
    s = torch.einsum("ihd,jhd->hij", q[..., :D], k)
    if Dr:
        s = s + torch.einsum("ihd,jd->hij", rotate_pairs(q[..., D:], m["rot"]), rotate_pairs(d[:, R:], m["rot"]))
    w = sink_softmax(s * m["scale"], visible(T), W[p + "sink"])
    return torch.einsum("hij,jhd->ihd", w, v).reshape(T, H * Dv) @ W[p + "o"].T


def dense_ff(W, p, h):
    g = torch.clamp(h @ W[p + "gate"].T + W[p + "gate.b"], min=0.0)
    return (g * (h @ W[p + "up"].T + W[p + "up.b"])) @ W[p + "down"].T + W[p + "down.b"]


def clamped_glu(g, u, limit):
    if limit is not None:
        g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def route(z, top, correction):
    """logits z [T, E + identity] -> weights of the same shape: scores = softmax over all columns, the `top` largest of score +
    correction keep their score, every other column 0 (lowest index wins a tie)"""
    s = torch.softmax(z, -1)
    out = torch.zeros_like(s)
    for t in range(z.shape[0]):
        c = s[t] + correction
        for e in sorted(range(z.shape[1]), key=lambda e: (-c[e].item(), e))[:top]:
            out[t, e] = s[t, e]
    return out


def moe_ff(W, p, ml, h):
    r = ml["router"]
    E = r["experts"]
    w = route(h @ W[p + "router"].T, r["top"], W[p + "correction"])
    out = w[:, E:].sum(-1, keepdim=True) * h                      # the identity experts hand their input on
    for e in range(E):
        rows = torch.nonzero(w[:, e]).view(-1)
        if rows.numel():
            he = h[rows]
            a = clamped_glu(he @ W[p + f"e{e}.gate"].T, he @ W[p + f"e{e}.up"].T, ml["expert"].get("limit"))
            out[rows] += w[rows, e].view(-1, 1) * (a @ W[p + f"e{e}.down"].T)
    return out


def token_input(W, p, x, e, eps):
    g = gelu_tanh(x @ W[p + "gate"].T) * e
    return norm(g @ W[p + "proj"].T, W[p + "norm"], eps)


class Oracle:
    def __init__(self, cfg, W, dtype=torch.float64):
        self.cfg, self.dtype = cfg, dtype
        self.W = {k: v.to(dtype) for k, v in W.items()}

    def forward(self, ids, layers_out=None):
        """ids [T] -> logits [T, vocab]; layers_out (a list) receives the stream after every layer"""
        cfg, W = self.cfg, self.W
        eps, mult = cfg["norm"]["eps"], cfg.get("residual_mult", 1.0)
        ids = torch.as_tensor(ids).long()
        x = norm(W["embed"][ids], W["embed.norm"], eps)
        v_first = None
        for i, L in enumerate(cfg["layers"]):
            p, m = f"l{i}.", L["mixer"]
            h = norm(x, W[p + "norm1"], eps)
            if L["type"] == "attention":
                y, v_first = attention_mixer(W, p + "mix.", m, h, eps, v_first)
            else:
                y = latent_mixer(W, p + "mix.", m, h, eps)
            x = x + mult * norm(y, W[p + "norm1b"], eps)
            if L.get("mlp"):
                h = norm(x, W[p + "norm2"], eps)
                y = moe_ff(W, p + "mlp.", L["mlp"], h) if L["mlp"].get("kind", "dense") == "moe" else dense_ff(W, p + "mlp.", h)
                x = x + mult * norm(y, W[p + "norm2b"], eps)
            if cfg.get("token_side"):
                n = cfg["token_side"]["dim"]
                x = x + mult * token_input(W, p + "side.", x, W["side.embed"][ids][:, i * n:(i + 1) * n], eps)
            if layers_out is not None:
                layers_out.append(x.clone())
        return norm(x, W["final.norm"], eps) @ W["head"].T
