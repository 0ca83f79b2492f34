"""Plain float64 restatement of the Zivitar decoder: one function per mechanism, whole sequences only, dense masks, explicit
token loops for the recurrence.  No cache, no state hand-over, no packed weights - nothing is shared with the product path.

Notation: h [T, width] the input of a sublayer, W [out, in] applied as h @ W.T, p the position (0-based) of a token.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms(y, eps):
    return y / torch.sqrt((y * y).mean(dim=-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def causal_conv(h, w):
    """h [T, C], w [C, taps]: out_t = sum_j w[:, j] * h_(t - taps + 1 + j), zeros before the first token (the last column
    of w meets the token itself)"""
    T, taps = h.shape[0], w.shape[1]
    out = torch.zeros_like(h)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            out[back:] += h[: T - back] * w[:, j]
    return out


def rotation_table(rot):
    """-> (one frequency per rotated pair, the factor on cos and sin).  Without `scaling`: base^(-2 i / dims) and 1."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=F64), 1.0
    factor, original = float(sc["factor"]), float(sc["original"])

    def turns(t):                  # the (real-valued) pair index whose wave turns t times over `original` positions
        return dims * math.log(original / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo = max(math.floor(turns(float(sc["fast"]))), 0)
    hi = min(math.ceil(turns(float(sc["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * r + fi * (1.0 - r))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(factor) + 1.0


def rotate_half(x, rot):
    """x [T, heads, D]: the pair (i, i + dims / 2), i < dims / 2, turns by p times its frequency; dimensions >= dims pass"""
    dims = int((rot or {}).get("dims", 0))
    if not dims:
        return x
    f, amp = rotation_table(rot)
    half = dims // 2
    ang = torch.arange(x.shape[0], dtype=F64)[:, None] * f[None]
    c, s = (torch.cos(ang) * amp)[:, None, :], (torch.sin(ang) * amp)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


def visible(T, size, keep_first):
    """[T, T] bool: query i sees key j <= i when it is less than `size` back (size None: no window) or among the kept first"""
    i = torch.arange(T)
    dist = i[:, None] - i[None, :]
    seen = dist >= 0
    if size is not None:
        seen = seen & ((dist < size) | (i[None, :] < keep_first))
    return seen


def softmax_map(q, k, v, scale, seen):
    """one attention map: q [T, D], k [T, D], v [T, Dv] -> [T, Dv]"""
    s = ((q @ k.T) * scale).masked_fill(~seen, -math.inf)
    return torch.softmax(s, dim=-1) @ v


def lambda_of(lq1, lk1, lq2, lk2, diff):
    return float(torch.exp((lq1 * lk1).sum()) - torch.exp((lq2 * lk2).sum()) + diff)


def differential_attention(q, k, v, scale, seen, lam, diff, eps):
    """q [T, H, 2, D], k [T, G, 2, D], v [T, G, Dv] -> [T, H, Dv]: the difference of two maps over the same values, RMS per head"""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        a1 = softmax_map(q[:, h, 0], k[:, g, 0], v[:, g], scale, seen)
        a2 = softmax_map(q[:, h, 1], k[:, g, 1], v[:, g], scale, seen)
        out[:, h] = rms(a1 - lam * a2, eps) * (1.0 - diff)
    return out


def attention_mixer(h, W, p, m, eps):
    T = h.shape[0]
    H, G, D, Dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (causal_conv(h @ W[p + n].T, W[p + n + ".conv"]) if int(m.get("conv") or 0) else h @ W[p + n].T for n in "qkv")
    q = rotate_half(q.view(T, H * 2, D), m.get("rot")).view(T, H, 2, D)
    k = rotate_half(k.view(T, G * 2, D), m.get("rot")).view(T, G, 2, D)
    mask = m.get("mask") or {}
    seen = visible(T, int(mask["size"]) if mask.get("size") is not None else None, int(mask.get("keep_first") or 0))
    lam = lambda_of(W[p + "lq1"], W[p + "lk1"], W[p + "lq2"], W[p + "lk2"], float(m["diff"]))
    o = differential_attention(q, k, v.view(T, G, Dv), float(m["scale"]), seen, lam, float(m["diff"]), eps)
    return o.reshape(T, H * Dv) @ W[p + "o"].T


def fixed_decay_recurrence(q, k, v, decay):
    """q, k [T, H, D], v [T, H, Dv], decay [H]: S <- decay S + k v^T, o = S^T q"""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64)
    o = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(dim=1)
    return o


def lightning_mixer(h, W, p, m, eps):
    T = h.shape[0]
    H, D, Dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k = (silu(h @ W[p + n].T).view(T, H, D) for n in "qk")
    v = silu(h @ W[p + "v"].T).view(T, H, Dv)
    o = fixed_decay_recurrence(q, k, v, torch.tensor(m["decay"], dtype=F64)).reshape(T, H * Dv)
    o = rms(o, eps) * W[p + "norm"]                                  # over ALL heads together
    return (o * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def clamped_glu(g, u, limit):
    g = torch.clamp(g, max=limit)
    return g * torch.sigmoid(1.702 * g) * (torch.clamp(u, -limit, limit) + 1.0)


def feed_forward(h, W, p, mlp):
    return clamped_glu(h @ W[p + "gate"].T, h @ W[p + "up"].T, float(mlp["limit"])) @ W[p + "down"].T


MIXERS = {"attention": attention_mixer, "lightning": lightning_mixer}


def hyper_read(X, w_in):
    """X [s, T, width] -> the sublayer's input before its norm"""
    return torch.einsum("s,std->td", w_in, X)


def hyper_write(X, y, mix, out):
    """every new stream from the old ones (mix is [from, to]) and the sublayer's result"""
    return torch.einsum("st,snd->tnd", mix, X) + out[:, None, None] * y[None]


def source(cfg, i):
    """the layer whose tensors layer i uses"""
    while cfg["layers"][i].get("weights_of") is not None:
        i = int(cfg["layers"][i]["weights_of"])
    return i


def head(cfg, W, x):
    lg = (rms(x, float(cfg["norm"]["eps"])) * W["final.norm"]) @ W["head"].T * float(cfg.get("logit_scale", 1.0))
    cap = cfg.get("logit_softcap")
    return float(cap) * torch.tanh(lg / float(cap)) if cap else lg


def forward(cfg, W, tokens):
    """-> (logits [T, vocab], [sum of the streams after every layer])   W: {name: float64 tensor}"""
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    X = x[None].repeat(int(cfg["streams"]), 1, 1)
    after = []
    for i, L in enumerate(cfg["layers"]):
        p = f"l{source(cfg, i)}."
        subs = [("1", lambda h: MIXERS[L["type"]](h, W, p + "mix.", L["mixer"], eps))]
        if L.get("mlp"):
            subs.append(("2", lambda h: feed_forward(h, W, p + "mlp.", L["mlp"])))
        for n, sub in subs:
            hc = p + f"hc{n}."
            y = sub(rms(hyper_read(X, W[hc + "in"]), eps) * W[p + "norm" + n])
            X = hyper_write(X, y, W[hc + "mix"], W[hc + "out"])
        after.append(X.sum(dim=0))
    return head(cfg, W, X.sum(dim=0)), after
