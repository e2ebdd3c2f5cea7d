"""Slow float64 oracle of the Mugipel design, one function per mechanism, written from the design's
equations and sharing no code with the product path.

Notation: x is the residual stream [T, width] of ONE sequence, positions 0 .. T-1; a layer is
x <- x + m (mixer(h) + ff(h)) with h = N(x), N an RMS norm whose weight is stored around zero; some
layers form a loop that runs several times in a row with the same weights, each pass mixing the
embedding output back in.  Weights come as a dict under the checkpoint's names ('l<i>.mix.<name>',
'l<i>.mlp.<name>'), the configuration as the parsed config.json.
"""
import math

import torch

F64 = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    """RMS norm with a weight stored around zero."""
    return unit_rms(x, eps) * (1.0 + w)


def frequencies(rot):
    """Rotation frequencies [dims / 2] (f64) and the factor on cos and sin.  With YaRN scaling a
    frequency that turns often inside the original length stays, one that turns seldom is divided
    by the factor, with a linear ramp over the dimension index in between."""
    dims, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def index(turns):       # the dimension index whose frequency makes ``turns`` turns in the original length
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(index(sc["fast"])), 0), min(math.ceil(index(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate_half(x, pos, rot):
    """Rotate pairs (i, i + dims / 2) of the last axis of x [T, heads, d]; entries from ``dims`` on
    pass unchanged."""
    out = x.clone()
    if not rot:
        return out
    f, mul = frequencies(rot)
    half = rot["dims"] // 2
    for i in range(half):
        a = pos.to(F64) * f[i]
        c, s = (torch.cos(a) * mul)[:, None], (torch.sin(a) * mul)[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def same_chunk(i, j, size):
    """Does position i see position j <= i?  Only inside its own chunk of ``size`` positions."""
    return j <= i and (not size or i // size == j // size)


def cap(s, c):
    return c * torch.tanh(s / c) if c else s


def attention(h, W, p, m):
    """Grouped-query attention inside chunks: soft-capped scores, one learned sink term per head in
    the softmax denominator, a sigmoid gate on the concatenated heads."""
    T, H = h.shape[0], m["heads"]
    G, d = m.get("kv_heads", H), m["dim"]
    dv = m.get("vdim", d)
    pos = torch.arange(T)
    q = rotate_half((h @ W[p + "q"].T).view(T, H, d), pos, m.get("rot"))
    k = rotate_half((h @ W[p + "k"].T).view(T, G, d), pos, m.get("rot"))
    v = (h @ W[p + "v"].T).view(T, G, dv)
    size = (m.get("mask") or {}).get("size", 0)
    out = torch.zeros(T, H, dv, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        for i in range(T):
            js = torch.tensor([j for j in range(i + 1) if same_chunk(i, j, size)])
            s = cap((k[js, g] @ q[i, hd]) * m["scale"], m.get("softcap"))
            top = max(float(s.max()), float(W[p + "sink"][hd]))
            e = torch.exp(s - top)
            pr = e / (e.sum() + torch.exp(W[p + "sink"][hd] - top))
            out[i, hd] = pr @ v[js, g]
    return (out.reshape(T, H * dv) * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def latent_attention(h, W, p, m, eps):
    """Causal attention whose keys and values are projections of one normed latent per token, without
    positions; a sigmoid gate on the concatenated heads."""
    T, H, d = h.shape[0], m["heads"], m["dim"]
    dv = m.get("vdim", d)
    q = (h @ W[p + "q"].T).view(T, H, d)
    c = unit_rms(h @ W[p + "dkv"].T, eps) * W[p + "dkv.norm"]
    k, v = (c @ W[p + "uk"].T).view(T, H, d), (c @ W[p + "uv"].T).view(T, H, dv)
    out = torch.zeros(T, H, dv, dtype=F64)
    for hd in range(H):
        for i in range(T):
            pr = torch.softmax((k[:i + 1, hd] @ q[i, hd]) * m["scale"], -1)
            out[i, hd] = pr @ v[:i + 1, hd]
    return (out.reshape(T, H * dv) * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def feed_forward(h, W, p):
    return torch.relu(h @ W[p + "up"].T) ** 2 @ W[p + "down"].T


def layer(x, W, i, L, eps, mult):
    p, m = f"l{i}.", L["mixer"]
    h = norm(x, W[p + "norm1"], eps)
    if L["type"] == "attention":
        y = attention(h, W, p + "mix.", m)
    else:
        assert L["type"] == "latent_attention"
        y = latent_attention(h, W, p + "mix.", m, eps)
    if L.get("mlp"):
        y = y + feed_forward(h, W, p + "mlp.")
    return x + mult * y


def runs(cfg):
    """[(layer, pass of the loop that starts with it or None)] in the order they run."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        out += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return out + [(i, None) for i in range(lp["stop"], n)]


def forward(tokens, W, cfg, taps=None):
    """Logits [T, vocab] of one sequence; ``taps`` (a list) receives the stream after every layer run."""
    W = {k: v.to(F64) for k, v in W.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x0 = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    x = x0
    for i, t in runs(cfg):
        if t is not None:
            x = torch.cat([x, x0], -1) @ W["loop.in"].T + W["loop.step"][t]
        x = layer(x, W, i, cfg["layers"][i], eps, mult)
        if taps is not None:
            taps.append(x.clone())
    return norm(x, W["final.norm"], eps) @ W["embed"].T


