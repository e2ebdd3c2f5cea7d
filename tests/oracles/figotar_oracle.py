"""Slow float64 oracle of the Figotar design, one function per mechanism, written from the design's
equations and sharing no code with the product path.

Notation: x is the residual stream [T, width] of ONE sequence, positions 0 .. T-1.  Every layer is
x <- x + N1b(mixer(N1(x))), then x <- x + N2b(ff(N2(x))) when it has a feed-forward; these N are RMS
norms whose weight is stored around zero.  Weights come as a dict under the checkpoint's names
('l<i>.mix.<name>', 'l<i>.mlp.<name>'), the configuration as the parsed config.json.
"""
import math

import torch

F64 = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    """RMS norm with a weight stored around zero."""
    return unit_rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def slope(head, heads):
    """Score lost per token of distance."""
    return 2.0 ** (-8.0 * (head + 1) / heads)


def temperature(p, qt):
    """Growth of the queries with their position."""
    return 1.0 + qt["coef"] * math.log(math.floor((p + 1) / qt["every"]) + 1.0) if qt else 1.0


def visible(i, j, size):
    """Does position i see position j?  ``size`` 0: everything up to itself."""
    return j <= i and (not size or i - j < size)


def rotate_half(x, dims, base):
    """Rotate pairs (i, i + dims / 2) of the last axis of x [T, ..., d]; entries from ``dims`` on pass."""
    out, half = x.clone(), dims // 2
    for i in range(half):
        for t in range(x.shape[0]):
            a = t * base ** (-2.0 * i / dims)
            u, v = x[t, ..., i], x[t, ..., i + half]
            out[t, ..., i] = u * math.cos(a) - v * math.sin(a)
            out[t, ..., i + half] = v * math.cos(a) + u * math.sin(a)
    return out


def head_gates(h, W, p):
    """One number per head and token."""
    return sigmoid(h @ W[p + "g"].T)


def attention(h, W, p, m):
    """Grouped-query attention inside a window, without rotation: biased projections, queries that grow
    with the position, scores that fall with the distance."""
    T, H, d = h.shape[0], m["heads"], m["dim"]
    G, dv = m.get("kv_heads", H), m.get("vdim", d)
    q = (h @ W[p + "q"].T + W[p + "q.b"]).view(T, H, d)
    k = (h @ W[p + "k"].T + W[p + "k.b"]).view(T, G, d)
    v = (h @ W[p + "v"].T + W[p + "v.b"]).view(T, G, dv)
    size = (m.get("mask") or {}).get("size", 0)
    gate = head_gates(h, W, p)
    out = torch.zeros(T, H, dv, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        for i in range(T):
            lo = next(j for j in range(max(0, i - size) if size else 0, i + 1) if visible(i, j, size))
            qi = q[i, hd] * temperature(i, m.get("q_temp"))
            s = (k[lo:i + 1, g] @ qi) * m["scale"]
            s = s - slope(hd, H) * (i - torch.arange(lo, i + 1, dtype=F64))
            out[i, hd] = torch.softmax(s, -1) @ v[lo:i + 1, g] * gate[i, hd]
    return out.reshape(T, H * dv) @ W[p + "o"].T


def latent_attention(h, W, p, m, eps):
    """Causal attention on one normed latent and one rotated key part per token, queries through a normed
    latent of their own, one learned sink per head in the softmax denominator."""
    T, H, d, rd, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    dv = m["vdim"]
    cq = unit_rms(h @ W[p + "dq"].T, eps) * W[p + "dq.norm"]
    q = (cq @ W[p + "uq"].T).view(T, H, d + rd)
    down = h @ W[p + "dkv"].T
    c = unit_rms(down[:, :rank], eps) * W[p + "dkv.norm"]
    k, v = (c @ W[p + "uk"].T).view(T, H, d), (c @ W[p + "uv"].T).view(T, H, dv)
    kr = down[:, rank:]
    qr = q[:, :, d:]
    if rd:
        kr, qr = rotate_half(kr, rd, m["rot"]["base"]), rotate_half(qr, rd, m["rot"]["base"])
    gate = head_gates(h, W, p)
    out = torch.zeros(T, H, dv, dtype=F64)
    for hd in range(H):
        sink = W[p + "sink"][hd]
        for i in range(T):
            s = (k[:i + 1, hd] @ q[i, hd, :d] + kr[:i + 1] @ qr[i, hd]) * m["scale"]
            top = torch.maximum(s.max(), sink)
            e = torch.exp(s - top)
            out[i, hd] = (e / (e.sum() + torch.exp(sink - top))) @ v[:i + 1, hd] * gate[i, hd]
    return out.reshape(T, H * dv) @ W[p + "o"].T


def mlstm(h, W, p, m, eps):
    """Matrix memory with capped exponential input gates, sigmoid forget gates in log space, a running
    maximum that starts at 0 and a normaliser."""
    T, H, d, dv, cap = h.shape[0], m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q = (h @ W[p + "q"].T).view(T, H, d) * d ** -0.5
    k, v = (h @ W[p + "k"].T).view(T, H, d), (h @ W[p + "v"].T).view(T, H, dv)
    ig = cap * torch.tanh((h @ W[p + "i"].T + W[p + "i.b"]) / cap)
    fg = -torch.log1p(torch.exp(-cap * torch.tanh((h @ W[p + "f"].T + W[p + "f.b"]) / cap)))
    out = torch.zeros(T, H, dv, dtype=F64)
    for hd in range(H):
        S, n, top = torch.zeros(d, dv, dtype=F64), torch.zeros(d, dtype=F64), torch.zeros((), dtype=F64)
        for t in range(T):
            new = torch.maximum(fg[t, hd] + top, ig[t, hd])
            a, b = torch.exp(fg[t, hd] + top - new), torch.exp(ig[t, hd] - new)
            S = a * S + b * k[t, hd][:, None] * v[t, hd][None, :]
            n, top = a * n + b * k[t, hd], new
            out[t, hd] = (S.T @ q[t, hd]) / (torch.maximum((n @ q[t, hd]).abs(), torch.exp(-top)) + 1e-6)
    y = unit_rms(out, eps).reshape(T, H * dv) * W[p + "norm"]
    return (y * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def feed_forward(h, W, p):
    lin = lambda n, z: z @ W[p + n].T + W[p + n + ".b"]
    return lin("down", gelu_tanh(lin("gate", h)) * lin("up", h))


def layer(x, W, i, L, eps):
    p, m = f"l{i}.", L["mixer"]
    h = norm(x, W[p + "norm1"], eps)
    if L["type"] == "attention":
        y = attention(h, W, p + "mix.", m)
    elif L["type"] == "latent_attention":
        y = latent_attention(h, W, p + "mix.", m, eps)
    else:
        assert L["type"] == "mlstm"
        y = mlstm(h, W, p + "mix.", m, eps)
    x = x + norm(y, W[p + "norm1b"], eps)
    if L.get("mlp"):
        x = x + norm(feed_forward(norm(x, W[p + "norm2"], eps), W, p + "mlp."), W[p + "norm2b"], eps)
    return x


def forward(tokens, W, cfg, taps=None):
    """Logits [T, vocab] of one sequence; ``taps`` (a list) receives the stream after every layer."""
    W = {k: v.to(F64) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, L in enumerate(cfg["layers"]):
        x = layer(x, W, i, L, eps)
        if taps is not None:
            taps.append(x.clone())
    return norm(x, W["final.norm"], eps) @ W["head"].T
