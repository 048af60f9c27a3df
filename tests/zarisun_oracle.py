"""Plain float64 oracle of the Zarisun design, one function per mechanism.

Written from the design's equations only: whole sequences, dense attention
rows, a token-by-token recurrence, per-head keys and values expanded from the
latent. It shares no code with the engine, its ops or their torch reference
forms, reads a checkpoint's tensors by their checkpoint names, and knows
nothing of pages, slots, portions or batches.

Notation: W width, n tokens, x the residual stream [n, W] (which the sublayers
read as it is), positions 0 .. n-1.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


def causal_conv(u, w):
    """u [n, C], w [C, taps]: y_t = sum_j w[:, j] * u_(t - taps + 1 + j), zeros
    before the start."""
    n, C = u.shape
    taps = w.shape[1]
    y = torch.zeros(n, C, dtype=F64)
    for j in range(taps):
        back = taps - 1 - j
        if back < n:
            y[back:] += w[:, j] * u[:n - back]
    return y


def turning_number_dim(rot, turns):
    """The (fractional) pair index whose wave turns `turns` times within the
    original context."""
    sc = rot["scaling"]
    return rot["dims"] * math.log(sc["original"] / (2.0 * math.pi * turns)) / \
        (2.0 * math.log(rot["base"]))


def frequencies(rot):
    """base^(-2i/dims); with scaling, pairs below `lo` keep their frequency,
    pairs above `hi` are divided by the factor, a linear ramp between."""
    dims, sc = rot["dims"], rot.get("scaling")
    out = [rot["base"] ** (-2.0 * i / dims) for i in range(dims // 2)]
    if sc:
        lo = max(math.floor(turning_number_dim(rot, sc["fast"])), 0)
        hi = min(math.ceil(turning_number_dim(rot, sc["slow"])), dims - 1)
        for i, f in enumerate(out):
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            out[i] = f / sc["factor"] * ramp + f * (1.0 - ramp)
    return out


def amplitude(rot):
    """The factor on cos and sin of scaled rotations."""
    return 0.1 * math.log(rot["scaling"]["factor"]) + 1.0 if rot.get("scaling") else 1.0


def rotate_pairs(x, rot, first_pos=0):
    """x [n, heads, d]: pair (2i, 2i + 1) of the first `dims` channels turns by
    position * f_i and is stretched by the amplitude; the rest passes."""
    out = x.clone()
    a = amplitude(rot)
    pos = torch.arange(first_pos, first_pos + x.shape[0], dtype=F64).view(-1, 1)
    for i, f in enumerate(frequencies(rot)):
        c, s = a * torch.cos(pos * f), a * torch.sin(pos * f)
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * c - v * s
        out[:, :, 2 * i + 1] = v * c + u * s
    return out


def visible(n, window):
    """[n, n]: row i sees column j iff 0 <= i - j (< window, if there is one)."""
    d = torch.arange(n).view(n, 1) - torch.arange(n).view(1, n)
    return (d >= 0) & (d < window) if window else d >= 0


def softmax_with_sink(s, seen, sink):
    """Weights of the seen scores; exp(sink) joins the denominator."""
    s = s.masked_fill(~seen, float("-inf"))
    top = torch.clamp(s.max(dim=1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - top)
    return e / (torch.exp(sink - top) + e.sum(dim=1, keepdim=True))


def head_gates(t, p, h):
    return sigmoid(h @ t[p + "g"].T)                       # [n, H]


def conv_attention(t, p, h, m, eps):
    """Grouped-head attention whose values are its keys as they leave the short
    convolution; q and k are RMS-normed over the whole projection, then
    rotated; a window, a sink and one gate per head."""
    n = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q = causal_conv(h @ t[p + "q"].T, t[p + "q.conv"])
    k = causal_conv(h @ t[p + "k"].T, t[p + "k.conv"])
    v = k.view(n, G, D)
    q = rotate_pairs((rms(q, eps) * t[p + "q.norm"]).view(n, H, D), m["rot"])
    k = rotate_pairs((rms(k, eps) * t[p + "k.norm"]).view(n, G, D), m["rot"])
    seen = visible(n, (m.get("mask") or {}).get("size"))
    out = torch.zeros(n, H, D, dtype=F64)
    for a in range(H):
        g = a // (H // G)
        w = softmax_with_sink((q[:, a] @ k[:, g].T) * m["scale"], seen, t[p + "sink"][a])
        out[:, a] = w @ v[:, g]
    out = out * head_gates(t, p, h).view(n, H, 1)
    return out.reshape(n, H * D) @ t[p + "o"].T


def latent_rows(t, p, h, m, eps):
    """What a latent layer remembers of a token: the normed latent and the
    rotated key part."""
    n, R = h.shape[0], m["kv_rank"]
    w = h @ t[p + "dkv"].T
    c = rms(w[:, :R], eps) * t[p + "dkv.norm"]
    return c, rotate_pairs(w[:, R:].view(n, 1, m["rot_dim"]), m["rot"])[:, 0]


def latent_attention(t, p, h, m, rows):
    n = h.shape[0]
    H, D, DR, DV = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = rows
    q = (h @ t[p + "q"].T).view(n, H, D + DR)
    qr = rotate_pairs(q[:, :, D:], m["rot"])
    k = (c @ t[p + "uk"].T).view(n, H, D)
    v = (c @ t[p + "uv"].T).view(n, H, DV)
    seen = visible(n, (m.get("mask") or {}).get("size"))
    out = torch.zeros(n, H, DV, dtype=F64)
    for a in range(H):
        s = (q[:, a, :D] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"]
        out[:, a] = softmax_with_sink(s, seen, t[p + "sink"][a]) @ v[:, a]
    out = out * head_gates(t, p, h).view(n, H, 1)
    return out.reshape(n, H * DV) @ t[p + "o"].T


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_recurrence(q, k, v, beta, decay):
    """q, k [n, H, D] unit vectors, v [n, H, DV], beta and decay [n, H]: the
    outputs [n, H, DV] and the last state [H, D, DV]."""
    n, H, D = k.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64)
    out = torch.zeros(n, H, v.shape[2], dtype=F64)
    for r in range(n):
        S = decay[r].view(H, 1, 1) * S
        u = beta[r].view(H, 1) * (v[r] - (S * k[r].view(H, D, 1)).sum(1))
        S = S + k[r].view(H, D, 1) * u.view(H, 1, -1)
        out[r] = (S * q[r].view(H, D, 1)).sum(1)
    return out, S


def gated_delta(t, p, h, m, eps):
    """A [dim, vdim] memory per head with ONE decay per head and token,
    corrected towards v by the part of v it does not hold yet."""
    n = h.shape[0]
    H, G, D, DV = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(causal_conv(h @ t[p + "q"].T, t[p + "q.conv"])).view(n, G, D)
    k = silu(causal_conv(h @ t[p + "k"].T, t[p + "k.conv"])).view(n, G, D)
    v = silu(causal_conv(h @ t[p + "v"].T, t[p + "v.conv"])).view(n, H, DV)
    of = torch.tensor([a // (H // G) for a in range(H)])       # a head's q/k head
    beta = sigmoid(h @ t[p + "b"].T)
    decay = torch.exp(-torch.exp(t[p + "A_log"]) * softplus(h @ t[p + "a"].T + t[p + "dt_bias"]))
    out, _ = delta_recurrence((unit(q) * D ** -0.5)[:, of], unit(k)[:, of], v, beta, decay)
    y = (rms(out, eps) * t[p + "norm"]).reshape(n, H * DV) * silu(h @ t[p + "g"].T)
    return y @ t[p + "o"].T


def dense_ff(t, p, h):
    return (silu(h @ t[p + "gate"].T) * (h @ t[p + "up"].T)) @ t[p + "down"].T


def forward(cfg, t, ids, layer_outputs=None):
    """Logits [n, vocab] of one whole sequence; t maps checkpoint names to
    float64 tensors."""
    eps = cfg["norm"]["eps"]
    x = t["embed"][torch.as_tensor(ids)]
    latents = {}
    for i, lc in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lc["mixer"]
        if lc["type"] == "attention":
            y = conv_attention(t, p + "mix.", x, m, eps)
        elif lc["type"] == "delta":
            y = gated_delta(t, p + "mix.", x, m, eps)
        else:
            if m.get("kv_from") is None:
                latents[i] = latent_rows(t, p + "mix.", x, m, eps)
            y = latent_attention(t, p + "mix.", x, m, latents[i if m.get("kv_from") is None
                                                              else m["kv_from"]])
        x = x + rms(y, eps) * t[p + "norm1"]
        if lc.get("mlp"):
            x = x + rms(dense_ff(t, p + "mlp.", x), eps) * t[p + "norm2"]
        if layer_outputs is not None:
            layer_outputs.append(x.clone())
    return (rms(x, eps) * t["final.norm"]) @ t["embed"].T * cfg["logit_scale"]


def greedy(cfg, t, ids, n):
    """n greedy continuations of ids, each from a whole forward pass."""
    ids, out = list(ids), []
    for _ in range(n):
        nxt = int(forward(cfg, t, ids)[-1].argmax())
        out.append(nxt)
        ids.append(nxt)
    return out
