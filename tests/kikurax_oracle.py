"""Plain float64 oracle of the Kikurax design, one function per mechanism.

Written from the design's equations only: whole sequences, dense attention
rows, token-by-token recurrences, a per-token loop over chosen experts. It
shares no code with the engine, its ops or their torch reference forms, reads
a checkpoint's tensors by their checkpoint names, and knows nothing of pages,
slots, portions or batches.

Notation: W width, n tokens, x the residual stream [n, W], h a sublayer's
normed input, positions 0 .. n-1.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, w, eps, groups):
    """The vector in `groups` equal consecutive parts, each divided by its own
    root mean square, the whole times w."""
    n, W = x.shape
    return rms(x.reshape(n, groups, W // groups), eps).reshape(n, W) * w


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


def frequencies(rot):
    """base^(-2i/dims), then the wavelength-dependent slowdown: long waves
    divided by factor, short ones kept, a linear blend between."""
    dims, sc = rot["dims"], rot.get("scaling")
    out = []
    for i in range(dims // 2):
        f = rot["base"] ** (-2.0 * i / dims)
        if sc:
            wave = 2.0 * math.pi / f
            lo_wave, hi_wave = sc["original"] / sc["low"], sc["original"] / sc["high"]
            if wave > lo_wave:
                f = f / sc["factor"]
            elif wave >= hi_wave:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate_half(x, rot, first_pos=0):
    """x [n, heads, d]: pair (i, i + dims/2) of the first `dims` channels turns
    by position * f_i; the rest passes."""
    half = rot["dims"] // 2
    out = x.clone()
    pos = torch.arange(first_pos, first_pos + x.shape[0], dtype=F64).view(-1, 1)
    for i, f in enumerate(frequencies(rot)):
        c, s = torch.cos(pos * f), torch.sin(pos * f)
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def causal_conv(u, w, b=None):
    """u [n, C], w [C, taps]: y_t = b + sum_j w[:, j] * u_(t - taps + 1 + j),
    zeros before the start."""
    n, C = u.shape
    taps = w.shape[1]
    y = torch.zeros(n, C, dtype=F64)
    for j in range(taps):
        back = taps - 1 - j
        if back < n:
            y[back:] += w[:, j] * u[:n - back]
    return y if b is None else y + b


def query_temperature(pos, coef, every):
    return 1.0 + coef * math.log(math.floor((pos + 1) / every) + 1.0)


def sigmoid_attention(t, p, h, m, eps):
    """Unrotated grouped-head attention whose weights are sigmoids of the
    scores (not normalised over keys), with unit-norm q and k, a position-
    dependent query temperature and an elementwise output gate."""
    n = h.shape[0]
    H, G, D, DV = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ t[p + "q"].T).view(n, H, D), eps)
    k = rms((h @ t[p + "k"].T).view(n, G, D), eps)
    v = (h @ t[p + "v"].T).view(n, G, DV)
    if m.get("q_temp"):
        q = q * torch.tensor([query_temperature(i, m["q_temp"]["coef"], m["q_temp"]["every"])
                              for i in range(n)], dtype=F64).view(n, 1, 1)
    seen = torch.ones(n, n, dtype=F64).tril()
    out = torch.zeros(n, H, DV, dtype=F64)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * m["scale"] + t[p + "pb"][a]
        out[:, a] = (sigmoid(s) * seen) @ v[:, g]
    y = out.reshape(n, H * DV) * sigmoid(h @ t[p + "g"].T)
    return y @ t[p + "o"].T


def gated_delta_rule(t, p, h, m, eps):
    """A [dim, vdim] memory per head that is decayed per key channel and
    corrected towards v by the part of v it does not hold yet."""
    n = h.shape[0]
    H, G, D, DV = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(causal_conv(h @ t[p + "q"].T, t[p + "q.conv"])).view(n, G, D)
    k = silu(causal_conv(h @ t[p + "k"].T, t[p + "k.conv"])).view(n, G, D)
    v = silu(causal_conv(h @ t[p + "v"].T, t[p + "v.conv"])).view(n, H, DV)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * D ** -0.5
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    beta = sigmoid(h @ t[p + "b"].T)
    z = (h @ t[p + "a1"].T) @ t[p + "a2"].T + t[p + "dt_bias"]
    decay = torch.exp(-torch.exp(t[p + "A_log"]).view(1, H, 1) * softplus(z).view(n, H, D))
    of = torch.tensor([a // (H // G) for a in range(H)])       # a head's q/k head
    out = torch.zeros(n, H, DV, dtype=F64)
    S = torch.zeros(H, D, DV, dtype=F64)
    for r in range(n):
        S = decay[r].view(H, D, 1) * S
        held = (S * k[r, of].view(H, D, 1)).sum(1)
        u = beta[r].view(H, 1) * (v[r] - held)
        S = S + k[r, of].view(H, D, 1) * u.view(H, 1, DV)
        out[r] = (S * q[r, of].view(H, D, 1)).sum(1)
    gate = sigmoid((h @ t[p + "g1"].T) @ t[p + "g2"].T)
    y = (rms(out, eps) * t[p + "norm"]).reshape(n, H * DV) * gate
    return y @ t[p + "o"].T


def parallel_mixer(t, p, h, m, eps):
    left = sigmoid_attention(t, p + "left.", h, m["left"], eps)
    right = gated_delta_rule(t, p + "right.", h, m["right"], eps)
    return 0.5 * (rms(left, eps) * t[p + "left.out"] + rms(right, eps) * t[p + "right.out"])


def mamba2(t, p, h, m, eps):
    """State-space duality: one decay per head and token, B and C shared by
    the heads of a group, the gate before a norm on equal parts."""
    n = h.shape[0]
    H, DV, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * DV
    w = h @ t[p + "in"].T
    z, xbc, dt = w[:, :inner], w[:, inner:2 * inner + 2 * G * N], w[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, t[p + "conv"], t[p + "conv.b"]))
    x = xbc[:, :inner].view(n, H, DV)
    B = xbc[:, inner:inner + G * N].view(n, G, N)
    C = xbc[:, inner + G * N:].view(n, G, N)
    dt = softplus(dt + t[p + "dt_bias"])
    of = torch.tensor([a // (H // G) for a in range(H)])       # a head's group
    rate = torch.exp(t[p + "A_log"])
    out = torch.zeros(n, H, DV, dtype=F64)
    S = torch.zeros(H, N, DV, dtype=F64)
    for r in range(n):
        S = torch.exp(-rate * dt[r]).view(H, 1, 1) * S + \
            dt[r].view(H, 1, 1) * B[r, of].view(H, N, 1) * x[r].view(H, 1, DV)
        out[r] = (S * C[r, of].view(H, N, 1)).sum(1) + t[p + "D"].view(H, 1) * x[r]
    y = out.reshape(n, inner) * silu(z)
    return group_norm(y, t[p + "norm"], eps, m["norm_groups"]) @ t[p + "o"].T


def rotary_attention(t, p, h, m, eps, v_first):
    """Biased projections, rotation then unit norm of q and k, a temperature
    per head, tanh-capped scores, a softmax with 1 added to the denominator,
    and values blended with the first blending layer's. Returns the output
    and this layer's own values (before any blend)."""
    n = h.shape[0]
    H, G, D, DV = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ t[p + "q"].T + t[p + "q.b"]).view(n, H, D)
    k = (h @ t[p + "k"].T + t[p + "k.b"]).view(n, G, D)
    own = (h @ t[p + "v"].T + t[p + "v.b"]).view(n, G, DV)
    v = own
    if m.get("v_mix") and v_first is not None:
        lam = float(t[p + "vmix"])
        v = (1.0 - lam) * own + lam * v_first
    q, k = rms(rotate_half(q, m["rot"]), eps), rms(rotate_half(k, m["rot"]), eps)
    cap = m.get("softcap")
    seen = torch.ones(n, n, dtype=torch.bool).tril()
    out = torch.zeros(n, H, DV, dtype=F64)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * m["scale"] * t[p + "temp"][a]
        if cap:
            s = cap * torch.tanh(s / cap)
        s = s.masked_fill(~seen, float("-inf"))
        top = torch.clamp(s.max(dim=1, keepdim=True).values, min=0.0)
        e = torch.exp(s - top)
        out[:, a] = (e @ v[:, g]) / (torch.exp(-top) + e.sum(dim=1, keepdim=True))
    return out.reshape(n, H * DV) @ t[p + "o"].T, own


def clamped_expert(t, p, h, limit):
    g = torch.clamp(h @ t[p + "gate"].T, max=limit)
    u = torch.clamp(h @ t[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ t[p + "down"].T


def routed_experts(t, p, h, mlp):
    """The `top` largest biased router logits; weights are the softmax over
    the chosen logits only."""
    E, top, limit = mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["limit"]
    z = h @ t[p + "router"].T + t[p + "router.b"]
    out = torch.zeros_like(h)
    for row in range(h.shape[0]):
        chosen = sorted(range(E), key=lambda e: (-float(z[row, e]), e))[:top]
        wgt = torch.softmax(z[row, chosen], dim=0)
        for w, e in zip(wgt, chosen):
            out[row] += w * clamped_expert(t, f"{p}e{e}.", h[row:row + 1], limit)[0]
    return out


def forward(cfg, t, ids, layer_outputs=None):
    """Logits [n, vocab] of one whole sequence; t maps checkpoint names to
    float64 tensors."""
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = t["embed"][torch.as_tensor(ids)] * cfg["embedding"]["scale"]
    v_first = None
    for i, lc in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lc["mixer"]
        h = group_norm(x, t[p + "norm1"], eps, groups)
        if lc["type"] == "parallel":
            y = parallel_mixer(t, p + "mix.", h, m, eps)
        elif lc["type"] == "mamba2":
            y = mamba2(t, p + "mix.", h, m, eps)
        else:
            y, own = rotary_attention(t, p + "mix.", h, m, eps, v_first)
            if m.get("v_mix") and v_first is None:
                v_first = own
        x = x + y
        if lc.get("mlp"):
            x = x + routed_experts(t, p + "mlp.", group_norm(x, t[p + "norm2"], eps, groups), lc["mlp"])
        if layer_outputs is not None:
            layer_outputs.append(x.clone())
    return group_norm(x, t["final.norm"], eps, groups) @ t["embed"].T


def greedy(cfg, t, ids, n):
    """n greedy continuations of ids, each from a whole forward pass."""
    ids, out = list(ids), []
    for _ in range(n):
        nxt = int(forward(cfg, t, ids)[-1].argmax())
        out.append(nxt)
        ids.append(nxt)
    return out
