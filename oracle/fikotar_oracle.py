"""Fikotar, restated plainly: float64, one function per mechanism, whole sequences at once (no cache, no state, no batching), so that
nothing here shares code or structure with the package.  `cfg` is the parsed config.json, `w` maps checkpoint names to tensors.

    x = embed[token];   layer: h = norm1(x), x += (left_scale * attention(h) + right_scale * retention(h)) + experts(h)
    logits = logit_scale * head (final norm(x))
    norm(x) = (x - mean) / sqrt(variance + eps) * w + b
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


# ---- what queries, keys and values pass ---------------------------------------------------------------------------------------
def causal_conv(u, taps):
    """u (T, C), taps (C, N): y[t, c] = sum_n taps[c, n] u[t - (N - 1) + n, c], zeros ahead of the first token."""
    t, n = u.shape[0], taps.shape[1]
    y = torch.zeros_like(u)
    for back in range(n):
        if back < t:
            y[back:] += taps[:, n - 1 - back] * u[:t - back]
    return y


def frequencies(dims, base, scaling=None):
    """One frequency per pair; `scaling` divides the slow ones by `factor` and blends in a band of wavelengths."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            turn = 2.0 * math.pi / f
            low, high, orig = scaling["low"], scaling["high"], scaling["original"]
            if turn > orig / low:
                f = f / scaling["factor"]
            elif turn >= orig / high:
                s = (orig / turn - low) / (high - low)
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def turned(x, pos, rot):
    """x (T, heads, size): pairs (i, i + dims / 2) of each head's first `dims` entries turned by position * frequency."""
    if not rot or not rot["dims"]:
        return x
    half = rot["dims"] // 2
    a = pos.to(F64)[:, None] * frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


# ---- attention -----------------------------------------------------------------------------------------------------------------
def sees(pos_q, pos_k, window, keep):
    """Which keys a query sees: itself and the window - 1 before it, and the sequence's first `keep` tokens; nothing ahead of it."""
    far = pos_q[:, None] - pos_k[None, :]
    near = far < window if window else far >= 0
    return (far >= 0) & (near | (pos_k[None, :] < keep))


def sink_softmax_readout(q, k, v, mask, scale, sink):
    """One head.  The softmax's sum has one more term exp(sink), which has no value (sink None: it has not)."""
    s = torch.where(mask, (q @ k.T) * scale, torch.full((), -math.inf, dtype=q.dtype))
    top = s.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.clamp(top, min=float(sink))
    e = torch.exp(s - top)
    total = e.sum(-1, keepdim=True) + (torch.exp(sink - top) if sink is not None else 0.0)
    return (e / total) @ v


def prepared(h, w, p, m, eps):
    """(queries (T, H, D), keys (T, G, D), values (T, G, E)) of a window attention: projected, convolved, turned, queries and keys normed."""
    t, pos = h.shape[0], torch.arange(h.shape[0])
    q, k, v = (h @ w[p + n].T for n in "qkv")
    if m.get("conv"):
        q, k, v = (causal_conv(u, w[p + n + ".conv"]) for u, n in ((q, "q"), (k, "k"), (v, "v")))
    q, k = q.view(t, m["heads"], m["dim"]), k.view(t, m["kv_heads"], m["dim"])
    return unit_rms(turned(q, pos, m.get("rot")), eps), unit_rms(turned(k, pos, m.get("rot")), eps), v.view(t, m["kv_heads"], m["vdim"])


def attention(h, w, p, m, eps):
    q, k, v = prepared(h, w, p, m, eps)
    mask = m.get("mask") or {}
    pos = torch.arange(h.shape[0])
    seen = sees(pos, pos, mask.get("size"), mask.get("keep_first", 0))
    of = lambda j: j // (m["heads"] // m["kv_heads"])
    heads = [sink_softmax_readout(q[:, j], k[:, of(j)], v[:, of(j)], seen, m["scale"], w[p + "sink"][j]) for j in range(m["heads"])]
    return torch.cat(heads, -1) @ w[p + "o"].T


# ---- retention -----------------------------------------------------------------------------------------------------------------
def decayed_memory(q, k, v, decay, start=None):
    """One head: S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t.  Returns (o (T, vdim), S after the last token)."""
    s = torch.zeros(k.shape[1], v.shape[1], dtype=q.dtype) if start is None else start
    out = []
    for t in range(q.shape[0]):
        s = decay * s + k[t][:, None] * v[t][None, :]
        out.append(q[t] @ s)
    return torch.stack(out), s


def retention_memory(q, k, v, pos, rot, decays):
    """q, k (T, H, D), v (T, H, E) as projected -> every head's read-out (T, H, E): turned, keys times D^(-1/2)."""
    q, k = turned(q, pos, rot), turned(k, pos, rot) * k.shape[2] ** -0.5
    return torch.stack([decayed_memory(q[:, j], k[:, j], v[:, j], decays[j])[0] for j in range(q.shape[1])], 1)


def retention(h, w, p, m, eps):
    t, n, d, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = (h @ w[p + "q"].T).view(t, n, d), (h @ w[p + "k"].T).view(t, n, d), (h @ w[p + "v"].T).view(t, n, e)
    o = unit_rms(retention_memory(q, k, v, torch.arange(t), m.get("rot"), m["decay"]), eps).reshape(t, n * e)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---- feed-forward --------------------------------------------------------------------------------------------------------------
def glu(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def chosen(logits, top):
    """(expert ids, their weights: the softmax over the chosen logits) of one token."""
    ids = sorted(range(len(logits)), key=lambda e: (-float(logits[e]), e))[:top]
    return ids, torch.softmax(logits[ids], 0)


def experts(h, w, p, mlp):
    z = h @ w[p + "router"].T
    out = torch.zeros(h.shape[0], w[p + "e0.down"].shape[0], dtype=h.dtype)
    for t in range(h.shape[0]):
        ids, share = chosen(z[t], mlp["router"]["top"])
        for e, s in zip(ids, share):
            out[t] += s * glu(h[t], w, f"{p}e{e}.")
    if mlp.get("shared"):
        out = out + torch.sigmoid(h @ w[p + "shared.sg"].T) * glu(h, w, p + "shared.")
    return out


# ---- the stack -----------------------------------------------------------------------------------------------------------------
def forward(cfg, w, tokens, streams=None):
    """float64 logits (T, vocab) of one sequence from its first token; `streams`, a list, takes the residual stream after every layer."""
    w = {k: v.to(F64) if v.is_floating_point() else v for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(list(tokens))]
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps)
        y = m["left_scale"] * attention(h, w, p + "mix.left.", m["left"], eps) + m["right_scale"] * retention(h, w, p + "mix.right.", m["right"], eps)
        if layer.get("mlp"):
            y = y + experts(h, w, p + "mlp.", layer["mlp"])
        x = x + y
        if streams is not None:
            streams.append(x)
    return layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["head"].T * cfg["logit_scale"]
