"""Zenedra, restated plainly: float64, one function per mechanism, whole sequences at once (no cache, no state, no batching), so that
nothing here shares code or structure with the package.  `cfg` is the parsed config.json, `w` maps checkpoint names to tensors.

    x = x0 = embed[token] + bigram row + pos row;   layer: x += mixer(norm1(x)), x += ff(norm2(x));   logits = head (final norm(x))
    norm(x) = x / rms(x) * (1 + w)
    layers start .. stop - 1 run `times` times with the same weights; ahead of each pass t:  x = W_in [x; x0] + step[t].
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64
GLU_SLOPE = 1.702


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_around_one(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ---- embedding --------------------------------------------------------------------------------------------------------------
def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Row of the pair table per token: a hash of (predecessor, token); the first token of a sequence has the extra row `buckets`."""
    return [buckets if i == 0 else (tokens[i - 1] * mul_prev + tokens[i] * mul_cur) % buckets for i in range(len(tokens))]


def embedding(tokens, w, cfg):
    x = w["embed"][torch.as_tensor(tokens)]
    pair = (cfg.get("embedding") or {}).get("bigram")
    if pair:
        x = x + w["bigram"][torch.as_tensor(bigram_rows(list(tokens), pair["buckets"], pair["mul_prev"], pair["mul_cur"]))]
    return x + w["pos"][:len(tokens)]


# ---- mixers -----------------------------------------------------------------------------------------------------------------
def distance_slopes(heads):
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=F64)


def chunk_softmax_readout(q, k, v, pos_q, pos_k, scale, slope, chunk):
    """One head: scores scale * q . k - slope * (i - j); position i sees j <= i inside its own chunk (positions i // chunk equal;
    chunk None: all j <= i)."""
    far = (pos_q[:, None] - pos_k[None, :]).to(q.dtype)
    s = (q @ k.T) * scale - slope * far
    seen = far >= 0
    if chunk:
        seen = seen & ((pos_q[:, None] // chunk) == (pos_k[None, :] // chunk))
    return torch.softmax(torch.where(seen, s, torch.full_like(s, -math.inf)), -1) @ v


def attention(h, w, p, m, eps):
    """Grouped heads; the value of a token is its key as projected, the keys that are scored are normed per head, as the queries are."""
    t, hq, g, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    pos = torch.arange(t)
    q = rms((h @ w[p + "q"].T + w[p + "q.b"]).view(t, hq, d), eps) * w[p + "q.norm"]
    raw = (h @ w[p + "k"].T + w[p + "k.b"]).view(t, g, d)
    k = rms(raw, eps) * w[p + "k.norm"]
    slopes = distance_slopes(hq)
    chunk = (m.get("mask") or {}).get("size")
    heads = [chunk_softmax_readout(q[:, j], k[:, j // (hq // g)], raw[:, j // (hq // g)], pos, pos, m["scale"], slopes[j], chunk) for j in range(hq)]
    return torch.cat(heads, -1) @ w[p + "o"].T + w[p + "o.b"]


def channel_decay(z, tau):
    return torch.sigmoid(z) ** (1.0 / tau)


def channel_decay_memory(q, k, v, alpha, start=None):
    """One head: S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t.  Returns (o (T, vdim), S after the last token)."""
    s = torch.zeros(k.shape[1], v.shape[1], dtype=q.dtype) if start is None else start
    out = []
    for t in range(q.shape[0]):
        s = alpha[t][:, None] * s + k[t][:, None] * v[t][None, :]
        out.append(q[t] @ s)
    return torch.stack(out), s


def gla(h, w, p, m, eps):
    t, n, d, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(t, n, d) * d ** -0.5
    k = (h @ w[p + "k"].T).view(t, n, d)
    v = (h @ w[p + "v"].T).view(t, n, e)
    alpha = channel_decay(((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]).view(t, n, d), m["tau"])
    o = torch.stack([channel_decay_memory(q[:, j], k[:, j], v[:, j], alpha[:, j])[0] for j in range(n)], 1)
    o = (rms(o, eps) * w[p + "norm"]).reshape(t, n * e)
    g = h @ w[p + "g"].T
    return (o * g * torch.sigmoid(g)) @ w[p + "o"].T


def exp_gated_memory(q, k, v, i, f, start=None):
    """One head of the matrix memory with a log input gate i and a log forget gate f: m' = max(f + m, i) from m = 0,
    S' = e^(f + m - m') S + e^(i - m') k v^T, n' likewise with k, o = S'^T q / (max(|n' . q|, e^-m') + 1e-6)."""
    s, n, m = start if start is not None else (torch.zeros(k.shape[1], v.shape[1], dtype=q.dtype), torch.zeros(k.shape[1], dtype=q.dtype), 0.0)
    out = []
    for t in range(q.shape[0]):
        top = max(float(f[t]) + m, float(i[t]))
        keep, put = math.exp(float(f[t]) + m - top), math.exp(float(i[t]) - top)
        m = top
        s = keep * s + put * k[t][:, None] * v[t][None, :]
        n = keep * n + put * k[t]
        out.append((q[t] @ s) / (max(abs(float(n @ q[t])), math.exp(-m)) + 1e-6))
    return torch.stack(out), (s, n, m)


def mlstm(h, w, p, m, eps):
    t, n, d, e, cap = h.shape[0], m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q = (h @ w[p + "q"].T).view(t, n, d) * d ** -0.5
    k = (h @ w[p + "k"].T).view(t, n, d)
    v = (h @ w[p + "v"].T).view(t, n, e)
    i = cap * torch.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    f = torch.nn.functional.logsigmoid(cap * torch.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    o = torch.stack([exp_gated_memory(q[:, j], k[:, j], v[:, j], i[:, j], f[:, j])[0] for j in range(n)], 1)
    o = rms(o, eps).reshape(t, n * e) * w[p + "norm"]
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---- feed-forward -----------------------------------------------------------------------------------------------------------
def dense_ff(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def limited_glu(g, u, limit):
    g = torch.clamp(g, max=limit)
    return g * torch.sigmoid(GLU_SLOPE * g) * (torch.clamp(u, -limit, limit) + 1.0)


def expert(h, w, p, limit):
    return limited_glu(h @ w[p + "gate"].T, h @ w[p + "up"].T, limit) @ w[p + "down"].T


def route_logits(z, correction, router):
    """(ids, weights) of one token's logits z (list of floats): sigmoid scores, choice scores = score + correction, groups ranked by the
    sum of their two largest choice scores, the `top` experts of the kept groups with the largest choice scores, weights from the
    uncorrected scores."""
    n, top = router["experts"], router["top"]
    s = [1.0 / (1.0 + math.exp(-v)) for v in z]
    c = [a + b for a, b in zip(s, correction)]
    groups = router.get("groups")
    allowed = set(range(n))
    if groups:
        per = n // groups["count"]
        rank = sorted(range(groups["count"]), key=lambda g: -sum(sorted(c[g * per:(g + 1) * per], reverse=True)[:2]))
        allowed = {e for g in rank[:groups["keep"]] for e in range(g * per, (g + 1) * per)}
    ids = sorted(allowed, key=lambda e: -c[e])[:top]
    return ids, [s[e] * router.get("scale", 1.0) for e in ids]


def moe_ff(h, w, p, mlp):
    out = torch.zeros_like(h)
    z = h @ w[p + "router"].T
    for t in range(h.shape[0]):
        ids, wts = route_logits(z[t].tolist(), w[p + "correction"].tolist(), mlp["router"])
        for e, a in zip(ids, wts):
            out[t] += a * expert(h[t:t + 1], w, f"{p}e{e}.", mlp["expert"]["limit"])[0]
    if mlp.get("shared"):
        out = out + expert(h, w, p + "shared.", mlp["shared"]["limit"])
    return out


# ---- the stack --------------------------------------------------------------------------------------------------------------
def layer_order(n_layers, loop):
    """[(layer, pass or None)] in the order they run."""
    if not loop:
        return [(i, None) for i in range(n_layers)]
    a, b = loop["start"], loop["stop"]
    return ([(i, None) for i in range(a)] + [(i, t) for t in range(loop["times"]) for i in range(a, b)] + [(i, None) for i in range(b, n_layers)])


def forward(cfg: dict, weights: dict, tokens, layer_streams: list | None = None):
    """Logits (T, vocab) of one sequence computed whole.  `layer_streams`, a list, receives the residual stream after every layer run."""
    w = {k: (v.to(F64) if v.is_floating_point() else v) for k, v in weights.items()}
    eps, loop = cfg["norm"]["eps"], cfg.get("loop")
    x0 = embedding(list(tokens), w, cfg)
    x = x0
    mixers = {"gla": gla, "attention": attention, "mlstm": mlstm}
    for i, t in layer_order(len(cfg["layers"]), loop):
        if t is not None and i == loop["start"]:
            x = torch.cat([x, x0], -1) @ w["loop.in"].T + w["loop.step"][t]
        layer, p = cfg["layers"][i], f"l{i}."
        x = x + mixers[layer["type"]](norm_around_one(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            h = norm_around_one(x, w[p + "norm2"], eps)
            x = x + (dense_ff(h, w, p + "mlp.") if mlp["kind"] == "dense" else moe_ff(h, w, p + "mlp.", mlp))
        if layer_streams is not None:
            layer_streams.append(x)
    return norm_around_one(x, w["final.norm"], eps) @ w["head"].T
