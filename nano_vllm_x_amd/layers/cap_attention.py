"""Causal attention with grouped key/value heads and separate key and value sizes over per-token key and value rows in the
token cache: SoftcapAttention (rotary positions on a leading part of each head, unit-mean-square values, capped scores) and
NormedAttention (query/key RMS norms, optional rotation of keys AND values, window, distance penalty, output gate, borrowed
keys and values), TiedAttention (one cached row per token and head is key and value, linear distance penalty, chunks of positions),
ConvAttention (a short convolution over time ahead of rotation and norm, a sink per head, a window behind which the first tokens stay)."""
from __future__ import annotations

import torch
from torch import nn

from .. import ops
from .rotary_embedding import rotary_frequencies


class SoftcapAttention(nn.Module):
    """q = W_q h, k = W_k h (rotated by position), v = W_v h (each head divided by its root mean square, cached so);
    score = scale * q . k, then cap * tanh(score / cap) (cap None or 0: none), softmax over the causal prefix, W_o on the
    concatenated heads.  Query head j reads key/value head j // (heads / kv_heads).  `rot` = {dims, base, scaling | None}.
    The three projections are one matrix product; the cache holds two rows per token under `cache_names`."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, rot: dict, scale: float, softcap, eps: float, cache_names):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("query heads must be a multiple of key/value heads")
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.scale, self.softcap, self.eps = float(scale), float(softcap or 0.0), eps
        self.k_name, self.v_name = cache_names
        self.rot_dims = int(rot["dims"]) if rot else 0
        if self.rot_dims % 2 or self.rot_dims > dim:
            raise ValueError("the rotated part of a head must be even and within the head")
        if self.rot_dims:
            freq, self.mag = rotary_frequencies(self.rot_dims, rot["base"], rot.get("scaling"))
            self.register_buffer("freq", freq.to(torch.float64), persistent=False)
        else:
            self.freq, self.mag = None, 1.0
        self.qkv_proj = nn.Linear(width, heads * dim + kv_heads * (dim + vdim), bias=False)     # rows: q | k | v
        self.o_proj = nn.Linear(heads * vdim, width, bias=False)

    def cache_rows(self) -> dict:
        return {self.k_name: self.kv_heads * self.dim, self.v_name: self.kv_heads * self.vdim}

    def forward(self, h: torch.Tensor, positions: torch.Tensor, md) -> torch.Tensor:
        k_cache, v_cache = md.cache.latent(self.k_name), md.cache.latent(self.v_name)
        q = ops.rope_vnorm_store(self.qkv_proj(h), positions, self.freq, self.mag, self.rot_dims, self.eps, md.out_slots, k_cache, v_cache,
                                 self.heads, self.kv_heads, self.dim, self.vdim)
        o = ops.softcap_attn(q, k_cache, v_cache, md.kv_indices, md.kv_start, md.kv_len, md.layout, self.scale, self.softcap, self.heads,
                             self.kv_heads, self.dim, self.vdim)
        return self.o_proj(o)


class NormedAttention(nn.Module):
    """Softmax attention whose queries and keys pass an RMS norm, with these parts, each optional:
      qk_norm   "head": every q and k head by its own root mean square, weight (dim) shared by the heads; "row": all heads of a
                token's q (and of its k) at once, weights of heads * dim and kv_heads * dim entries; "none"
      rot       {dims, base, interleaved, scaling}: the first `dims` of every q and k head turned by position * f_m, f_m = base^(-2m/dims)
                (stretched by `scaling`, see rotary_frequencies; one that changes the magnitude is refused), pair m being (m, m + dims/2),
                or (2m, 2m + 1) if interleaved
      rotate_values   the value of position j is cached turned by j * base^(-2m/vdim) over all of vdim (same pair layout) and a
                head's read-out at position i is turned back by i, so every value enters in the frame of its distance to i
      softcap   scores through cap tanh(. / cap);   window   a token sees itself and the window - 1 before it
      distance_penalty   r1_h ln(1 + r2_h (i - j)) taken off the score (r1, r2: one number per head)
      sink_score   the softmax's sum has one more term exp(sink_score) without a value (0.0: one is added to the denominator)
      out_gate  the concatenated heads times sigmoid(W_g h): True, one gate per element; "head", one per head
      bias      q, k, v projections with biases;   o_bias   the output projection too
      kv_source (k_name, v_name) of another layer's cache rows: no key/value projections here, that layer's rows are read.
    The projections q | k | v | g are rows of ONE matrix product: the module's own (`forward`), or a wider one that the caller
    shares between several mechanisms (`attend`, with the first column of this module's block)."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, eps: float, cache_names, qk_norm: str = "head",
                 rot: dict | None = None, rotate_values: bool = False, softcap=None, window=None, distance_penalty: bool = False,
                 out_gate=False, bias: bool = False, kv_source=None, own_proj: bool = True, sink_score=None, o_bias: bool = False):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("query heads must be a multiple of key/value heads")
        if qk_norm not in ("head", "row", "none"):
            raise ValueError(f"unknown query/key norm {qk_norm!r}")
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.scale, self.softcap, self.eps, self.window = float(scale), float(softcap or 0.0), eps, int(window or 0)
        if out_gate not in (False, True, "head"):
            raise ValueError(f"unknown output gate {out_gate!r}")
        self.qk_norm, self.out_gate, self.borrows = qk_norm, out_gate, kv_source is not None
        self.sink_score = None if sink_score is None else float(sink_score)
        self.k_name, self.v_name = kv_source if self.borrows else cache_names
        self.rot_dims = int(rot["dims"]) if rot else 0
        self.interleaved = bool(rot and rot.get("interleaved"))
        if self.rot_dims % 2 or self.rot_dims > dim:
            raise ValueError("the rotated part of a head must be even and within the head")
        if rotate_values and (not rot or vdim % 2):
            raise ValueError("rotated values need a rotation base and an even value size")
        freq = None
        if self.rot_dims:
            freq, mag = rotary_frequencies(self.rot_dims, rot["base"], rot.get("scaling"))
            if mag != 1.0:
                raise NotImplementedError("a frequency scaling that changes the rotation's magnitude is not built for this attention")
        self.register_buffer("freq", freq.to(torch.float64) if self.rot_dims else None, persistent=False)
        self.register_buffer("vfreq", rotary_frequencies(vdim, rot["base"])[0].to(torch.float64) if rotate_values else None, persistent=False)
        n_w = {"head": (dim, dim), "row": (heads * dim, kv_heads * dim), "none": (0, 0)}[qk_norm]
        if n_w[0]:
            self.q_norm = nn.Parameter(torch.zeros(n_w[0], dtype=torch.float32))
            if not self.borrows:
                self.k_norm = nn.Parameter(torch.zeros(n_w[1], dtype=torch.float32))
        if distance_penalty:
            self.r1 = nn.Parameter(torch.zeros(heads, dtype=torch.float32))
            self.r2 = nn.Parameter(torch.zeros(heads, dtype=torch.float32))
        else:
            self.r1 = self.r2 = None
        # columns of this module's block of a projection: q | k | v | g
        self.q_cols = heads * dim
        self.k_cols = 0 if self.borrows else kv_heads * dim
        self.v_cols = 0 if self.borrows else kv_heads * vdim
        self.g_cols = heads if out_gate == "head" else heads * vdim if out_gate else 0
        self.proj_rows = self.q_cols + self.k_cols + self.v_cols + self.g_cols
        self.has_bias = bias
        if own_proj:
            self.in_proj = nn.Linear(width, self.proj_rows, bias=bias)
            if bias:
                nn.init.zeros_(self.in_proj.bias)      # the gate's rows have no bias: theirs stays zero
        self.o_proj = nn.Linear(heads * vdim, width, bias=o_bias)

    def cache_rows(self) -> dict:
        return {} if self.borrows else {self.k_name: self.kv_heads * self.dim, self.v_name: self.kv_heads * self.vdim}

    def attend(self, x: torch.Tensor, col0: int, positions: torch.Tensor, md) -> torch.Tensor:
        k_cache, v_cache = md.cache.latent(self.k_name), md.cache.latent(self.v_name)
        k0 = col0 + self.q_cols
        v0 = k0 + self.k_cols
        g0 = v0 + self.v_cols
        own = not self.borrows
        q, v_turn = ops.attn_prep_store(x, (col0, k0, v0), positions, getattr(self, "q_norm", None), getattr(self, "k_norm", None), self.qk_norm, self.eps,
                                self.freq, self.rot_dims, self.interleaved, self.vfreq, md.out_slots if own else None,
                                k_cache if own else None, v_cache if own else None, self.heads, self.kv_heads if own else 0, self.dim, self.vdim)
        o = ops.softcap_attn(q, k_cache, v_cache, md.kv_indices, md.kv_start, md.kv_len, md.layout, self.scale, self.softcap, self.heads,
                             self.kv_heads, self.dim, self.vdim, window=self.window, r1=self.r1, r2=self.r2, v_turn=v_turn,
                             v_interleaved=self.interleaved, gate=x[:, g0:g0 + self.g_cols] if self.out_gate else None,
                             sink_score=self.sink_score)
        return self.o_proj(o)

    def forward(self, h: torch.Tensor, positions: torch.Tensor, md) -> torch.Tensor:
        return self.attend(self.in_proj(h), 0, positions, md)


def geometric_slopes(heads: int, base: float = 8.0):
    """One slope per head for a linear distance penalty: 2^(-base (h + 1) / heads), h = 0 .. heads - 1."""
    return [2.0 ** (-base * (h + 1) / heads) for h in range(heads)]


class TiedAttention(nn.Module):
    """Grouped-head softmax attention whose VALUES ARE ITS KEYS as projected: q = W_q h, k = W_k h (optional biases); queries and keys are
    scored after an RMS norm per head (weights of `dim` entries shared by the heads), the read-out sums the keys as they came out of the
    projection.  score = scale * q . k - slopes[h] * (i - j) (slopes None: no penalty); `window` > 0: a token sees itself and the window
    - 1 before it; `chunk` > 0: it sees the earlier tokens of its own chunk of positions, i // chunk == j // chunk.
    The cache holds ONE row per token under `cache_name`, the raw key, and beside it one float32 number per key/value head, the
    reciprocal root mean square of the key: the norm's weight goes into the queries, the number multiplies the score, and neither the
    norm nor a second row costs cache or bandwidth.  The projections q | k are rows of one matrix product.
    `at`: the name of another set of cache rows (a layer that runs several times over a sequence has one per run)."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, scale: float, eps: float, cache_name, slopes=None, window=None, chunk=None,
                 bias: bool = False, o_bias: bool = False):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("query heads must be a multiple of key/value heads")
        if window and chunk:
            raise ValueError("a window or chunks, not both")
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, dim
        self.scale, self.eps, self.window, self.chunk, self.cache_name = float(scale), eps, int(window or 0), int(chunk or 0), cache_name
        self.q_cols, self.k_cols = heads * dim, kv_heads * dim
        self.in_proj = nn.Linear(width, self.q_cols + self.k_cols, bias=bias)      # rows: q | k
        self.q_norm = nn.Parameter(torch.zeros(dim, dtype=torch.float32))
        self.k_norm = nn.Parameter(torch.zeros(dim, dtype=torch.float32))
        if slopes is not None and len(slopes) != heads:
            raise ValueError(f"{heads} heads need {heads} slopes, got {len(slopes)}")
        self.register_buffer("slopes", torch.tensor([float(s) for s in slopes], dtype=torch.float32) if slopes is not None else None, persistent=False)
        self.o_proj = nn.Linear(heads * dim, width, bias=o_bias)

    def cache_rows(self, at=None) -> dict:
        n = self.cache_name if at is None else at
        return {(n, "k"): self.kv_heads * self.dim, (n, "rn"): (self.kv_heads, torch.float32)}

    def forward(self, h: torch.Tensor, md, at=None) -> torch.Tensor:
        n = self.cache_name if at is None else at
        rows, rn = md.cache.latent((n, "k")), md.cache.latent((n, "rn"))
        q = ops.tied_prep_store(self.in_proj(h), (0, self.q_cols), self.q_norm, self.k_norm, self.eps, md.out_slots, rows, rn, self.heads,
                                self.kv_heads, self.dim)
        o = ops.softcap_attn(q, rows, rows, md.kv_indices, md.kv_start, md.kv_len, md.layout, self.scale, 0.0, self.heads, self.kv_heads, self.dim,
                             self.dim, window=self.window, chunk=self.chunk, slopes=self.slopes, k_rn=rn)
        return self.o_proj(o)


class ConvAttention(nn.Module):
    """Grouped-head softmax attention whose queries, keys and values pass a short causal convolution per channel between their projection
    and everything else: u_t = sum_j w[j] x_(t - taps + 1 + j), zeros before the sequence's start.  Then queries and keys are rotated by
    position (the first rot dims of each head, halves layout) and divided by their root mean square per head (no weight).
      window      a token sees itself and the window - 1 before it (None: all before it), and the sequence's first `keep_first` tokens
      sinks       True: the softmax's sum has one more term exp(sink_h) without a value, a learned number per head
      out_mul     the read-out is multiplied by this number before the output projection
    The module is a block of a layer that shares its matrix products between several mechanisms: `attend` reads q | k | v from `col0` of the
    layer's input product on and writes its heads into `out`, the columns of the layer's output product that belong to it.  The rotation
    comes from the step's table (see TurnTables).  State: the convolution's last taps - 1 inputs (float32), under (state_name, "conv")."""

    def __init__(self, heads: int, kv_heads: int, dim: int, vdim: int, taps: int, scale: float, eps: float, cache_names, state_name, rot_key=None,
                 rot_dims: int = 0, window=None, keep_first: int = 0, sinks: bool = True, out_mul: float = 1.0):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("query heads must be a multiple of key/value heads")
        if taps < 1:
            raise ValueError("a convolution has at least one tap")
        if rot_dims % 2 or rot_dims > dim:
            raise ValueError("the rotated part of a head must be even and within the head")
        self.heads, self.kv_heads, self.dim, self.vdim, self.taps = heads, kv_heads, dim, vdim, taps
        self.scale, self.eps, self.out_mul, self.rot_key = float(scale), eps, float(out_mul), rot_key
        self.window, self.keep_first = int(window or 0), int(keep_first or 0) if window else 0
        self.k_name, self.v_name = cache_names
        self.state_name = state_name
        self.q_cols, self.k_cols, self.v_cols = heads * dim, kv_heads * dim, kv_heads * vdim
        self.proj_rows, self.out_cols = self.q_cols + self.k_cols + self.v_cols, heads * vdim
        self.conv_w = nn.Parameter(torch.zeros(taps, self.proj_rows, dtype=torch.float32))      # row j: the tap taps - 1 - j tokens back
        self.sinks = nn.Parameter(torch.zeros(heads, dtype=torch.float32)) if sinks else None

    def cache_rows(self) -> dict:
        return {self.k_name: self.k_cols, self.v_name: self.v_cols}

    def state_shapes(self) -> dict:
        return {(self.state_name, "conv"): (self.taps - 1, self.proj_rows)} if self.taps > 1 else {}

    def attend(self, x: torch.Tensor, col0: int, turn, md, out: torch.Tensor):
        k_cache, v_cache = md.cache.latent(self.k_name), md.cache.latent(self.v_name)
        q = ops.conv_attn_prep(x[:, col0:col0 + self.proj_rows], self.conv_w, md.cache.state((self.state_name, "conv")) if self.taps > 1 else None, md.layout,
                               turn, self.eps, md.out_slots, k_cache, v_cache, self.heads, self.kv_heads, self.dim, self.vdim)
        ops.softcap_attn(q, k_cache, v_cache, md.kv_indices, md.kv_start, md.kv_len, md.layout, self.scale, 0.0, self.heads, self.kv_heads, self.dim,
                         self.vdim, window=self.window, keep_first=self.keep_first, sinks=self.sinks, out_mul=self.out_mul, out=out)
