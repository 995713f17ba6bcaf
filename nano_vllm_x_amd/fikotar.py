"""Fikotar: a decoder stack over a float32 residual stream whose layers have ONE norm and run everything side by side on it:
    x = embed[token];   h = norm1(x),  x <- x + (left_scale * attention(h) + right_scale * retention(h)) + experts(h)
    logits = logit_scale * head (final norm(x))               (norm: layer norm with weight and bias)
  attention   grouped heads behind a short causal convolution on queries, keys and values; rotary positions (frequencies stretched by
              wavelength bands), unit-mean-square queries and keys, a sliding window with kept first tokens, a learned sink per head;
  retention   linear attention with a constant decay per head, rotated queries and keys, unit-mean-square heads behind a silu gate;
  experts     a mixture of gated feed-forwards behind a softmax router (weights: the softmax over the chosen logits), beside a shared one
              behind a gate of one number per token; or absent.

config.json gives every size, the order of the layers and the constants; the mechanisms live in layers/ (cap_attention.py, recurrent.py,
moe.py) with their constants as arguments.  Because all of a layer reads the same h and ends in the same sum, a layer is TWO matrix
products around its kernels: one with the projections of both mixers and of the shared expert, one over the concatenated read-outs [left |
right | shared hidden] with their output matrices side by side (the scales and the shared gate are factors of the read-outs).  Norm,
router, scores, positions and angles, the recurrence and its state, and the stream are float32 in every activation format.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Iterable

import torch
from torch import nn

from . import distributed as tpd
from . import ops
from .layers.cap_attention import ConvAttention
from .layers.moe import GatedSharedExpert, GroupedSoftmaxMoE
from .layers.recurrent import Retention
from .layers.rotary_embedding import TurnTables

MIXERS = ("parallel",)


def _rot(m: dict):
    rot = m.get("rot")
    if not rot or not int(rot.get("dims") or 0):
        return None
    out = {"dims": int(rot["dims"]), "base": float(rot["base"])}
    if rot.get("scaling"):
        out["scaling"] = {k: float(v) for k, v in rot["scaling"].items()}
    return out


@dataclass
class FikotarConfig:
    vocab_size: int
    width: int
    eps: float
    logit_scale: float
    layers: list = field(default_factory=list)     # per layer: {"type", "mixer": {"left", "right", "left_scale", "right_scale"}, "mlp": {...} | None}
    torch_dtype: str = "bfloat16"
    architecture: str = "Fikotar"

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, d: dict) -> "FikotarConfig":
        layers = []
        for i, layer in enumerate(d["layers"]):
            kind, m, mlp = layer["type"], layer["mixer"], layer.get("mlp")
            if kind not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {kind!r} (known: {MIXERS})")
            a, r = m["left"], m["right"]
            mask = a.get("mask") or {}
            left = {"heads": int(a["heads"]), "kv_heads": int(a.get("kv_heads", a["heads"])), "dim": int(a["dim"]), "vdim": int(a.get("vdim", a["dim"])),
                    "conv": int(a.get("conv") or 0) or None, "scale": float(a["scale"]), "rot": _rot(a), "window": int(mask.get("size") or 0) or None,
                    "keep_first": int(mask.get("keep_first") or 0)}
            right = {"heads": int(r["heads"]), "dim": int(r["dim"]), "vdim": int(r.get("vdim", r["dim"])), "decay": [float(x) for x in r["decay"]], "rot": _rot(r)}
            if mlp is not None:
                if mlp.get("kind") != "moe":
                    raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
                shared = mlp.get("shared")
                mlp = {"kind": "moe", "expert": {"ff": int(mlp["expert"]["ff"])},
                       "router": {"experts": int(mlp["router"]["experts"]), "top": int(mlp["router"]["top"])},
                       "shared": {"ff": int(shared["ff"])} if shared else None}
            layers.append({"type": kind, "mixer": {"left": left, "right": right, "left_scale": float(m.get("left_scale", 1.0)),
                                                   "right_scale": float(m.get("right_scale", 1.0))}, "mlp": mlp})
        return cls(vocab_size=int(d["vocab"]), width=int(d["width"]), eps=float(d["norm"]["eps"]), logit_scale=float(d.get("logit_scale", 1.0)),
                   layers=layers, torch_dtype=d.get("torch_dtype", d.get("dtype", "bfloat16")))

    def to_dict(self) -> dict:
        layers = []
        for layer in self.layers:
            m, mlp = layer["mixer"], layer["mlp"]
            left = {k: v for k, v in m["left"].items() if k not in ("window", "keep_first") and v is not None}
            if m["left"]["window"]:
                left["mask"] = {"size": m["left"]["window"], "keep_first": m["left"]["keep_first"]}
            mixer = {**m, "left": left, "right": {k: v for k, v in m["right"].items() if v is not None}}
            layers.append({"type": layer["type"], "mixer": mixer, "mlp": mlp if mlp is None else {k: v for k, v in mlp.items() if v is not None}})
        return {"architecture": self.architecture, "vocab": self.vocab_size, "width": self.width, "norm": {"eps": self.eps},
                "logit_scale": self.logit_scale, "layers": layers}


def _f32(*shape):
    return nn.Parameter(torch.zeros(*shape, dtype=torch.float32))


class FikotarLayer(nn.Module):
    """The blocks of one layer and its two shared products: rows of in_proj are left q | k | v, right q | k | v | g, shared gate | up; columns
    of out_proj are left heads, right heads, shared hidden."""

    def __init__(self, cfg: FikotarConfig, i: int, turns: TurnTables):
        super().__init__()
        spec, w = cfg.layers[i], cfg.width
        m, mlp = spec["mixer"], spec["mlp"]
        a, r = m["left"], m["right"]
        dims = lambda rot: rot["dims"] if rot else 0
        self.left = ConvAttention(a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["conv"] or 1, a["scale"], cfg.eps, cache_names=((i, "k"), (i, "v")),
                                  state_name=i, rot_key=turns.add(a["rot"]), rot_dims=dims(a["rot"]), window=a["window"], keep_first=a["keep_first"],
                                  out_mul=m["left_scale"])
        self.right = Retention(r["heads"], r["dim"], r["vdim"], r["decay"], cfg.eps, state_name=i, rot_key=turns.add(r["rot"]), rot_dims=dims(r["rot"]),
                               out_mul=m["right_scale"])
        if not a["conv"]:
            nn.init.ones_(self.left.conv_w)          # no convolution: one tap of weight one
        self.moe, self.shared = None, None
        if mlp is not None:
            self.moe = GroupedSoftmaxMoE(w, mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"], float("inf"), 1.0, shift=0.0, norm_eps=0.0)
            if mlp["shared"]:
                self.shared = GatedSharedExpert(mlp["shared"]["ff"])
                # the shared expert's gate is one more row beside the router's: one float32 projection gives both
                self.moe.router = _f32(self.moe.experts + 1, w)
        blocks = [b for b in (self.left, self.right, self.shared) if b is not None]
        self.in_at, self.out_at = [0], [0]
        for b in blocks:
            self.in_at.append(self.in_at[-1] + b.proj_rows)
            self.out_at.append(self.out_at[-1] + b.out_cols)
        self.in_proj = nn.Linear(w, self.in_at[-1], bias=False)
        self.out_proj = nn.Linear(self.out_at[-1], w, bias=False)
        self.norm1, self.norm1_b = _f32(w), _f32(w)

    def forward(self, h: torch.Tensor, turns: TurnTables, table, md, decode_step: bool):
        """(mixers and shared expert, experts or None): what the stream takes up behind this layer."""
        z = plan = None
        if self.moe is not None:      # first of all: the experts' counts reach the host while the mixers run
            z = ops.skinny_proj(h, self.moe.router)
            plan = self.moe.plan(z[:, :self.moe.experts], decode_step)
        x, at, to = self.in_proj(h), self.in_at, self.out_at
        o = torch.empty((h.shape[0], to[-1]), dtype=h.dtype, device=h.device)
        self.left.attend(x, at[0], turns.at(table, self.left.rot_key), md, o[:, to[0]:to[1]])
        self.right.mix(x, at[1], turns.at(table, self.right.rot_key), md, o[:, to[1]:to[2]])
        if self.shared is not None:
            self.shared.hidden(x, at[2], z[:, self.moe.experts], o[:, to[2]:to[3]])
        y = self.out_proj(o)
        return y, self.moe(h, decode_step, plan=plan) if self.moe is not None else None


class FikotarForCausalLM(nn.Module):
    family = "seq_state"       # per-token cache rows + per-sequence state slots; ragged steps

    def __init__(self, cfg: FikotarConfig):
        super().__init__()
        if tpd.tp_size() * tpd.pp_size() != 1:
            raise NotImplementedError("Fikotar runs on one rank: its recurrent state and token cache are not sharded")
        self.config = cfg
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, cfg.width))
        self.turns = TurnTables()
        self.layers = nn.ModuleList(FikotarLayer(cfg, i, self.turns) for i in range(len(cfg.layers)))
        self.register_buffer("turn_freq", self.turns.freq(), persistent=False)
        self.final_norm, self.final_norm_b = _f32(cfg.width), _f32(cfg.width)      # times logit_scale: the logits' factor rides on the last norm
        self.head = nn.Parameter(torch.empty(cfg.vocab_size, cfg.width))
        self.metadata = None
        self.layer_streams = None      # a list: forward() appends a copy of the residual stream after every layer (diagnostics)
        self.start_layer, self.end_layer = 0, len(cfg.layers)

    # -- what the runner asks -------------------------------------------------------------------------
    def finalize(self):
        pass

    def pack_decode_weights(self):
        pass

    def set_attention_metadata(self, metadata):
        self.metadata = metadata

    def latent_ranks(self) -> dict:
        """Rows of the per-token cache: name -> elements per token (every layer's keys and values)."""
        rows = {}
        for l in self.layers:
            rows.update(l.left.cache_rows())
        return rows

    def state_shapes(self) -> dict:
        shapes = {}
        for l in self.layers:
            shapes.update(l.left.state_shapes())
            shapes.update(l.right.state_shapes())
        return shapes

    # -- forward ----------------------------------------------------------------------------------------
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """Final-normed hidden states (tokens, width), times logit_scale, in the activations' format."""
        md, eps = self.metadata, self.config.eps
        assert md is not None
        decode_step = md.layout.qo_indptr is None
        table = self.turns.step(positions, self.turn_freq)
        norms = [(l.norm1, l.norm1_b) for l in self.layers] + [(self.final_norm, self.final_norm_b)]
        x, h = ops.embed_sum(input_ids, self.embed, md.layout, w=norms[0][0], w_bias=norms[0][1], eps=eps)
        for i, layer in enumerate(self.layers):
            y, y2 = layer(h, self.turns, table, md, decode_step)
            h = ops.residual_norm(x, y, y2, w=norms[i + 1][0], w_bias=norms[i + 1][1], eps=eps)
            if self.layer_streams is not None:
                self.layer_streams.append(x.clone())
        return h

    def compute_logits(self, hidden_states: torch.Tensor) -> torch.Tensor:
        """float32 logits."""
        return ops.product_f32(hidden_states, self.head)

    # -- weights ----------------------------------------------------------------------------------------
    @torch.no_grad()
    def load_weights(self, weights: Iterable):
        """Checkpoint tensors under the design's names ('embed', 'l<i>.mix.left.q.conv', 'l<i>.mlp.e<j>.up', ...) -> the fused parameters.
        Every tensor the configuration calls for must be there, in its shape; a tensor it does not call for is left out with a warning
        (nothing of the model reads it)."""
        wanted, got, surplus = checkpoint_shapes(self.config), set(), []
        for name, w in weights:
            if name not in wanted:
                surplus.append(name)
                continue
            if tuple(w.shape) != wanted[name]:
                raise ValueError(f"{name}: checkpoint shape {tuple(w.shape)}, model wants {wanted[name]}")
            self._load_one(name, w)
            got.add(name)
        missing = [n for n in wanted if n not in got]
        if missing:
            raise KeyError(f"checkpoint lacks {len(missing)} tensors, e.g. {missing[:4]}")
        if surplus:
            import warnings
            warnings.warn(f"checkpoint holds {len(surplus)} tensors that this configuration does not use, e.g. {surplus[:4]}")
        self.pack_decode_weights()

    def _load_one(self, name: str, w: torch.Tensor):
        if name in ("embed", "head"):
            return getattr(self, name).copy_(w)
        if name in ("final.norm", "final.norm.b"):
            p = self.final_norm if name == "final.norm" else self.final_norm_b
            return p.copy_(w.float() * self.config.logit_scale)
        head, _, rest = name.partition(".")
        layer = self.layers[int(head[1:])]
        if rest in ("norm1", "norm1.b"):
            return (layer.norm1 if rest == "norm1" else layer.norm1_b).copy_(w)
        part, _, what = rest.partition(".")
        if part == "mlp":
            return self._load_mlp(layer, what, w)
        side, _, what = what.partition(".")
        block, k = (layer.left, 0) if side == "left" else (layer.right, 1)
        if what == "sink":
            return block.sinks.copy_(w)
        if what == "o":
            return layer.out_proj.weight[:, layer.out_at[k]:layer.out_at[k + 1]].copy_(w)
        q, _, conv = what.partition(".")
        at = 0                                            # rows of the block: q | k | v (| g)
        for n, rows in self._block_rows(block):
            if n == q:
                if conv:                                  # stored (channels, taps), kept (taps, channels)
                    return block.conv_w[:, at:at + rows].copy_(w.t())
                return layer.in_proj.weight[layer.in_at[k] + at:layer.in_at[k] + at + rows].copy_(w)
            at += rows
        raise KeyError(f"unexpected tensor {name!r}")

    @staticmethod
    def _block_rows(block) -> list:
        if isinstance(block, ConvAttention):
            return [("q", block.q_cols), ("k", block.k_cols), ("v", block.v_cols)]
        hd, he = block.heads * block.dim, block.heads * block.vdim
        return [("q", hd), ("k", hd), ("v", he), ("g", he)]

    @staticmethod
    def _load_mlp(layer, what: str, w: torch.Tensor):
        moe = layer.moe
        if what == "router":
            return moe.router[:moe.experts].copy_(w)
        e, _, part = what.partition(".")
        if e == "shared":
            ff, row = layer.shared.ff, layer.in_at[2]
            if part == "sg":
                return moe.router[moe.experts:].copy_(w)
            if part == "down":
                return layer.out_proj.weight[:, layer.out_at[2]:layer.out_at[3]].copy_(w)
            return layer.in_proj.weight[row + (ff if part == "up" else 0):row + (2 * ff if part == "up" else ff)].copy_(w)
        j, ff = int(e[1:]), moe.ff
        return {"gate": moe.w_gu[j, :ff], "up": moe.w_gu[j, ff:], "down": moe.w_d[j]}[part].copy_(w)

    @torch.no_grad()
    def init_random(self, seed: int = 0):
        self.load_weights(random_checkpoint(self.config, seed))


def checkpoint_shapes(cfg: FikotarConfig) -> dict:
    """name -> shape of every tensor of a checkpoint of this configuration."""
    w, shapes = cfg.width, {"embed": (cfg.vocab_size, cfg.width)}
    for i, layer in enumerate(cfg.layers):
        p, a, r, mlp = f"l{i}.", layer["mixer"]["left"], layer["mixer"]["right"], layer["mlp"]
        shapes.update({p + "norm1": (w,), p + "norm1.b": (w,)})
        left, right = p + "mix.left.", p + "mix.right."
        rows = {"q": a["heads"] * a["dim"], "k": a["kv_heads"] * a["dim"], "v": a["kv_heads"] * a["vdim"]}
        shapes.update({left + n: (c, w) for n, c in rows.items()})
        if a["conv"]:
            shapes.update({f"{left}{n}.conv": (c, a["conv"]) for n, c in rows.items()})
        shapes.update({left + "sink": (a["heads"],), left + "o": (w, a["heads"] * a["vdim"])})
        hd, he = r["heads"] * r["dim"], r["heads"] * r["vdim"]
        shapes.update({right + "q": (hd, w), right + "k": (hd, w), right + "v": (he, w), right + "g": (he, w), right + "o": (w, he)})
        if mlp is not None:
            glus = [(f"e{j}.", mlp["expert"]["ff"]) for j in range(mlp["router"]["experts"])]
            shapes[p + "mlp.router"] = (mlp["router"]["experts"], w)
            if mlp["shared"]:
                glus.append(("shared.", mlp["shared"]["ff"]))
                shapes[p + "mlp.shared.sg"] = (1, w)
            for s, ff in glus:
                shapes.update({f"{p}mlp.{s}gate": (ff, w), f"{p}mlp.{s}up": (ff, w), f"{p}mlp.{s}down": (w, ff)})
    shapes.update({"final.norm": (w,), "final.norm.b": (w,), "head": (cfg.vocab_size, w)})
    return shapes


def checkpoint_names(cfg: FikotarConfig) -> list:
    return list(checkpoint_shapes(cfg))


def random_checkpoint(cfg: FikotarConfig, seed: int = 0):
    """(name, tensor) pairs of a seeded random checkpoint, rounded to bfloat16 values (as a stored checkpoint is), one tensor at a time.
    Matrices are scaled by 1/sqrt(fan-in); norm weights are near one; a convolution's last tap (the token itself) is near one and the
    others are smaller; sinks and norm biases are small."""
    gen = torch.Generator(device="cpu").manual_seed(seed)
    for name, shape in checkpoint_shapes(cfg).items():
        rnd = torch.randn(shape, generator=gen)
        if name.endswith(("norm1", "final.norm")):
            w = 1.0 + 0.1 * rnd
        elif name.endswith(".b"):
            w = 0.1 * rnd
        elif name.endswith(".conv"):
            w = 0.4 * rnd
            w[:, -1] += 1.0
        elif name.endswith(".sink") or name == "embed":
            w = rnd
        else:
            w = rnd * shape[-1] ** -0.5
        yield name, w.to(torch.bfloat16).float()
