"""Zenedra: a pre-normed decoder stack over a float32 residual stream, some of whose layers run several times over a sequence with the
same weights:
    x0 = embed[token] + pair[hash(previous token, token)] + position[p]            (the pair table has one more row for a first token)
    x <- x + mixer(norm1(x));   x <- x + ff(norm2(x))                              (norm(x) = x / rms(x) * (1 + w))
    logits = head (final norm(x)).
Layers loop.start .. loop.stop - 1 run loop.times times in a row, then the rest follow; ahead of pass t the stream becomes
W_in [x; x0] + step[t].  Every pass has cache rows and states of its own.

A layer's mixer is one of
  attention  grouped heads whose values are their keys as projected, per-head query/key norm, a linear distance penalty, chunks of
             positions (a token sees the earlier tokens of its own chunk);
  gla        gated linear attention: a matrix memory per head with a decay per key channel and token;
  mlstm      a matrix memory per head with an exponential input gate, kept finite by a running maximum;
and its feed-forward is dense (gelu-gated), a mixture of experts behind a sigmoid router with groups, beside an expert that every token
passes, or absent.

config.json gives every size, the order of the layers and the constants; the mechanisms live in layers/ (cap_attention.py,
recurrent.py, moe.py) with their constants as arguments.  Between the matrix products (library GEMMs; all input projections of a mixer
are ONE product) every step is a HIP kernel of this package, one launch per sublayer boundary (ops.residual_norm).  The stream, norms,
attention scores, positions, routers, gates and decays of the recurrences and their states are float32 in every activation format, and
the product that joins x and x0 ahead of a pass sees the stream as a hi + lo pair of 16-bit numbers and returns float32.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Iterable

import torch
import torch.nn.functional as F
from torch import nn

from . import distributed as tpd
from . import ops
from .layers.cap_attention import TiedAttention, geometric_slopes
from .layers.moe import DenseGLU, GeluGLU, GroupedSigmoidMoE
from .layers.recurrent import MLSTM, GatedLinearAttention

MIXERS = ("attention", "gla", "mlstm")
GLU_SLOPE = 1.702         # expert: y = g sigmoid(1.702 g) (u + 1)
DECAY_RANK = 16           # inner size of the decay's two projections in a model that is built without a checkpoint


@dataclass
class ZenedraConfig:
    vocab_size: int
    width: int
    eps: float
    max_positions: int
    bigram: dict | None                            # {"buckets", "mul_prev", "mul_cur"}
    loop: dict | None                              # {"start", "stop", "times"}
    layers: list = field(default_factory=list)     # per layer: {"type", "mixer": {...}, "mlp": {...} | None}
    torch_dtype: str = "bfloat16"
    architecture: str = "Zenedra"

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, d: dict) -> "ZenedraConfig":
        layers = []
        for i, layer in enumerate(d["layers"]):
            kind, m, mlp = layer["type"], layer["mixer"], layer.get("mlp")
            heads, dim = int(m["heads"]), int(m["dim"])
            if kind == "attention":
                if int(m.get("vdim", dim)) != dim:
                    raise ValueError(f"layer {i}: the values are the keys, so their sizes are equal")
                m = {"heads": heads, "kv_heads": int(m.get("kv_heads", heads)), "dim": dim, "vdim": dim, "scale": float(m["scale"]),
                     "chunk": int((m.get("mask") or {}).get("size") or 0) or None}
            elif kind == "gla":
                # the inner size of the decay's two projections is a tensor's shape in a checkpoint; "decay_rank" only sizes a model
                # that is built without one
                m = {"heads": heads, "dim": dim, "vdim": int(m.get("vdim", dim)), "tau": float(m["tau"]), "decay_rank": int(m.get("decay_rank", DECAY_RANK))}
            elif kind == "mlstm":
                m = {"heads": heads, "dim": dim, "vdim": int(m.get("vdim", dim)), "gate_cap": float(m["gate_cap"])}
            else:
                raise ValueError(f"layer {i}: unknown mixer {kind!r} (known: {MIXERS})")
            if mlp is not None:
                if mlp.get("kind") == "dense":
                    mlp = {"kind": "dense", "ff": int(mlp["ff"])}
                elif mlp.get("kind") == "moe":
                    r, groups, shared = mlp["router"], mlp["router"].get("groups"), mlp.get("shared")
                    mlp = {"kind": "moe", "expert": {"ff": int(mlp["expert"]["ff"]), "limit": float(mlp["expert"]["limit"])},
                           "router": {"experts": int(r["experts"]), "top": int(r["top"]), "scale": float(r.get("scale", 1.0)),
                                      "groups": {"count": int(groups["count"]), "keep": int(groups["keep"])} if groups else None},
                           "shared": {"ff": int(shared["ff"]), "limit": float(shared["limit"])} if shared else None}
                else:
                    raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
            layers.append({"type": kind, "mixer": m, "mlp": mlp})
        loop = d.get("loop")
        if loop is not None:
            loop = {k: int(loop[k]) for k in ("start", "stop", "times")}
            if not (0 <= loop["start"] < loop["stop"] <= len(layers) and loop["times"] >= 1):
                raise ValueError(f"loop {loop} does not name a run of layers")
        pair = (d.get("embedding") or {}).get("bigram")
        return cls(vocab_size=int(d["vocab"]), width=int(d["width"]), eps=float(d["norm"]["eps"]), max_positions=int(d["max_positions"]),
                   bigram={k: int(pair[k]) for k in ("buckets", "mul_prev", "mul_cur")} if pair else None, loop=loop, layers=layers,
                   torch_dtype=d.get("torch_dtype", d.get("dtype", "bfloat16")))

    def to_dict(self) -> dict:
        layers = []
        for layer in self.layers:
            m, mlp = dict(layer["mixer"]), layer["mlp"]
            if layer["type"] == "attention":
                chunk = m.pop("chunk")
                if chunk:
                    m["mask"] = {"size": chunk}
            if mlp is not None and mlp["kind"] == "moe":
                mlp = {**{k: v for k, v in mlp.items() if v is not None}, "router": {k: v for k, v in mlp["router"].items() if v is not None}}
            layers.append({"type": layer["type"], "mixer": m, "mlp": mlp})
        out = {"architecture": self.architecture, "vocab": self.vocab_size, "width": self.width, "norm": {"eps": self.eps},
               "max_positions": self.max_positions, "layers": layers}
        if self.bigram:
            out["embedding"] = {"bigram": dict(self.bigram)}
        if self.loop:
            out["loop"] = dict(self.loop)
        return out

    def runs(self) -> list:
        """[(layer, name, pass)] in the order they run: `name` is what the run's cache rows and states go by, `pass` the number of the pass
        that begins with this run (None elsewhere)."""
        n = len(self.layers)
        a, b, times = (self.loop["start"], self.loop["stop"], self.loop["times"]) if self.loop else (n, n, 0)
        out = [(i, (i, 0), None) for i in range(a)]
        out += [(i, (i, t), t if i == a else None) for t in range(times) for i in range(a, b)]
        return out + [(i, (i, 0), None) for i in range(b, n)]


def _f32(*shape):
    return nn.Parameter(torch.zeros(*shape, dtype=torch.float32))


class ZenedraLayer(nn.Module):
    def __init__(self, cfg: ZenedraConfig, i: int):
        super().__init__()
        spec = cfg.layers[i]
        w, m = cfg.width, spec["mixer"]
        self.kind = spec["type"]
        if self.kind == "attention":
            self.mixer = TiedAttention(w, m["heads"], m["kv_heads"], m["dim"], m["scale"], cfg.eps, cache_name=(i, 0),
                                       slopes=geometric_slopes(m["heads"]), chunk=m["chunk"], bias=True, o_bias=True)
        elif self.kind == "gla":
            self.mixer = GatedLinearAttention(w, m["heads"], m["dim"], m["vdim"], m["tau"], m["decay_rank"], cfg.eps, state_name=(i, 0))
        else:
            self.mixer = MLSTM(w, m["heads"], m["dim"], m["vdim"], m["gate_cap"], cfg.eps, state_name=(i, 0))
        self.norm1 = _f32(w)                       # 1 + the stored weight, as norm2 and the final norm
        mlp = spec["mlp"]
        self.mlp_kind = mlp["kind"] if mlp is not None else None
        self.mlp = None
        if mlp is not None:
            if mlp["kind"] == "dense":
                self.mlp = GeluGLU(w, mlp["ff"])
            else:
                r, g, s = mlp["router"], mlp["router"]["groups"], mlp["shared"]
                self.mlp = GroupedSigmoidMoE(w, r["experts"], r["top"], mlp["expert"]["ff"], mlp["expert"]["limit"], GLU_SLOPE, 1.0,
                                             groups=g["count"] if g else None, keep=g["keep"] if g else None, scale=r["scale"],
                                             shared=DenseGLU(w, s["ff"], s["limit"], GLU_SLOPE) if s else None)
            self.norm2 = _f32(w)


class ZenedraForCausalLM(nn.Module):
    family = "seq_state"       # per-token cache rows + per-sequence state slots; ragged steps

    def __init__(self, cfg: ZenedraConfig):
        super().__init__()
        if tpd.tp_size() * tpd.pp_size() != 1:
            raise NotImplementedError("Zenedra runs on one rank: its recurrent state and token cache are not sharded")
        self.config = cfg
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, cfg.width))
        self.pair = nn.Parameter(torch.empty(cfg.bigram["buckets"] + 1, cfg.width)) if cfg.bigram else None
        self.pos = nn.Parameter(torch.empty(cfg.max_positions, cfg.width))
        self.layers = nn.ModuleList(ZenedraLayer(cfg, i) for i in range(len(cfg.layers)))
        self.final_norm = _f32(cfg.width)
        self.head = nn.Parameter(torch.empty(cfg.vocab_size, cfg.width))
        if cfg.loop:
            self.loop_in = nn.Parameter(torch.empty(2, cfg.width, cfg.width))      # what the stream, and what the embedding output is multiplied with
            self.loop_step = _f32(cfg.loop["times"], cfg.width)
            self._join_w = None
        self.runs = cfg.runs()
        self.metadata = None
        self.layer_streams = None      # a list: forward() appends a copy of the residual stream after every layer run (diagnostics)
        self.start_layer, self.end_layer = 0, len(cfg.layers)

    # -- what the runner asks -------------------------------------------------------------------------
    def finalize(self):
        pass

    def pack_decode_weights(self):
        """Called when the weights are in place: the two matrices of the join, each side by side with itself for the [hi | lo] rows."""
        if self.config.loop:
            self._join_w = [w if w.dtype == torch.float32 else torch.cat([w, w], 1) for w in self.loop_in.detach()]

    def set_attention_metadata(self, metadata):
        self.metadata = metadata

    def latent_ranks(self) -> dict:
        """Rows of the per-token cache, for every run of an attention layer: the keys, and a float32 number per key/value head."""
        rows = {}
        for i, name, _ in self.runs:
            if self.layers[i].kind == "attention":
                rows.update(self.layers[i].mixer.cache_rows(at=name))
        return rows

    def state_shapes(self) -> dict:
        shapes = {"prev_id": (1,)} if self.pair is not None else {}
        for i, name, _ in self.runs:
            if self.layers[i].kind != "attention":
                shapes.update(self.layers[i].mixer.state_shapes(at=name))
        return shapes

    # -- forward ----------------------------------------------------------------------------------------
    def _join(self, x: torch.Tensor, pair_rows, which: int) -> torch.Tensor:
        """One half of W_in [x; x0] in float32: `pair_rows` are the [hi | lo] rows of x (16-bit formats)."""
        w = self._join_w[which]
        return F.linear(x, w) if pair_rows is None else ops.product_f32(pair_rows, w)

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """Final-normed hidden states (tokens, width) in the activations' format."""
        md, cfg = self.metadata, self.config
        assert md is not None
        eps, dtype, runs, layers = cfg.eps, self.embed.dtype, self.runs, self.layers
        decode_step = md.layout.qo_indptr is None
        pairs = dtype != torch.float32
        b = cfg.bigram or {"mul_prev": 0, "mul_cur": 0}
        norms = [layers[i].norm1 for i, _, _ in runs] + [self.final_norm]
        starts = [p for _, _, p in runs] + [None]
        x, h = ops.embed_sum(input_ids, self.embed, md.layout, pair=self.pair, mul_prev=b["mul_prev"], mul_cur=b["mul_cur"],
                             prev_id=md.cache.state("prev_id") if self.pair is not None else None, pos_table=self.pos, positions=positions,
                             w=None if cfg.loop else norms[0], eps=eps, split=bool(cfg.loop) and pairs)
        from_x0 = None
        if cfg.loop:
            from_x0 = self._join(x, h if pairs else None, 1)       # the same for every pass
            if starts[0] is None:
                h = ops.residual_norm(x, w=norms[0], eps=eps, dtype=dtype)
            else:
                x, h = self._begin_pass(x, h if pairs else None, from_x0, starts[0], norms[0])
        for n, (i, name, _) in enumerate(runs):
            layer = layers[i]
            y, y2 = layer.mixer(h, md, at=name), None
            if layer.mlp is not None:
                h = ops.residual_norm(x, y, w=layer.norm2, eps=eps)
                y = layer.mlp(h) if layer.mlp_kind == "dense" else layer.mlp(h, decode_step)
                if layer.mlp_kind == "moe":
                    y, y2 = y
            if starts[n + 1] is None:
                h = ops.residual_norm(x, y, y2, w=norms[n + 1], eps=eps)
            else:
                h = ops.residual_norm(x, y, y2, split=pairs, dtype=dtype)
            if self.layer_streams is not None:
                self.layer_streams.append(x.clone())
            if starts[n + 1] is not None:
                x, h = self._begin_pass(x, h, from_x0, starts[n + 1], norms[n + 1])
        return h

    def _begin_pass(self, x, pair_rows, from_x0, t: int, norm):
        """(stream, its norm) at the head of pass t: x <- W_x x + W_0 x0 + step[t]."""
        x = self._join(x, pair_rows, 0)
        return x, ops.residual_norm(x, add=from_x0, bias=self.loop_step[t], w=norm, eps=self.config.eps, dtype=self.embed.dtype)

    def compute_logits(self, hidden_states: torch.Tensor) -> torch.Tensor:
        """float32 logits."""
        return ops.product_f32(hidden_states, self.head)

    # -- weights ----------------------------------------------------------------------------------------
    @torch.no_grad()
    def load_weights(self, weights: Iterable):
        """Checkpoint tensors under the design's names ('embed', 'l<i>.mix.q', 'l<i>.mlp.e<j>.up', 'loop.in', ...) -> the fused parameters.
        Every tensor the configuration calls for must be there, in its shape; a tensor it does not call for is left out with a warning
        (nothing of the model reads it)."""
        wanted, got, surplus = checkpoint_shapes(self.config), set(), []
        for name, w in weights:
            if name not in wanted:
                surplus.append(name)
                continue
            self._load_one(name, w)
            got.add(name)
        missing = [n for n in wanted if n not in got]
        if missing:
            raise KeyError(f"checkpoint lacks {len(missing)} tensors, e.g. {missing[:4]}")
        for i, l in enumerate(self.layers):
            if l.kind == "gla" and l.mixer.a1.shape[0] != l.mixer.a2.shape[1]:
                raise ValueError(f"layer {i}: the decay's two projections disagree on their inner size")
        if surplus:
            import warnings
            warnings.warn(f"checkpoint holds {len(surplus)} tensors that this configuration does not use, e.g. {surplus[:4]}")
        self.pack_decode_weights()

    def _load_one(self, name: str, w: torch.Tensor):
        def put(p, rows=None):
            dst = p if rows is None else p[rows[0]:rows[1]]
            if dst.shape != w.shape:
                raise ValueError(f"{name}: checkpoint shape {tuple(w.shape)}, model wants {tuple(dst.shape)}")
            dst.copy_(w)

        def put_around_one(p):
            put(p)
            p.add_(1.0)

        top = {"embed": self.embed, "bigram": self.pair, "pos": self.pos, "head": self.head}
        if top.get(name) is not None:
            return put(top[name])
        if name == "final.norm":
            return put_around_one(self.final_norm)
        if self.config.loop and name == "loop.in":
            width = self.config.width
            if tuple(w.shape) != (width, 2 * width):
                raise ValueError(f"{name}: checkpoint shape {tuple(w.shape)}, model wants {(width, 2 * width)}")
            return self.loop_in.copy_(w.view(width, 2, width).transpose(0, 1))
        if self.config.loop and name == "loop.step":
            return put(self.loop_step)
        head, _, rest = name.partition(".")
        if not (head[:1] == "l" and head[1:].isdigit() and int(head[1:]) < len(self.layers)):
            raise KeyError(f"unexpected tensor {name!r}")
        layer = self.layers[int(head[1:])]
        if rest in ("norm1", "norm2") and hasattr(layer, rest):
            return put_around_one(getattr(layer, rest))
        if rest.startswith("mlp.") and layer.mlp is not None:
            what, f = rest[4:], layer.mlp
            glu = None
            if layer.mlp_kind == "dense":
                glu = f
            else:
                if what == "router":
                    return put(f.router)
                if what == "correction":
                    return put(f.correction)
                e, _, part = what.partition(".")
                if e[:1] == "e" and e[1:].isdigit() and int(e[1:]) < f.experts:
                    j, ff = int(e[1:]), f.ff
                    where = {"gate": (f.w_gu[j], (0, ff)), "up": (f.w_gu[j], (ff, 2 * ff)), "down": (f.w_d[j], None)}
                    if part in where:
                        return put(*where[part])
                if e == "shared":
                    glu, what = f.shared, part
            if glu is not None:
                where = {"gate": (glu.gu_proj.weight, (0, glu.ff)), "up": (glu.gu_proj.weight, (glu.ff, 2 * glu.ff)), "down": (glu.down.weight, None)}
                if what in where:
                    return put(*where[what])
        if rest.startswith("mix."):
            what, m = rest[4:], layer.mixer
            if layer.kind == "gla" and what in ("a1", "a2"):
                # the decay's inner size comes with the checkpoint: the two parameters take the stored shapes
                own = getattr(m, what)
                fixed = 1 if what == "a1" else 0
                if w.dim() != 2 or w.shape[fixed] != own.shape[fixed]:
                    raise ValueError(f"{name}: checkpoint shape {tuple(w.shape)} does not fit the model")
                return setattr(m, what, nn.Parameter(w.to(device=m.a2_b.device, dtype=torch.float32).contiguous(), requires_grad=False))
            where = self._mixer_targets(layer).get(what)
            if where is not None:
                return put(*where)
        raise KeyError(f"unexpected tensor {name!r}")

    @staticmethod
    def _mixer_targets(layer) -> dict:
        """Checkpoint name below '<layer>.mix.' -> (parameter, row range or None)."""
        m = layer.mixer
        if layer.kind == "attention":
            p, q, k = m.in_proj, m.q_cols, m.k_cols
            return {"q": (p.weight, (0, q)), "q.b": (p.bias, (0, q)), "k": (p.weight, (q, q + k)), "k.b": (p.bias, (q, q + k)),
                    "q.norm": (m.q_norm, None), "k.norm": (m.k_norm, None), "o": (m.o_proj.weight, None), "o.b": (m.o_proj.bias, None)}
        hd, he, h, p = m.heads * m.dim, m.heads * m.vdim, m.heads, m.qkvg_proj.weight
        out = {"q": (p, (0, hd)), "k": (p, (hd, 2 * hd)), "v": (p, (2 * hd, 2 * hd + he)), "g": (p, (2 * hd + he, 2 * hd + 2 * he)),
               "o": (m.o_proj.weight, None), "norm": (m.norm, None)}
        if layer.kind == "gla":
            out["a2.b"] = (m.a2_b, None)
        else:
            out.update({"i": (m.gate_w, (0, h)), "f": (m.gate_w, (h, 2 * h)), "i.b": (m.gate_b, (0, h)), "f.b": (m.gate_b, (h, 2 * h))})
        return out

    @torch.no_grad()
    def init_random(self, seed: int = 0):
        self.load_weights(random_checkpoint(self.config, seed))


def checkpoint_shapes(cfg: ZenedraConfig) -> dict:
    """name -> shape of every tensor of a checkpoint of this configuration (the inner size of a gla layer's decay is the checkpoint's own)."""
    w, shapes = cfg.width, {"embed": (cfg.vocab_size, cfg.width)}
    if cfg.bigram:
        shapes["bigram"] = (cfg.bigram["buckets"] + 1, w)
    shapes["pos"] = (cfg.max_positions, w)
    if cfg.loop:
        shapes.update({"loop.in": (w, 2 * w), "loop.step": (cfg.loop["times"], w)})
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.", layer["mixer"]
        h, hd = m["heads"], m["heads"] * m["dim"]
        shapes[p + "norm1"] = (w,)
        if layer["type"] == "attention":
            kd = m["kv_heads"] * m["dim"]
            shapes.update({p + "mix.q": (hd, w), p + "mix.q.b": (hd,), p + "mix.k": (kd, w), p + "mix.k.b": (kd,), p + "mix.q.norm": (m["dim"],),
                           p + "mix.k.norm": (m["dim"],), p + "mix.o": (w, hd), p + "mix.o.b": (w,)})
        else:
            he = h * m["vdim"]
            shapes.update({p + "mix.q": (hd, w), p + "mix.k": (hd, w), p + "mix.v": (he, w), p + "mix.g": (he, w), p + "mix.o": (w, he)})
            if layer["type"] == "gla":
                r = m["decay_rank"]
                shapes.update({p + "mix.norm": (m["vdim"],), p + "mix.a1": (r, w), p + "mix.a2": (hd, r), p + "mix.a2.b": (hd,)})
            else:
                shapes.update({p + "mix.norm": (he,), p + "mix.i": (h, w), p + "mix.i.b": (h,), p + "mix.f": (h, w), p + "mix.f.b": (h,)})
        mlp = layer["mlp"]
        if mlp is not None:
            shapes[p + "norm2"] = (w,)
            glus = [("", mlp["ff"])] if mlp["kind"] == "dense" else [(f"e{j}.", mlp["expert"]["ff"]) for j in range(mlp["router"]["experts"])]
            if mlp["kind"] == "moe":
                shapes.update({p + "mlp.router": (mlp["router"]["experts"], w), p + "mlp.correction": (mlp["router"]["experts"],)})
                if mlp["shared"]:
                    glus.append(("shared.", mlp["shared"]["ff"]))
            for s, ff in glus:
                shapes.update({f"{p}mlp.{s}gate": (ff, w), f"{p}mlp.{s}up": (ff, w), f"{p}mlp.{s}down": (w, ff)})
    shapes["final.norm"] = (w,)
    shapes["head"] = (cfg.vocab_size, w)
    return shapes


def checkpoint_names(cfg: ZenedraConfig) -> list:
    return list(checkpoint_shapes(cfg))


def random_checkpoint(cfg: ZenedraConfig, seed: int = 0):
    """(name, tensor) pairs of a seeded random checkpoint, rounded to bfloat16 values (as a stored checkpoint is), one tensor at a
    time.  Matrices are scaled by 1/sqrt(fan-in); norm weights are near one (stored around zero where the design adds the one); biases
    are small, gates and decays of the recurrences such that memories neither vanish nor saturate over a few hundred tokens."""
    gen = torch.Generator(device="cpu").manual_seed(seed)
    for name, shape in checkpoint_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        rnd = torch.randn(shape, generator=gen)
        if leaf in ("norm1", "norm2") or name == "final.norm":
            w = 0.1 * rnd
        elif leaf == "norm":
            w = 1.0 + 0.1 * rnd
        elif name.endswith(".f.b"):
            w = 2.0 + 0.5 * rnd
        elif name.endswith(".a2.b"):
            w = 1.0 + 0.5 * rnd
        elif name.endswith(".i.b"):
            w = 0.5 * rnd
        elif leaf in ("b", "correction", "step"):
            w = 0.2 * rnd
        elif name == "embed":
            w = rnd
        elif name in ("bigram", "pos"):
            w = 0.5 * rnd
        else:
            w = rnd * shape[-1] ** -0.5
        yield name, w.to(torch.bfloat16).float()
