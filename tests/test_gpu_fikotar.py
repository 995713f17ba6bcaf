"""Fikotar through the engine, and its kernels alone, against the plain restatement in oracle/fikotar_oracle.py.

Every test makes its own small configuration and weights.  The engine is built on a directory that holds config.json (and,
where the weights are made by the test, model.safetensors), as a user's would be; steps are given with Engine.run_given (the
replay entry point) or chosen by the scheduler (Engine.step / LLM.generate).  Comparisons are in float32 unless a test says
otherwise: there a structural fault (a key outside the window, a lost kept token, a missing sink, a stale convolution input) stands far
above rounding.
"""
import asyncio
import json
import os

import numpy as np
import pytest
import torch

from oracle import fikotar_oracle as fo
from seq_drivers import F32_TOL, close, cuts_of, greedy, make_engine, model_dir, replay, step_layout, tokens

pytestmark = pytest.mark.gpu

BANDS = {"factor": 5.0, "low": 1.0, "high": 3.0, "original": 40}
LEFT = {"heads": 6, "kv_heads": 2, "dim": 20, "vdim": 14, "conv": 4, "scale": 1.7, "mask": {"size": 37, "keep_first": 3},
        "rot": {"dims": 12, "base": 5000.0, "scaling": BANDS}}
RIGHT = {"heads": 3, "dim": 10, "vdim": 18, "decay": [0.9, 0.75, 0.998], "rot": {"dims": 8, "base": 700.0}}
MOE = {"kind": "moe", "expert": {"ff": 16}, "router": {"experts": 6, "top": 3}, "shared": {"ff": 28}}
MOE1 = {"kind": "moe", "expert": {"ff": 10}, "router": {"experts": 4, "top": 1}}


def layer(left=None, right=None, mlp=MOE, left_scale=0.8, right_scale=1.3):
    """One layer's entry; `left` / `right` change the sizes above (a value of None takes the key out)."""
    def merged(base, change):
        return {k: v for k, v in {**base, **(change or {})}.items() if v is not None}
    return json.loads(json.dumps({"type": "parallel", "mlp": mlp, "mixer": {"left": merged(LEFT, left), "right": merged(RIGHT, right),
                                                                             "left_scale": left_scale, "right_scale": right_scale}}))


STACK = [layer(), layer(left={"heads": 4, "kv_heads": 4, "mask": {"size": 64, "keep_first": 1}, "conv": 2}, mlp=None),
         layer(left={"mask": None, "rot": {"dims": 20, "base": 90.0}}, right={"heads": 2, "decay": [1.0, 0.5], "rot": None}, mlp=MOE1)]


def make_cfg(layers, width=40, vocab=61, eps=1e-5, logit_scale=0.6):
    return {"architecture": "Fikotar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "layers": json.loads(json.dumps(layers))}


def weights_of(cfg, seed=0):
    """The weights an engine built on a directory without a checkpoint draws for `seed`."""
    from nano_vllm_x_amd.fikotar import FikotarConfig, random_checkpoint
    return dict(random_checkpoint(FikotarConfig.from_dict(cfg), seed))


def near(got, want, rel, what=""):
    """Every value within `rel` of its own size (and of a fiftieth of the values' mean size: results near zero)."""
    got, want = got.double(), want.double()
    err = ((got - want).abs() / (want.abs() + 0.02 * want.abs().mean() + 1e-12)).max().item()
    assert err < rel, f"{what}: a value is off by {err:.3e} of its size (tolerance {rel})"


def within_rounding(got, want, what=""):
    err = (got.double() - want).abs().amax(dim=1) / want.std()
    assert err.median() < 0.08 and err.max() < 0.5, (what, err.median().item(), err.max().item())


def forward(cfg, w, toks):
    return fo.forward(cfg, w, toks)


# ---- kernels alone -------------------------------------------------------------------------------------------------------
def _walk(full, cuts, slot, order, run):
    """Sequences `full` (id -> rows) cut into steps (`cuts`: id -> sizes), `order` naming the live ids of every step; run(x, lens,
    pos0, slots, decode) -> rows.  Returns id -> all rows."""
    cuts = {i: list(c) for i, c in cuts.items()}
    at = {i: 0 for i in full}
    got = {i: [] for i in full}
    for live in order:
        live = [i for i in live if at[i] < len(full[i]) and cuts[i]]
        if not live:
            continue
        lens = [cuts[i].pop(0) for i in live]
        x = torch.cat([full[i][at[i]:at[i] + n] for i, n in zip(live, lens)])
        decode = all(n == 1 for n in lens) and all(at[i] > 0 for i in live)
        out = run(x, lens, [at[i] for i in live], [slot[i] for i in live], decode)
        a = 0
        for i, n in zip(live, lens):
            got[i].append(out[a:a + n])
            a += n
            at[i] += n
    assert all(at[i] == len(full[i]) for i in full)
    return {i: torch.cat(r) for i, r in got.items()}


ORDER = [[0, 1]] * 6 + [[0]] * 12 + [[1]] * 6 + [[2, 1]] * 6 + [[2]] * 6
SLOT = {0: 2, 1: 0, 2: 2}          # the third sequence takes over the first one's slot


def positions_of(pos0, lens):
    return torch.cat([torch.arange(a, a + n) for a, n in zip(pos0, lens)])


def turns_of(ops, rot, pos, ahead=0):
    """(ops.Turn, table) of a rotation; `ahead` columns of another rotation stand in front of it in the table."""
    f = fo.frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    freq = torch.cat([torch.linspace(0.1, 2.0, ahead, dtype=torch.float64), f]) if ahead else f
    return ops.Turn(ops.turn_table(pos.cuda(), freq.cuda()), ahead, rot["dims"])


def test_rotation_table_of_a_step():
    """Far positions keep their angles (formed and reduced in double precision); two rotations share a row."""
    from nano_vllm_x_amd import ops
    from nano_vllm_x_amd.layers.rotary_embedding import TurnTables
    tabs = TurnTables()
    a = tabs.add({"dims": 12, "base": 5000.0, "scaling": BANDS})
    b = tabs.add({"dims": 8, "base": 700.0})
    assert tabs.add({"dims": 12, "base": 5000.0, "scaling": dict(BANDS)}) == a and tabs.add(None) is None and tabs.add({"dims": 0, "base": 3.0}) is None
    pos = torch.tensor([0, 1, 77, 4096, 1000003])
    table = tabs.step(pos.cuda(), tabs.freq().cuda())
    assert table.shape == (5, 20)
    for key, f in ((a, fo.frequencies(12, 5000.0, BANDS)), (b, fo.frequencies(8, 700.0))):
        t = tabs.at(table, key)
        n = table.shape[1] // 2
        ang = pos.double()[:, None] * f
        got = table.cpu().double()
        assert (got[:, t.first:t.first + t.dims // 2] - torch.cos(ang)).abs().max() < 1e-6
        assert (got[:, n + t.first:n + t.first + t.dims // 2] - torch.sin(ang)).abs().max() < 1e-6


@pytest.mark.parametrize("fmt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [1, 33, 64, 300, 4100])
def test_layer_norm_at_the_layer_boundary_and_behind_the_embedding(fmt, width):
    """A mean far from zero: the variance is that of the deviations."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(width)
    t, eps = 5, 1e-3 if width > 1 else 1.0
    rnd = lambda *s: torch.randn(*s, generator=g)
    x, y, y2, w, b = rnd(t, width) + 30.0, rnd(t, width).to(fmt), rnd(t, width).to(fmt), rnd(width), rnd(width)
    tol = 1e-3 if fmt == torch.float32 else 8e-3
    for use in ((), ("y",), ("y", "y2")):
        terms = {k: v.cuda() for k, v in (("y", y), ("y2", y2)) if k in use}
        want = x.double() + sum(v.double() for k, v in (("y", y), ("y2", y2)) if k in use)
        xd = x.cuda()
        h = ops.residual_norm(xd, w=w.cuda(), w_bias=b.cuda(), eps=eps, dtype=fmt, **terms)
        assert h.dtype == fmt
        close(xd.cpu(), want, 1e-5 if width > 1 else 1e-1, f"stream {use}")
        near(h.float().cpu(), fo.layer_norm(want, w.double(), b.double(), eps), tol, f"norm {use}")
    table = (rnd(9, width) + 4.0).to(fmt)
    ids = torch.tensor([3, 3, 8, 0])
    s, h = ops.embed_sum(ids.cuda(), table.cuda(), w=w.cuda(), w_bias=b.cuda(), eps=eps)
    assert torch.equal(s.cpu(), table[ids].float())
    near(h.float().cpu(), fo.layer_norm(table[ids].double(), w.double(), b.double(), eps), tol, "norm of the embedding")


@pytest.mark.parametrize("fmt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,kvh,dim,vdim,taps,rot", [(6, 2, 20, 14, 4, 12), (4, 2, 64, 48, 3, 32), (2, 2, 128, 128, 4, 128), (3, 1, 8, 16, 1, 0), (2, 1, 200, 40, 2, 16),
                                                         (1, 1, 264, 512, 3, 48), (5, 5, 7, 3, 2, 2), (2, 1, 64, 64, 7, 32), (4, 1, 40, 24, 3, 24)])
def test_queries_keys_and_values_through_convolution_rotation_and_norm(fmt, heads, kvh, dim, vdim, taps, rot):
    """Portions of one token and of many, portions shorter than the convolution, a slot that changes hands (its old inputs must not
    count), single tokens of several sequences in one step, a padding row; sizes with 16-byte rows and without, one tap to seven."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(dim + taps)
    eps = 1e-2
    nq, nk, nv = heads * dim, kvh * dim, kvh * vdim
    ch, gap = nq + nk + nv, 8 if dim % 8 == 0 else 3
    full = {0: torch.randn(90, gap + ch, generator=g).to(fmt), 1: torch.randn(23, gap + ch, generator=g).to(fmt), 2: torch.randn(12, gap + ch, generator=g).to(fmt)}
    w = torch.randn(taps, ch, generator=g)
    spec = {"dims": rot, "base": 300.0}
    state = torch.full((3, taps - 1, ch), 7.0).cuda() if taps > 1 else None
    kc, vc = torch.full((130, nk), 9.0).to(fmt).cuda(), torch.full((130, nv), 9.0).to(fmt).cuda()

    def want_of(x):
        pos = torch.arange(len(x))
        u = fo.causal_conv(x[:, gap:].double(), w.double().t())
        q, k, v = u[:, :nq].view(-1, heads, dim), u[:, nq:nq + nk].view(-1, kvh, dim), u[:, nq + nk:]
        return torch.cat([fo.unit_rms(fo.turned(q, pos, spec), eps).reshape(-1, nq), fo.unit_rms(fo.turned(k, pos, spec), eps).reshape(-1, nk), v], 1)

    def run(x, lens, pos0, slots, decode):
        pos = positions_of(pos0, lens)
        lay = step_layout(ops, lens, pos0, slots, decode)
        out_slots = torch.randperm(130, generator=torch.Generator().manual_seed(len(x)))[:len(x)].to(torch.int64)
        turn = turns_of(ops, spec, pos, ahead=8 if rot % 16 == 0 else 5) if rot else None
        q = ops.conv_attn_prep(x.cuda()[:, gap:], w.cuda(), state, lay, turn, eps, out_slots.cuda(), kc, vc, heads, kvh, dim, vdim)
        assert q.dtype == fmt
        return torch.cat([q.float().cpu(), kc.float().cpu()[out_slots], vc.float().cpu()[out_slots]], 1)
    cuts = {0: cuts_of(90, [1, 2, 9, 1, 1, 40, 1, 1, 17, 90]), 1: cuts_of(23, [5, 1, 1, 2, 1, 1, 23]), 2: cuts_of(12, [2, 1, 1, 5, 1, 2])}
    got = _walk(full, cuts, SLOT, ORDER, run)
    for i in full:
        near(got[i], want_of(full[i]), 1e-3 if fmt == torch.float32 else 2e-2, f"sequence {i}")
    # a padding row of a captured step: no slot in the state or the cache is touched
    if taps > 1:
        before = [t.clone() for t in (state, kc, vc)]
        lay = ops.StepLayout(2, 2, torch.tensor([0, 3]).cuda(), torch.tensor([-1, -1], dtype=torch.int32).cuda())
        turn = turns_of(ops, spec, torch.tensor([0, 3])) if rot else None
        ops.conv_attn_prep(full[0][:2].cuda()[:, gap:], w.cuda(), state, lay, turn, eps, torch.tensor([-1, -1]).cuda(), kc, vc, heads, kvh, dim, vdim)
        assert all(torch.equal(a, b) for a, b in zip(before, (state, kc, vc)))


def test_long_walks_of_the_convolution_cross_sequences():
    """A step of thousands of tokens, where a lane group walks several tokens at a time over the borders of many short sequences."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(1)
    heads, kvh, dim, vdim, taps = 8, 4, 64, 64, 4
    lens = ([5, 1, 7, 8, 9, 3, 2, 30] * 400)[:2600]
    pos0 = [0 if k % 3 else 6 for k in range(len(lens))]
    n, ch = sum(lens), (heads + 2 * kvh) * dim
    x = torch.randn(n, ch, generator=g)
    w, state = torch.randn(taps, ch, generator=g), torch.randn(len(lens), taps - 1, ch, generator=g)
    lay = step_layout(ops, lens, pos0, list(range(len(lens))))
    kc, vc = torch.zeros(n, kvh * dim).cuda(), torch.zeros(n, kvh * vdim).cuda()
    st = state.cuda()
    q = ops.conv_attn_prep(x.cuda(), w.cuda(), st, lay, None, 1e-6, torch.arange(n).cuda(), kc, vc, heads, kvh, dim, vdim, norm=False)
    a, pieces, tails = 0, [], []
    for k, m in enumerate(lens):
        head = state[k] if pos0[k] else torch.zeros(taps - 1, ch)
        rows = torch.cat([head, x[a:a + m]])
        pieces.append(fo.causal_conv(rows.double(), w.double().t())[taps - 1:])
        tails.append(rows[-(taps - 1):])
        a += m
    want = torch.cat(pieces)
    close(torch.cat([q.cpu(), kc.cpu(), vc.cpu()], 1), want, 1e-5, "rows")
    assert torch.equal(st.cpu(), torch.stack(tails))


def _attention_reference(q, k, v, scale, window, keep, sinks):
    """Every head's read-out of one whole sequence, (T, heads * vdim)."""
    heads, kvh = q.shape[1], k.shape[1]
    pos = torch.arange(q.shape[0])
    seen = fo.sees(pos, pos, window, keep)
    of = lambda h: h // (heads // kvh)
    return torch.cat([fo.sink_softmax_readout(q[:, h].double(), k[:, of(h)].double(), v[:, of(h)].double(), seen, scale,
                                              None if sinks is None else sinks[h].double()) for h in range(heads)], -1)


def _cached(rows, n_slots, seed):
    perm = torch.randperm(n_slots, generator=torch.Generator().manual_seed(seed)).tolist()
    caches = [torch.zeros(n_slots, r.shape[1] * r.shape[2]) for r in rows[0]]
    lists = []
    for parts in rows:
        s = [perm.pop() for _ in range(parts[0].shape[0])]
        for c, r in zip(caches, parts):
            c[s] = r.reshape(len(s), -1)
        lists.append(s)
    return caches, lists


def _attend(ops, q_rows, lens, totals, lists, kc, vc, fmt, decode, **kw):
    """ops.softcap_attn for a step that brings the last lens[b] tokens of the first totals[b] of sequence b."""
    flat = torch.tensor([s for b, l in enumerate(lists) for s in l[:totals[b]]], dtype=torch.int32).cuda()
    start = torch.tensor(np.concatenate([[0], np.cumsum(totals)[:-1]]), dtype=torch.int64).cuda()
    kv_len = torch.tensor(totals, dtype=torch.int32).cuda()
    lay = step_layout(ops, lens, [n - l for n, l in zip(totals, lens)], list(range(len(lens))), decode)
    return ops.softcap_attn(q_rows.to(fmt).cuda(), kc, vc, flat, start, kv_len, lay, cap=0.0, **kw).float().cpu()


# (window, kept first tokens, the key that every query asks loudly for)
VIEWS = [(0, 0, 0), (50, 0, 100), (50, 4, 3), (50, 4, 4), (64, 1, 0), (1, 2, 1), (33, 40, 39), (33, 70, 70), (1000, 5, 2), (37, 3, 63)]


@pytest.mark.parametrize("heads,kvh,dim,vdim", [(6, 2, 24, 14), (4, 1, 64, 48), (5, 5, 7, 3), (2, 1, 200, 264)])
@pytest.mark.parametrize("window,keep,loud", VIEWS)
def test_window_attention_with_kept_tokens_and_sinks(heads, kvh, dim, vdim, window, keep, loud):
    """Two sequences of unequal length at scattered slots; every query asks loudly for key `loud`, so a window that is one key off, or a kept
    token that is lost or is one too many, shows; sinks from far below the scores to far above; portions and single tokens that end just
    inside and just outside, with and without the key split; the result goes into columns of a wider buffer, times a constant."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(dim + window + keep)
    scale = 0.3
    n = [200, 77]
    sinks = torch.tensor([8.0, -20.0, 4.0, 30.0, 0.5, 1.0][:heads])
    q = [torch.randn(t, heads, dim, generator=g) for t in n]
    k = [torch.randn(t, kvh, dim, generator=g) for t in n]
    v = [torch.randn(t, kvh, vdim, generator=g) for t in n]
    for b in range(2):
        if loud < n[b]:
            for h in range(heads):
                k0 = k[b][loud, h // (heads // kvh)]
                q[b][:, h] = q[b][:, h] * 0.3 + 24.0 * k0 / k0.norm() ** 2
    want = [_attention_reference(q[b], k[b], v[b], scale, window or None, keep, sinks) for b in range(2)]
    (kc, vc), lists = _cached(list(zip(k, v)), 300, 3)
    kc, vc = kc.cuda(), vc.cuda()
    kw = dict(scale=scale, heads=heads, kv_heads=kvh, dim=dim, vdim=vdim, window=window, keep_first=keep, sinks=sinks.cuda())
    edge = max(window, 1) + loud if window and window + loud < 200 else 120
    for lens, totals, decode in (([200, 77], [200, 77], False), ([3, 30], [103, 77], False), ([1, 1], [min(edge, 200), 50], True), ([1, 1], [min(edge + 1, 200), 2], True),
                                 ([2, 1], [65, 2], False), ([1, 1], [1, 64], True), ([14, 13], [64, 26], False)):
        rows = torch.cat([q[b][totals[b] - lens[b]:totals[b]].reshape(lens[b], -1) for b in range(2)])
        ref = torch.cat([want[b][totals[b] - lens[b]:totals[b]] for b in range(2)])
        for split in (1, 4, None):
            wide = torch.full((len(rows), heads * vdim + 5), 3.0).cuda()
            got = _attend(ops, rows, lens, totals, lists, kc, vc, torch.float32, decode, n_split=split, out_mul=0.7, out=wide[:, 2:2 + heads * vdim], **kw)
            near(got, 0.7 * ref, 2e-3, f"lens {lens} of {totals}, split {split}")
            assert (wide[:, :2] == 3.0).all() and (wide[:, 2 + heads * vdim:] == 3.0).all()
    # the restatement itself depends on the window's size, on the number of kept tokens and on the sinks
    if window and loud < 77 and 1 < window < 100 and loud == keep:
        assert (_attention_reference(q[0], k[0], v[0], scale, window, keep + 1, sinks) - want[0]).abs().max() > 0.2
    assert (_attention_reference(q[0], k[0], v[0], scale, window or None, keep, None) - want[0]).abs().max() > 0.2


@pytest.mark.parametrize("dim,vdim", [(64, 64), (64, 48), (128, 96), (40, 24), (96, 128), (8, 8), (72, 120), (128, 16)])
@pytest.mark.parametrize("window,keep,loud", [(0, 0, 0), (100, 0, 100), (100, 4, 3), (100, 4, 4), (33, 40, 39), (33, 70, 70), (64, 1, 0), (7, 32, 31)])
def test_window_attention_on_the_matrix_cores(dim, vdim, window, keep, loud):
    """Steps of many tokens in bfloat16 take the tile kernel: ragged prompts that end in the middle of a key tile, kept tokens inside one tile,
    across two and beyond the window's first one, head sizes of whole tiles and below them; against the restatement on the same
    bfloat16 values, and the kernel for few tokens beside it."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(dim + vdim)
    heads, kvh, scale = 4, 2, 0.2
    n = [200, 77, 300, 1]
    bf = lambda x: x.to(torch.bfloat16).float()
    sinks = torch.tensor([-9.0, 2.0, 7.0, 0.0])
    q = [bf(torch.randn(t, heads, dim, generator=g) * 0.3) for t in n]
    k = [bf(torch.randn(t, kvh, dim, generator=g)) for t in n]
    v = [bf(torch.randn(t, kvh, vdim, generator=g)) for t in n]
    for b in (0, 2):
        for h in range(heads):
            k0 = k[b][loud, h // (heads // kvh)]
            q[b][:, h] = bf(q[b][:, h] * 0.3 + 36.0 * k0 / k0.norm() ** 2)
    want = [_attention_reference(q[b], k[b], v[b], scale, window or None, keep, sinks) for b in range(len(n))]
    (kc, vc), lists = _cached(list(zip(k, v)), 700, 5)
    kc, vc = kc.to(torch.bfloat16).cuda(), vc.to(torch.bfloat16).cuda()
    kw = dict(scale=scale, heads=heads, kv_heads=kvh, dim=dim, vdim=vdim, window=window, keep_first=keep, sinks=sinks.cuda(), n_split=1)
    for lens, totals in ((n, n), ([70, 3, 130, 1], [200, 77, 300, 1]), ([129, 77, 1, 1], [130, 77, 65, 1])):
        rows = torch.cat([q[b][totals[b] - lens[b]:totals[b]].reshape(lens[b], -1) for b in range(len(n))])
        ref = torch.cat([want[b][totals[b] - lens[b]:totals[b]] for b in range(len(n))])
        for cores in (True, False):
            wide = torch.full((len(rows), heads * vdim + 16), 3.0).to(torch.bfloat16).cuda()
            got = _attend(ops, rows, lens, totals, lists, kc, vc, torch.bfloat16, False, matrix_cores=cores, out_mul=1.5, out=wide[:, 8:8 + heads * vdim], **kw)
            err = ((got.double() - 1.5 * ref).abs() / (1.5 * ref.abs() + 0.05 * ref.std())).max().item()
            assert err < 1e-2, f"matrix cores {cores}, lens {lens} of {totals}: {err:.2e}"
            assert (wide[:, :8] == 3.0).all() and (wide[:, 8 + heads * vdim:] == 3.0).all()


LONG_ORDER = [[0, 1]] * 4 + [[0]] * 6 + [[1]] * 5 + [[2, 1]] * 5 + [[2]] * 4
LONG_CUTS = {0: [1, 2, 9, 8, 1, 1, 280, 1, 1, 300], 1: [5, 1, 1, 2, 8], 2: [2, 1, 6]}


@pytest.mark.parametrize("chunk", [None, 0, 5, 64])
@pytest.mark.parametrize("heads,dim,vdim,rot", [(2, 40, 70, 24), (1, 3, 5, 2), (3, 128, 36, 128), (1, 300, 20, 64), (2, 32, 300, 0)])
def test_rotated_retention_over_cuts_and_reused_slots(chunk, heads, dim, vdim, rot):
    """Steps of 1, 2 and hundreds of tokens (those of 256 and more in chunks side by side unless `chunk` says otherwise), a sequence that takes
    over a used slot, decays from one that keeps everything to one that forgets at once; single tokens through the scan and through
    the kernel for them, which also norms and gates."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(dim)
    hd, he, eps = heads * dim, heads * vdim, 1e-4
    full = {i: torch.randn(t, 3 + 2 * hd + 2 * he, generator=g) for i, t in {0: 604, 1: 17, 2: 9}.items()}
    decay = torch.tensor([0.9995, 0.5, 1.0][:heads])
    spec = {"dims": rot, "base": 40.0}
    k_mul = 0.37 * dim ** 0.5
    at, g0 = (3, 3 + hd, 3 + 2 * hd), 3 + 2 * hd + he

    def ref(x):
        x = x.double()
        pos = torch.arange(len(x))
        q, k, v = x[:, 3:3 + hd].view(-1, heads, dim), x[:, 3 + hd:3 + 2 * hd].view(-1, heads, dim), x[:, 3 + 2 * hd:g0].view(-1, heads, vdim)
        o = fo.retention_memory(q, k * 0.37 * dim, v, pos, spec, decay.double())       # (its own factor is dim^(-1/2))
        y = 1.4 * fo.unit_rms(o, eps).reshape(-1, he) * fo.silu(x[:, g0:])
        return torch.cat([o.reshape(-1, he), y], 1), (q, k, v)
    want = {i: ref(x)[0] for i, x in full.items()}
    mem = torch.full((3, heads, dim, vdim), 7.0).cuda()

    def run(x, lens, pos0, slots, decode):
        xd, lay, pos = x.cuda(), step_layout(ops, lens, pos0, slots, decode), positions_of(pos0, lens)
        turn = turns_of(ops, spec, pos, ahead=3) if rot else None
        again = mem.clone()
        kw = dict(turn=turn, k_mul=k_mul)
        o = ops.decay_scan(xd, at, decay.cuda(), mem, lay, heads, dim, vdim, chunk=chunk, **kw)
        y = ops.head_norm_gate(o, None, eps, gate=xd[:, g0:], kind="silu", mul=1.4)
        if decode:
            assert ops.decay_step_fits(lay, dim, vdim) == (vdim <= (1024 if vdim % 4 == 0 else 256))
            wide = torch.full((len(x), he + 4), 5.0).cuda()
            ops.decay_step(xd, at, decay.cuda(), again, lay, heads, dim, vdim, eps, gate_off=g0, gate_kind="silu", mul=1.4, out=wide[:, 3:3 + he], **kw)
            near(wide[:, 3:3 + he].cpu(), y.cpu(), 2e-4, "single tokens")
            close(again.cpu(), mem.cpu(), 1e-5, "memory after single tokens")
            assert (wide[:, :3] == 5.0).all() and (wide[:, 3 + he:] == 5.0).all()
        return torch.cat([o.reshape(len(x), he), y], 1).cpu()
    got = _walk(full, LONG_CUTS, SLOT, LONG_ORDER, run)
    for i in full:
        close(got[i][:, :he], want[i][:, :he], 1e-4, f"read-out of sequence {i}")
        close(got[i][:, he:], want[i][:, he:], 1e-3, f"normed and gated, sequence {i}")


@pytest.mark.parametrize("fmt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,dim,vdim,rot,act,kind", [(3, 10, 18, 8, "none", "silu"), (4, 64, 128, 64, "silu", "sigmoid"), (1, 1, 1, 0, "none", "none"),
                                                         (2, 128, 256, 32, "none", "silu"), (2, 20, 1024, 4, "silu", "silu"), (2, 700, 12, 2, "none", "silu")])
def test_retention_of_single_tokens(fmt, heads, dim, vdim, rot, act, kind):
    """One token per sequence: a first token (whatever its slot held), later ones, a padding row; every gate, both activations."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(dim)
    hd, he, eps, n = heads * dim, heads * vdim, 1e-3, 5
    x = torch.randn(n, 2 * hd + 2 * he, generator=g).to(fmt)
    decay = torch.tensor([0.9, 0.99, 0.5, 1.0][:heads])
    mem0 = torch.randn(6, heads, dim, vdim, generator=g)
    pos0, slots = [0, 5, 1000, 3, 0], [4, 0, 5, 2, -1]
    spec = {"dims": rot, "base": 100.0}
    mem = mem0.cuda()
    out = ops.decay_step(x.cuda(), (0, hd, 2 * hd), decay.cuda(), mem, step_layout(ops, [1] * n, pos0, slots, True), heads, dim, vdim, eps, act=act,
                         turn=turns_of(ops, spec, torch.tensor(pos0)) if rot else None, k_mul=0.5, gate_off=2 * hd + he, gate_kind=kind).float().cpu()
    f = fo.silu if act == "silu" else (lambda z: z)
    gates = {"none": lambda z: 1.0, "sigmoid": torch.sigmoid, "silu": fo.silu}[kind]
    after = mem0.clone().double()
    for b in range(4):
        xb, pos = x[b:b + 1].double(), torch.tensor([pos0[b]])
        q, k = (fo.turned(f(xb[:, a:a + hd]).view(1, heads, dim), pos, spec) for a in (0, hd))
        v = f(xb[:, 2 * hd:2 * hd + he]).view(1, heads, vdim)
        o = []
        for h in range(heads):
            s = torch.zeros(dim, vdim).double() if pos0[b] == 0 else mem0[slots[b], h].double()
            oh, after[slots[b], h] = fo.decayed_memory(q[:, h], 0.5 * k[:, h], v[:, h], decay[h].double(), s)
            o.append(oh)
        want = fo.unit_rms(torch.stack(o, 1), eps).reshape(1, he) * gates(xb[:, 2 * hd + he:])
        near(out[b:b + 1], want, 2e-3 if fmt == torch.float32 else 2e-2, f"sequence {b}")
    close(mem.cpu(), after, 1e-5, "memories")
    assert (out[4] == 0).all() and torch.equal(mem.cpu()[[1, 3]], mem0[[1, 3]])


def test_weights_are_the_softmax_over_the_chosen_logits():
    """Rows of the logits are slices of wider rows (one more number per token stands beside them), large logits included."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(3)
    for n_exp, top, t, size in ((6, 3, 50, 1.0), (16, 2, 9, 40.0), (4, 1, 5, 1.0), (70, 8, 33, 3.0), (5, 5, 7, 1.0)):
        z = torch.randn(t, n_exp + 1, generator=g) * size
        idx, wts = ops.moe_route_softmax(z.cuda()[:, :n_exp], top, 0, 0, 0.0)
        for r in range(t):
            ids, share = fo.chosen(z[r, :n_exp].double(), top)
            assert idx[r].cpu().tolist() == ids
            assert torch.allclose(wts[r].cpu().double(), share, rtol=2e-5, atol=1e-7), (n_exp, top, r)


@pytest.mark.parametrize("fmt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("ff,t", [(28, 5), (64, 300), (7, 1)])
def test_shared_expert_hidden_rows_behind_their_gate(fmt, ff, t):
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(ff)
    x = torch.randn(t, 8 + 2 * ff, generator=g).to(fmt)
    z = torch.randn(t, 5, generator=g)
    wide = torch.full((t, ff + 16), 3.0).to(fmt).cuda()
    ops.moe_glu(x.cuda()[:, 8:], float("inf"), 1.0, 0.0, row_gate=z.cuda()[:, 4], out=wide[:, 8:8 + ff])
    want = torch.sigmoid(z[:, 4:].double()) * fo.silu(x[:, 8:8 + ff].double()) * x[:, 8 + ff:].double()
    near(wide[:, 8:8 + ff].float().cpu(), want, 1e-4 if fmt == torch.float32 else 1e-2)
    assert (wide[:, :8] == 3.0).all() and (wide[:, 8 + ff:] == 3.0).all()


@pytest.mark.parametrize("fmt", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("width,ff,n_exp,top,t", [(64, 48, 4, 2, 1), (72, 40, 3, 3, 37), (128, 16, 20, 2, 9), (520, 264, 2, 1, 50), (40, 8, 1, 1, 33), (36, 20, 5, 2, 6)])
@pytest.mark.parametrize("weight_out", [True, False])
def test_experts_of_a_step_of_few_tokens(fmt, width, ff, n_exp, top, t, weight_out):
    """An expert that every token chooses (more pairs than a tile of 16 holds), experts nobody chooses, depths that end inside a block of 128
    and inside 32, sizes without 16-byte rows; against the restatement on the same values, weights on the outputs and on the inputs;
    a token's result is the same bits alone and beside others."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(width + t)
    h = torch.randn(t, width, generator=g).to(fmt)
    w_gu, w_d = (torch.randn(n_exp, 2 * ff, width, generator=g) * width ** -0.5).to(fmt), (torch.randn(n_exp, width, ff, generator=g) * ff ** -0.5).to(fmt)
    idx = torch.stack([torch.cat([torch.zeros(1, dtype=torch.long), 1 + torch.randperm(n_exp - 1, generator=g)[:top - 1] // 1]) if n_exp > 1 else torch.zeros(1, dtype=torch.long)
                       for _ in range(t)])
    wts = torch.rand(t, top, generator=g) + 0.1
    rounded = lambda z: z.to(fmt).double()            # what a product hands on in the activations' format
    want = torch.zeros(t, width, dtype=torch.float64)
    for r in range(t):
        for e, s in zip(idx[r].tolist(), wts[r]):
            x = h[r].double() if weight_out else rounded(s * h[r].float())
            hidden = rounded(fo.silu(rounded(w_gu[e, :ff].double() @ x)) * rounded(w_gu[e, ff:].double() @ x))
            want[r] += (s.double() if weight_out else 1.0) * rounded(w_d[e].double() @ hidden)
    args = [x.cuda() for x in (h, idx.to(torch.int32), wts, w_gu, w_d)]
    got = ops.moe_expert_rows(*args, float("inf"), 1.0, 0.0, weight_out)
    near(got.float().cpu(), want, 1e-3 if fmt == torch.float32 else 3e-2, "experts")
    alone = torch.cat([ops.moe_expert_rows(args[0][r:r + 1], args[1][r:r + 1].contiguous(), args[2][r:r + 1].contiguous(), *args[3:], float("inf"), 1.0, 0.0, weight_out)
                       for r in range(min(t, 5))])
    assert torch.equal(alone, got[:len(alone)])


# ---- one mechanism at a time ---------------------------------------------------------------------------------------------
ONE = {
    "attention and retention side by side": ([layer(mlp=None)], {}),
    "attention alone (the other side weighs nothing)": ([layer(mlp=None, right_scale=0.0)], {}),
    "retention alone (the other side weighs nothing)": ([layer(mlp=None, left_scale=0.0)], {}),
    "both scales equal": ([layer(mlp=None, left_scale=1.0, right_scale=1.0)], {}),
    "all keys": ([layer(left={"mask": None}, mlp=None)], {}),
    "a window of one token": ([layer(left={"mask": {"size": 1, "keep_first": 0}}, mlp=None)], {}),
    "a window of one token behind two kept ones": ([layer(left={"mask": {"size": 1, "keep_first": 2}}, mlp=None)], {}),
    "more kept tokens than the window holds": ([layer(left={"mask": {"size": 5, "keep_first": 20}}, mlp=None)], {}),
    "a window of a page without kept tokens": ([layer(left={"mask": {"size": 64}}, mlp=None)], {}),
    "a window longer than the sequence": ([layer(left={"mask": {"size": 500, "keep_first": 9}}, mlp=None)], {}),
    "one tap": ([layer(left={"conv": 1}, mlp=None)], {}),
    "no convolution": ([layer(left={"conv": None}, mlp=None)], {}),
    "nine taps": ([layer(left={"conv": 9}, mlp=None)], {}),
    "rotation of whole heads, no scaling": ([layer(left={"rot": {"dims": 20, "base": 300.0}}, right={"rot": {"dims": 10, "base": 300.0}}, mlp=None)], {}),
    "no rotation": ([layer(left={"rot": None}, right={"rot": None}, mlp=None)], {}),
    "one rotation for both sides": ([layer(left={"rot": {"dims": 8, "base": 700.0}}, mlp=None)], {}),
    "one head each": ([layer(left={"heads": 1, "kv_heads": 1}, right={"heads": 1, "decay": [0.97]}, mlp=None)], {}),
    "five heads on one key, values wider than keys": ([layer(left={"heads": 5, "kv_heads": 1, "dim": 6, "vdim": 30, "rot": {"dims": 6, "base": 50.0}}, mlp=None)], {}),
    "memories that keep and memories that forget": ([layer(right={"decay": [1.0, 0.01, 0.9999]}, mlp=None)], {}),
    "experts beside a shared one": ([layer()], {}),
    "experts, all of all, no shared one": ([layer(mlp={"kind": "moe", "expert": {"ff": 8}, "router": {"experts": 3, "top": 3}})], {}),
    "one expert": ([layer(mlp={"kind": "moe", "expert": {"ff": 8}, "router": {"experts": 1, "top": 1}, "shared": {"ff": 5}})], {}),
    "top one of four": ([layer(mlp=MOE1)], {}),
    "logits as they are": ([layer()], {"logit_scale": 1.0}),
    "a large eps": ([layer()], {"eps": 0.3}),
}


@pytest.mark.parametrize("name", list(ONE))
def test_each_mechanism_alone_whole_cut_and_token_by_token(tmp_path, name):
    layers, kw = ONE[name]
    cfg = make_cfg(layers, **kw)
    w = weights_of(cfg, 1)
    eng = make_engine(model_dir(tmp_path, cfg, w), pool=256)
    toks = tokens(80, cfg["vocab"], 3)
    want = forward(cfg, w, toks)
    close(replay(eng, {"a": toks}, [[("a", 80)]])["a"], want, F32_TOL, "whole")
    close(replay(eng, {"b": toks}, [[("b", n)] for n in cuts_of(80, [2, 7, 1, 9, 3, 8, 16])])["b"], want, F32_TOL, "cut")
    close(replay(eng, {"c": toks}, [[("c", 2)]] * 40)["c"], want, F32_TOL, "portions of two")
    close(replay(eng, {"d": toks}, [[("d", 1)]] * 80)["d"], want, F32_TOL, "token by token")
    eng.shutdown()


def test_residual_after_every_layer(tmp_path):
    cfg = make_cfg(STACK)
    w = weights_of(cfg, 5)
    eng = make_engine(model_dir(tmp_path, cfg, w), pool=128)
    toks = tokens(23, cfg["vocab"], 1)
    streams = []
    fo.forward(cfg, w, toks, streams)
    model = eng.model_runner.model
    model.layer_streams = []
    replay(eng, {"a": toks}, [[("a", 23)]])
    got, model.layer_streams = model.layer_streams, None
    assert len(got) == len(streams) == 3
    for i, (a, b) in enumerate(zip(got, streams)):
        close(a.float().cpu(), b, 5e-5, f"after layer {i}")
    eng.shutdown()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sizes_that_fit_no_vector_width(tmp_path, dtype):
    """A width, head sizes, feed-forward sizes and a vocabulary that are multiples of nothing useful (no 16-byte rows anywhere)."""
    odd = [layer(left={"heads": 3, "kv_heads": 1, "dim": 10, "vdim": 11, "rot": {"dims": 6, "base": 99.0}, "mask": {"size": 21, "keep_first": 2}},
                 right={"heads": 5, "dim": 3, "vdim": 7, "decay": [0.9, 0.8, 0.99, 0.5, 0.95], "rot": {"dims": 2, "base": 10.0}},
                 mlp={"kind": "moe", "expert": {"ff": 9}, "router": {"experts": 9, "top": 3}, "shared": {"ff": 5}}),
           layer(left={"heads": 7, "kv_heads": 7, "dim": 5, "vdim": 1, "rot": None, "conv": 5}, right={"heads": 1, "dim": 1, "vdim": 3, "decay": [0.7], "rot": None},
                 mlp={"kind": "moe", "expert": {"ff": 3}, "router": {"experts": 2, "top": 1}})]
    cfg = make_cfg(odd, width=49, vocab=37)
    w = weights_of(cfg, 4)
    eng = make_engine(model_dir(tmp_path, cfg, w), dtype=dtype, pool=256)
    toks = tokens(45, 37, 8)
    want = forward(cfg, w, toks)
    got = replay(eng, {"a": toks}, [[("a", 33)], [("a", 2)]] + [[("a", 1)]] * 10)["a"]
    if dtype == "float32":
        close(got, want, F32_TOL, "float32")
        close(replay(eng, {"b": toks}, [[("b", 45)]])["b"], want, F32_TOL, "whole")
    else:
        within_rounding(got, want)
    eng.shutdown()


def loud_first_layer(cfg, w, key_token, by=9.0):
    """Queries of the first layer that ask for ONE token id: its key, as it comes out of projection and convolution, gets a direction of
    its own and every query carries it.  No rotation in that layer, one tap that counts."""
    left = cfg["layers"][0]["mixer"]["left"]
    assert "rot" not in left
    for n in "qk":
        w[f"l0.mix.left.{n}.conv"] = torch.zeros_like(w[f"l0.mix.left.{n}.conv"])
        w[f"l0.mix.left.{n}.conv"][:, -1] = 1.0
    x = w["embed"].double()
    h = fo.layer_norm(x, w["l0.norm1"].double(), w["l0.norm1.b"].double(), cfg["norm"]["eps"])
    mark = h[key_token] / h[key_token].norm() ** 2
    wk, wq, d = w["l0.mix.left.k"].double(), w["l0.mix.left.q"].double(), left["dim"]
    axis = torch.zeros(d).double()
    axis[0] = 1.0
    wk += by * torch.cat([axis] * left["kv_heads"])[:, None] * mark[None, :]
    common = torch.linalg.lstsq(h, torch.ones(len(h), 1).double()).solution[:, 0]           # h . common is close to one for every token
    wq += by * torch.cat([axis] * left["heads"])[:, None] * common[None, :]
    w["l0.mix.left.k"], w["l0.mix.left.q"] = wk.to(torch.bfloat16).float(), wq.to(torch.bfloat16).float()
    return w


def test_first_tokens_page_borders_and_window_edges_in_prompts_and_decoding(tmp_path):
    """Prompts of 1 to 129 tokens; pages of 64, key tiles and a window of 50 with two kept tokens crossed token by token and by portions that
    start, end and turn at them.  One token id, which stands once in the sequence, is what every query of the first layer asks for: inside
    the window it stands out, outside it is gone -- unless it is a kept one."""
    cfg = make_cfg([layer(left={"mask": {"size": 50, "keep_first": 2}, "rot": None, "scale": 1.0}), layer(left={"mask": {"size": 64, "keep_first": 1}}), STACK[2]])
    for place in (70, 1, 2):
        w = loud_first_layer(cfg, weights_of(cfg, 12), 60)
        toks = [t % 60 for t in tokens(200, cfg["vocab"], 6)]
        toks[place] = 60
        want = forward(cfg, w, toks)
        name = f"loud{place}"
        eng = make_engine(model_dir(tmp_path, cfg, w, name=name), pool=1024)
        for n in (1, 2, 3, 49, 50, 51, 52, 63, 64, 65, 128, 129):
            close(replay(eng, {f"p{n}": toks[:n]}, [[(f"p{n}", n)]])[f"p{n}"], want[:n], F32_TOL, f"prompt of {n}")
        sched = [[("a", 1)]] * 3 + [[("a", 45)]] + [[("a", 1)]] * 5 + [[("a", 2)], [("a", 8)], [("a", 2)], [("a", 32)]] + [[("a", 1)]] * 28 + \
                [[("a", 21)]] + [[("a", 1)]] * 6 + [[("a", 48)]]
        assert sum(n for step in sched for _, n in step) == 200
        close(replay(eng, {"a": toks}, sched)["a"], want, F32_TOL, "edges crossed token by token")
        eng.shutdown()
        # the window and the kept tokens count: one more of either is another function, from the place where it must be one on
        # -- exactly where the loud token leaves the window, and from its first absence on where it is the kept token in question
        for change, first, at in (({"size": 51, "keep_first": 2}, 50, 120 if place == 70 else None), ({"size": 50, "keep_first": 3}, 52, 52 if place == 2 else None),
                                  ({"size": 50, "keep_first": 1}, 51, 51 if place == 1 else None)):
            other = json.loads(json.dumps(cfg))
            other["layers"][0]["mixer"]["left"]["mask"] = change
            moved = (forward(other, w, toks) - want).abs().amax(dim=1)
            assert moved[:first].max() == 0, (place, change)
            if at is not None:
                assert moved[at] > 20 * moved[at - 1] and moved[at] > 100 * F32_TOL * want.std(), (place, change)


def test_far_tokens_and_old_state_count(tmp_path):
    """330 tokens, the first of them still seen at the end: as a kept token far behind the window (asked for loudly) and in memories with
    decays close to one."""
    cfg = make_cfg([layer(left={"mask": {"size": 40, "keep_first": 1}, "rot": None, "scale": 1.0}, right={"decay": [0.9995, 1.0, 0.999]}), layer()])
    w = loud_first_layer(cfg, weights_of(cfg, 7), 60)
    toks = [60] + [t % 60 for t in tokens(329, cfg["vocab"], 2)]
    want = forward(cfg, w, toks)
    eng = make_engine(model_dir(tmp_path, cfg, w), pool=512)
    got = replay(eng, {"a": toks}, [[("a", 255)], [("a", 1)], [("a", 1)], [("a", 2)], [("a", 30)]] + [[("a", 1)]] * 41)["a"]
    close(got, want, F32_TOL, "far tokens")
    close(replay(eng, {"b": toks}, [[("b", 330)]])["b"], want, F32_TOL, "whole, the memories in chunks side by side")
    for side in ("keep_first", "decay"):        # each of the two alone carries the first token to the end
        one = json.loads(json.dumps(cfg))
        if side == "keep_first":
            one["layers"][0]["mixer"]["right_scale"] = one["layers"][1]["mixer"]["right_scale"] = 0.0
        else:
            one["layers"][0]["mixer"]["left_scale"] = one["layers"][1]["mixer"]["left_scale"] = 0.0
        assert (forward(one, w, [(toks[0] + 1) % 61] + toks[1:])[-1] - forward(one, w, toks)[-1]).abs().max() > 8 * F32_TOL * want.std(), side
    eng.shutdown()


def test_sinks_take_their_share(tmp_path):
    """Sinks from silent to overwhelming, in prompts and single tokens; without them the logits are others."""
    cfg = make_cfg([layer(mlp=None), layer(left={"mask": {"size": 5, "keep_first": 0}}, mlp=None)])
    w = weights_of(cfg, 3)
    for i in (0, 1):
        w[f"l{i}.mix.left.sink"] = torch.tensor([-30.0, 0.0, 2.0, 5.0, 40.0, -1.0])
    toks = tokens(60, cfg["vocab"], 5)
    want = forward(cfg, w, toks)
    eng = make_engine(model_dir(tmp_path, cfg, w), pool=128)
    close(replay(eng, {"a": toks}, [[("a", 41)], [("a", 2)]] + [[("a", 1)]] * 17)["a"], want, F32_TOL, "cut")
    eng.shutdown()
    silent = dict(w, **{f"l{i}.mix.left.sink": torch.full((6,), -1e4) for i in (0, 1)})
    assert ((forward(cfg, silent, toks) - want).abs().amax(dim=1) > 8 * F32_TOL * want.std()).all()


def drawn_configuration(rnd):
    """A configuration drawn at random: 1 to 4 layers, sizes from small and odd to those the vector and matrix-core kernels take."""
    layers = []
    for _ in range(rnd.randint(1, 4)):
        kvh, dim = rnd.choice([1, 2, 3]), rnd.choice([6, 16, 64, 40, 96])
        left = {"heads": kvh * rnd.choice([1, 2, 4]), "kv_heads": kvh, "dim": dim, "vdim": rnd.choice([5, 16, 64, 48, 128]), "conv": rnd.choice([1, 2, 3, 4, 6]),
                "scale": rnd.choice([0.2, 1.0, 2.5]), "rot": rnd.choice([None, {"dims": rnd.choice([2, dim // 2 // 2 * 2, dim]), "base": rnd.choice([50.0, 1e4]),
                                                                               **({"scaling": BANDS} if rnd.random() < 0.5 else {})}]),
                "mask": rnd.choice([None, {"size": rnd.choice([3, 17, 64, 100]), "keep_first": rnd.choice([0, 1, 4, 33])}])}
        heads, rdim = rnd.choice([1, 2, 5]), rnd.choice([4, 16, 40])
        right = {"heads": heads, "dim": rdim, "vdim": rnd.choice([6, 32, 80]), "decay": [rnd.choice([0.5, 0.9, 0.99, 0.9995]) for _ in range(heads)],
                 "rot": rnd.choice([None, {"dims": rnd.choice([2, rdim]), "base": 30.0}])}
        n = rnd.choice([1, 3, 8])
        mlp = rnd.choice([None, {"kind": "moe", "expert": {"ff": rnd.choice([8, 20, 32])}, "router": {"experts": n, "top": rnd.randint(1, min(n, 4))}}])
        if mlp and rnd.random() < 0.7:
            mlp["shared"] = {"ff": rnd.choice([7, 40])}
        layers.append(layer(left=left, right=right, mlp=mlp, left_scale=rnd.choice([1.0, 0.4, 2.0]), right_scale=rnd.choice([1.0, 0.7])))
    return make_cfg(layers, width=rnd.choice([24, 50, 96, 160]), vocab=rnd.choice([37, 130, 301]), eps=rnd.choice([1e-5, 1e-3]), logit_scale=rnd.choice([1.0, 0.3, 4.0]))


@pytest.mark.parametrize("seed", range(12))
def test_configurations_drawn_at_random(tmp_path, seed):
    """Whole, in portions of drawn sizes with single tokens at the end, and two requests of unequal length side by side."""
    import random
    rnd = random.Random(seed)
    cfg = drawn_configuration(rnd)
    w = weights_of(cfg, seed)
    eng = make_engine(model_dir(tmp_path, cfg, w), pool=512)
    n = rnd.choice([70, 131, 200])
    toks, other = tokens(n, cfg["vocab"], seed), tokens(45, cfg["vocab"], seed + 100)
    want, want_other = forward(cfg, w, toks), forward(cfg, w, other)
    what = json.dumps(cfg)
    close(replay(eng, {"a": toks}, [[("a", n)]])["a"], want, F32_TOL, "whole: " + what)
    cuts = cuts_of(n - 9, [rnd.choice([2, 3, 17, 64, 65]) for _ in range(5)]) + [1] * 9
    close(replay(eng, {"b": toks}, [[("b", c)] for c in cuts])["b"], want, F32_TOL, "cut: " + what)
    sched = [[("c", 30), ("d", 2)], [("c", 1), ("d", 40)]] + [[("c", 1), ("d", 1)]] * 3 + [[("c", n - 34)]]
    got = replay(eng, {"c": toks, "d": other}, sched)
    close(got["c"], want, F32_TOL, "side by side: " + what)
    close(got["d"], want_other, F32_TOL, "side by side, the shorter one: " + what)
    eng.shutdown()


# ---- the whole stack ------------------------------------------------------------------------------------------------------
def test_batches_of_unequal_requests_in_a_small_pool(tmp_path):
    """Four live requests at most in a pool smaller than the sum of all: portions beside single tokens, a request that
    pauses for some steps, token slots and state slots that change hands (six requests, four state slots)."""
    cfg = make_cfg(STACK)
    w = weights_of(cfg, 2)
    eng = make_engine(model_dir(tmp_path, cfg, w), pool=160, max_bs=4)
    req = {f"r{k}": tokens(n, cfg["vocab"], 30 + k) for k, n in enumerate([70, 41, 1, 23, 55, 38])}
    want = {i: forward(cfg, w, t) for i, t in req.items()}
    sched = [[("r0", 16), ("r1", 2)], [("r0", 1), ("r1", 30), ("r2", 1)], [("r0", 40), ("r3", 3)], [("r1", 1), ("r3", 1)],
             [("r0", 1), ("r1", 1), ("r3", 17)], [("r0", 12), ("r1", 7), ("r3", 2)],          # r0, r1, r3 done: 134 slots come back
             [("r4", 2), ("r5", 30)], [("r4", 50), ("r5", 1)], [("r4", 1), ("r5", 1)], [("r4", 2), ("r5", 6)]]
    got = replay(eng, req, sched)
    for i in req:
        close(got[i], want[i], F32_TOL, i)
    assert eng.scheduler.state_slots.num_free() == 4
    eng.shutdown()


NO_EXPERTS = [json.loads(json.dumps(dict(x, mlp=None))) for x in STACK]


def test_bfloat16_stays_within_rounding(tmp_path):
    """No experts: a router's close call may go either way in 16 bits, which says nothing about the kernels."""
    cfg = make_cfg(NO_EXPERTS)
    toks = tokens(90, cfg["vocab"], 4)
    want = forward(cfg, weights_of(cfg, 2), toks)
    eng = make_engine(model_dir(tmp_path, cfg), dtype="bfloat16", seed=2)
    within_rounding(replay(eng, {"a": toks}, [[("a", 50)], [("a", 2)]] + [[("a", 1)]] * 38)["a"], want)
    eng.shutdown()


def test_bfloat16_with_heads_for_the_matrix_cores(tmp_path):
    """Head sizes the tile kernel is built for (and some it pads), prompts long enough to take it, one expert that every token takes: whole
    prompts against portions and single tokens, and both against the restatement within rounding."""
    one = {"kind": "moe", "expert": {"ff": 64}, "router": {"experts": 1, "top": 1}, "shared": {"ff": 32}}
    right = {"heads": 2, "dim": 64, "vdim": 96, "decay": [0.98, 0.999], "rot": {"dims": 32, "base": 1e4}}
    cfg = make_cfg([layer(left={"heads": 8, "kv_heads": 4, "dim": 64, "vdim": 64, "rot": {"dims": 32, "base": 1e4}, "mask": {"size": 150, "keep_first": 4}}, right=right, mlp=one),
                    layer(left={"heads": 4, "kv_heads": 1, "dim": 80, "vdim": 40, "rot": {"dims": 48, "base": 1e3}, "conv": 3, "mask": {"size": 90, "keep_first": 40}},
                          right=right, mlp=None)], width=128, vocab=97)
    w = weights_of(cfg, 3)
    eng = make_engine(model_dir(tmp_path, cfg, w), dtype="bfloat16", pool=1024)
    toks = tokens(400, 97, 9)
    want = forward(cfg, w, toks)
    within_rounding(replay(eng, {"a": toks}, [[("a", 400)]])["a"], want, "whole")
    within_rounding(replay(eng, {"b": toks}, [[("b", 230)], [("b", 100)], [("b", 2)], [("b", 63)]] + [[("b", 1)]] * 5)["b"], want, "cut")
    eng.shutdown()


def test_checkpoint_with_a_missing_or_misshapen_tensor_is_refused(tmp_path):
    cfg = make_cfg(STACK)
    w = weights_of(cfg, 0)
    for gone in ("l0.mix.left.k", "l1.mix.left.v.conv", "l0.mix.left.sink", "l0.mlp.shared.sg", "l2.mlp.e3.up", "l1.norm1.b", "final.norm.b", "l0.mix.right.g"):
        bad = dict(w)
        del bad[gone]
        with pytest.raises(KeyError):
            make_engine(model_dir(tmp_path, cfg, bad, name="missing_" + gone.replace(".", "_")))
    for k, (name, shape) in enumerate((("l0.mix.left.q.conv", (120, 3)), ("l0.mix.right.o", (40, 53)), ("head", (61, 41)), ("l0.mlp.router", (7, 40)))):
        bad = dict(w)
        bad[name] = torch.zeros(*shape)
        with pytest.raises(ValueError):
            make_engine(model_dir(tmp_path, cfg, bad, name=f"shape{k}"))


# ---- generation: the scheduler's own choices ---------------------------------------------------------------------------
def oracle_greedy(w, cfg, prompt, n_new):
    return greedy(lambda t: forward(cfg, w, t), prompt, n_new)


@pytest.mark.parametrize("chunked", [False, True], ids=["whole prompts", "chunked prefill"])
def test_greedy_generation_through_the_engine(tmp_path, chunked):
    """Prompts of unequal length admitted together, decoded as one batch; more requests than state slots, so the later ones wait
    for a slot that an earlier one gives back; with chunked prefill the prompts are computed in portions of seven tokens.  Long
    decoding (70 tokens, across a page of 64 and past the window) for one of them."""
    from nano_vllm_x_amd.core.common import SamplingParams
    cfg = make_cfg(STACK)
    kw = dict(max_prefill_tokens=7, chunked_prefill=True) if chunked else {}
    eng = make_engine(model_dir(tmp_path, cfg), pool=400, max_bs=3, seed=9, **kw)
    w = weights_of(cfg, 9)
    prompts = {f"r{k}": tokens(n, cfg["vocab"], 20 + k) for k, n in enumerate([5, 19, 1, 12, 9])}
    new = {"r0": 70, "r1": 5, "r2": 8, "r3": 4, "r4": 6}
    for i, p in prompts.items():
        eng.add_sequence(i, list(p), SamplingParams(temperature=0.0, ignore_eos=True, max_new_tokens=new[i]))
    out = {i: [] for i in prompts}
    steps = 0
    while eng.has_unfinished_sequences():
        for o in eng.step():
            out[o.seq_id].append(o.new_token_id)
        steps += 1
        assert steps < 600
    for i, p in prompts.items():
        assert out[i] == oracle_greedy(w, cfg, p, new[i]), i
    assert eng.scheduler.state_slots.num_free() == 3
    eng.shutdown()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decode_steps_replay_a_captured_graph(tmp_path, dtype):
    """With graphs on, every decode step replays the graph of its batch size, with prefill steps of later requests (eager work on
    the same cache and state) between the replays; batch sizes change as requests end.  float32: the tokens are the
    restatement's; bfloat16: the graph's tokens are those of eager steps (same kernels, same order)."""
    from nano_vllm_x_amd.core.common import SamplingParams
    from nano_vllm_x_amd.core.engine import Engine
    cfg = make_cfg(STACK)
    path = model_dir(tmp_path, cfg)
    prompts = {f"r{k}": tokens(n, cfg["vocab"], 40 + k) for k, n in enumerate([9, 26, 2, 17, 5])}
    new = {"r0": 20, "r1": 5, "r2": 11, "r3": 3, "r4": 7}

    def run(eager):
        eng = Engine(model=path, gpu_memory_utilization=0.5, max_bs=3, enforce_eager=eager, context_len=128, kv_cache_size=300,
                     dtype=dtype, seed=5)
        for i, p in prompts.items():
            eng.add_sequence(i, list(p), SamplingParams(temperature=0.0, ignore_eos=True, max_new_tokens=new[i]))
        out = {i: [] for i in prompts}
        while eng.has_unfinished_sequences():
            for o in eng.step():
                out[o.seq_id].append(o.new_token_id)
        stats = dict(eng.model_runner.stats)
        eng.shutdown()
        return out, stats

    got, stats = run(False)
    assert stats["graph_steps"] > 15 and stats["eager_decode_steps"] == 0
    if dtype == "float32":
        w = weights_of(cfg, 5)
        for i, p in prompts.items():
            assert got[i] == oracle_greedy(w, cfg, p, new[i]), i
    else:
        assert got == run(True)[0]


def test_generate_entry_point(tmp_path):
    from nano_vllm_x_amd import LLM, SamplingParams
    cfg = make_cfg(STACK, vocab=300)
    llm = LLM(model_dir(tmp_path, cfg), gpu_memory_utilization=0.5, max_bs=2, enforce_eager=True, context_len=256, kv_cache_size=256,
              dtype="float32", seed=4)
    prompt = tokens(11, 300, 1)

    async def run():
        ids = []
        async for o in llm.generate(list(prompt), SamplingParams(temperature=0.0, ignore_eos=True, max_new_tokens=5, eos_token_id=0)):
            ids.append(o.token_id)
        return ids

    assert asyncio.run(run()) == oracle_greedy(weights_of(cfg, 4), cfg, prompt, 5)
    llm.shutdown()


def test_preempted_sequence_starts_again_from_an_empty_state(tmp_path):
    from nano_vllm_x_amd.core.common import SamplingParams
    cfg = make_cfg(STACK)
    eng = make_engine(model_dir(tmp_path, cfg), pool=64, max_bs=2, seed=6)
    w = weights_of(cfg, 6)
    prompts = {"a": tokens(20, cfg["vocab"], 1), "b": tokens(25, cfg["vocab"], 2)}
    for i, p in prompts.items():
        eng.add_sequence(i, list(p), SamplingParams(temperature=0.0, ignore_eos=True, max_new_tokens=14))
    out = {i: [] for i in prompts}
    while eng.has_unfinished_sequences():       # 45 + 2 * 14 tokens do not fit 64 slots: the younger sequence is preempted
        for o in eng.step():
            out[o.seq_id].append(o.new_token_id)
    for i, p in prompts.items():
        assert out[i] == oracle_greedy(w, cfg, p, 14), i
    eng.shutdown()


def test_command_line_generates_what_the_restatement_does(tmp_path):
    import subprocess
    import sys
    cfg = make_cfg(STACK, vocab=90)
    path = model_dir(tmp_path, cfg)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = subprocess.run([sys.executable, "-m", "nano_vllm_x_amd", "--model", path, "--prompt-ids", "5,17,3,44", "--prompt-ids", "8",
                          "--max-new-tokens", "6", "--dtype", "float32", "--kv-cache-size", "128", "--context-len", "64", "--max-bs", "2",
                          "--seed", "3"], cwd=root, capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    lines = [json.loads(x) for x in out.stdout.splitlines() if x.startswith("{")]
    w = weights_of(cfg, 3)
    assert [x["prompt"] for x in lines] == [[5, 17, 3, 44], [8]]
    for x in lines:
        assert x["generated_ids"] == oracle_greedy(w, cfg, x["prompt"], 6)


def test_trace_runner_replays_steps_from_standard_input(tmp_path):
    """bin/trace_run on a model directory: two requests, portions beside single tokens, one request ended and its id used again;
    the logits it writes are the restatement's."""
    import subprocess
    cfg = make_cfg(STACK, vocab=80)
    w = weights_of(cfg, 11)
    path = model_dir(tmp_path, cfg, w)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    a, b = tokens(30, 80, 1), tokens(12, 80, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:9], "want": [0, 8]}, {"id": "b", "tokens": b[:1], "want": [0]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[9:29], "want": []}, {"id": "b", "tokens": b[1:], "want": [10]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[29:], "want": [0]}, {"id": "b", "tokens": a[:5], "want": [4]}], "end": ["a", "b"]}]
    out_dir = tmp_path / "out"
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(out_dir), "--max-tokens", "128"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=600, cwd=root)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    la, lb = forward(cfg, w, a), forward(cfg, w, b)
    got = [torch.from_numpy(np.fromfile(out_dir / f"{k}.f32", dtype="<f4").reshape(-1, 80).copy()) for k in range(3)]
    close(got[0], torch.stack([la[0], la[8], lb[0]]), F32_TOL, "step 0")
    close(got[1], lb[11:12], F32_TOL, "step 1")
    close(got[2], torch.stack([la[29], la[4]]), F32_TOL, "step 2")
