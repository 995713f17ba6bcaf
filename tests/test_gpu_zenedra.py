"""Zenedra through the engine, and its kernels alone, against the plain restatement in oracle/zenedra_oracle.py.

Every test makes its own small configuration and weights.  The engine is built on a directory that holds config.json (and,
where the weights are made by the test, model.safetensors), as a user's would be; steps are given with Engine.run_given (the
replay entry point) or chosen by the scheduler (Engine.step / LLM.generate).  Comparisons are in float32 unless a test says
otherwise: there a structural fault (a key of another chunk, a lost state, a pass that reads another pass's rows) stands far above
rounding.
"""
import asyncio
import json
import os

import numpy as np
import pytest
import torch

from oracle import zenedra_oracle as zo
from seq_drivers import F32_TOL, close, cuts_of, greedy, make_engine, model_dir, replay, step_layout, tokens

pytestmark = pytest.mark.gpu

DENSE = {"kind": "dense", "ff": 50}
MOE = {"kind": "moe", "expert": {"ff": 16, "limit": 1.3}, "shared": {"ff": 28, "limit": 0.9},
       "router": {"experts": 6, "top": 3, "scale": 2.5, "groups": {"count": 3, "keep": 2}}}
MOE1 = {"kind": "moe", "expert": {"ff": 10, "limit": 0.8}, "shared": {"ff": 6, "limit": 2.0}, "router": {"experts": 4, "top": 1, "scale": 1.0}}
ATT = {"type": "attention", "mixer": {"heads": 6, "kv_heads": 2, "dim": 24, "vdim": 24, "scale": 0.3, "mask": {"size": 37}}, "mlp": DENSE}
GLA = {"type": "gla", "mixer": {"heads": 3, "dim": 10, "vdim": 14, "tau": 5.0}, "mlp": MOE1}
MLS = {"type": "mlstm", "mixer": {"heads": 2, "dim": 12, "vdim": 20, "gate_cap": 9.0}, "mlp": MOE}
PAIR = {"buckets": 23, "mul_prev": 5, "mul_cur": 3}
LOOP = {"start": 1, "stop": 3, "times": 2}


def make_cfg(layers, width=40, vocab=61, eps=1e-5, loop=None, pair=PAIR, positions=512):
    cfg = {"architecture": "Zenedra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "max_positions": positions,
           "layers": json.loads(json.dumps(layers))}
    if loop is not None:
        cfg["loop"] = dict(loop)
    if pair is not None:
        cfg["embedding"] = {"bigram": dict(pair)}
    return cfg


def weights_of(cfg, seed=0):
    """The weights an engine built on a directory without a checkpoint draws for `seed`."""
    from nano_vllm_x_amd.zenedra import ZenedraConfig, random_checkpoint
    return dict(random_checkpoint(ZenedraConfig.from_dict(cfg), seed))


def sharpen(w, by=3.0):
    """Peaked attention scores: one key too many or too few then moves the result far."""
    for name in w:
        if name.endswith("mix.q.norm"):
            w[name] = (w[name] * by).to(torch.bfloat16).float()
    return w


def near(got, want, rel, what=""):
    """Every value within `rel` of its own size (and of a fiftieth of the values' mean size: results near zero)."""
    got, want = got.double(), want.double()
    err = ((got - want).abs() / (want.abs() + 0.02 * want.abs().mean() + 1e-12)).max().item()
    assert err < rel, f"{what}: a value is off by {err:.3e} of its size (tolerance {rel})"


def forward(cfg, w, toks):
    return zo.forward(cfg, w, toks)


# ---- kernels alone -------------------------------------------------------------------------------------------------------
def _walk(full, cuts, slot, order, run):
    """Sequences `full` (id -> rows) cut into steps (`cuts`: id -> sizes), `order` naming the live ids of every step; run(x, lens,
    pos0, slots, decode) -> rows.  Returns id -> all rows."""
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


ORDER = [[0, 1]] * 4 + [[0]] * 10 + [[1]] * 5 + [[2, 1]] * 5 + [[2]] * 4


@pytest.mark.parametrize("fmt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,buckets,muls", [(70, 23, (5, 3)), (64, 7, (1000003, 77777)), (5, 2, (1, 1))])
def test_embedding_sum_over_cuts_and_reused_slots(fmt, width, buckets, muls):
    """Token row + pair row + position row: portions whose first token has its predecessor in the step before, a first token (which has the
    extra pair row, whatever the slot held), a slot that changes hands, a padding row of a captured step."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(width)
    vocab = 19
    table, pair, pos = (torch.randn(n, width, generator=g).to(fmt) for n in (vocab, buckets + 1, 200))
    full = {0: torch.randint(0, vocab, (90,), generator=g), 1: torch.randint(0, vocab, (17,), generator=g), 2: torch.randint(0, vocab, (9,), generator=g)}
    w = {"embed": table.double(), "bigram": pair.double(), "pos": pos.double()}
    cfg = {"embedding": {"bigram": {"buckets": buckets, "mul_prev": muls[0], "mul_cur": muls[1]}}}
    want = {i: zo.embedding(t.tolist(), w, cfg) for i, t in full.items()}
    prev = torch.full((3, 1), 7.0).cuda()
    cuts = {0: cuts_of(90, [1, 2, 9, 8, 1, 1, 90]), 1: cuts_of(17, [5, 1, 1, 2, 17]), 2: cuts_of(9, [2, 1, 6])}
    wn, eps = torch.randn(width, generator=g), 1e-3
    dev = [x.cuda() for x in (table, pair, pos)]
    rows = {"normed": [], "split": []}

    def run(x, lens, pos0, slots, decode):
        lay = step_layout(ops, lens, pos0, slots, decode)
        p = torch.cat([torch.arange(a, a + n) for a, n in zip(pos0, lens)]).cuda()
        kw = dict(pair=dev[1], mul_prev=muls[0], mul_cur=muls[1], pos_table=dev[2], positions=p)
        again = prev.clone()
        s, hl = ops.embed_sum(x.cuda(), dev[0], lay, prev_id=again, split=True, **kw)
        out, h = ops.embed_sum(x.cuda(), dev[0], lay, prev_id=prev, w=wn.cuda(), eps=eps, **kw)
        assert torch.equal(s, out) and torch.equal(again, prev) and h.dtype == hl.dtype == fmt
        close(h.float().cpu(), zo.rms(out.cpu().double(), eps) * wn.double(), 1e-5 if fmt == torch.float32 else 2e-2, "norm of the sum")
        assert torch.equal(hl[:, :width], out.to(fmt))
        assert (hl[:, :width].double() + hl[:, width:].double() - out.double()).abs().max() < 1e-4 * out.abs().max()
        return out.cpu()
    got = _walk(full, cuts, {0: 2, 1: 0, 2: 2}, ORDER, run)
    for i in full:
        close(got[i], want[i], 1e-6, f"sequence {i}")
    # a padding row (no slot) changes no slot; without the two tables only the token rows are left
    before = prev.clone()
    lay = ops.StepLayout(2, 2, torch.tensor([3, 0]).cuda(), torch.tensor([1, -1], dtype=torch.int32).cuda())
    ops.embed_sum(torch.tensor([4, 5]).cuda(), dev[0], lay, pair=dev[1], mul_prev=1, mul_cur=1, prev_id=prev)
    assert torch.equal(prev[[0, 2]], before[[0, 2]]) and not torch.equal(prev[1], before[1])
    x, h = ops.embed_sum(torch.tensor([4, 5]).cuda(), dev[0])
    assert h is None and torch.equal(x.cpu(), table[[4, 5]].float())


@pytest.mark.parametrize("fmt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [1, 33, 64, 300, 4100])
def test_sublayer_boundary(fmt, width):
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(width)
    t, eps = 5, 1e-3 if width > 1 else 1.0
    rnd = lambda *s: torch.randn(*s, generator=g)
    x, y, y2, add, bias, w = rnd(t, width), rnd(t, width).to(fmt), rnd(t, width).to(fmt), rnd(t, width), rnd(width), rnd(width)
    tol = 1e-4 if fmt == torch.float32 else 8e-3
    for use in ((), ("y",), ("y", "y2"), ("add", "bias"), ("y", "y2", "add", "bias"), ("bias",)):
        ops_in = {k: v.cuda() for k, v in (("y", y), ("y2", y2), ("add", add), ("bias", bias)) if k in use}
        want = x.double() + sum(v.double() for k, v in (("y", y), ("y2", y2), ("add", add), ("bias", bias)) if k in use)
        xd = x.cuda()
        h = ops.residual_norm(xd, w=w.cuda(), eps=eps, dtype=fmt, **ops_in)
        close(xd.cpu(), want, 1e-6, f"stream {use}")
        near(h.float().cpu(), zo.rms(want, eps) * w.double(), tol, f"norm {use}")
        xd, out = x.cuda(), torch.full((t, width), 7.0).cuda()
        hl = ops.residual_norm(xd, split=True, dtype=fmt, out=out, **ops_in)
        assert torch.equal(xd.cpu(), x) and hl.shape == (t, 2 * width) and hl.dtype == fmt
        close(out.cpu(), want, 1e-6, f"stream beside the old one {use}")
        close((hl[:, :width].double() + hl[:, width:].double()).cpu(), want, 1e-4, f"hi + lo {use}")
        assert ops.residual_norm(xd, dtype=fmt, **ops_in) is None
        close(xd.cpu(), want, 1e-6, f"stream alone {use}")


@pytest.mark.parametrize("fmt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,kv_heads,dim,at", [(6, 2, 24, 3), (3, 3, 7, 3), (4, 1, 96, 8), (2, 2, 1, 5), (6, 2, 24, 8), (5, 1, 64, 16), (2, 1, 200, 8), (3, 1, 512, 0)])
def test_queries_are_normed_and_raw_keys_stored_with_their_reciprocal_norm(fmt, heads, kv_heads, dim, at):
    """The parts are slices of a wider projection, at columns that fit 16-byte loads and at columns that do not."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(dim)
    t, eps = 6, 1e-2
    nq, nk = heads * dim, kv_heads * dim
    gap = 8 if at % 8 == 0 else 2
    x = torch.randn(t, at + nq + gap + nk, generator=g).to(fmt)
    qw, kw = torch.randn(dim, generator=g), torch.randn(dim, generator=g)
    slots = torch.tensor([4, 0, -1, 7, 2, 5], dtype=torch.int64)
    cache, rn = torch.full((8, nk), 9.0).to(fmt).cuda(), torch.full((8, kv_heads), 9.0).cuda()
    q = ops.tied_prep_store(x.cuda(), (at, at + nq + gap), qw.cuda(), kw.cuda(), eps, slots.cuda(), cache, rn, heads, kv_heads, dim)
    want_q = zo.rms(x[:, at:at + nq].double().view(t, heads, dim), eps) * qw.double() * kw.double()
    close(q.float().cpu(), want_q.reshape(t, nq), 1e-5 if fmt == torch.float32 else 4e-2, "queries")
    k = x[:, at + nq + gap:]
    keep = slots >= 0
    assert torch.equal(cache.cpu()[slots[keep]], k[keep])
    want_rn = 1.0 / torch.sqrt((k.double().view(t, kv_heads, dim) ** 2).mean(-1) + eps)
    close(rn.cpu()[slots[keep]], want_rn[keep], 1e-5, "reciprocal norms")
    assert (cache.cpu()[[1, 3, 6]] == 9.0).all() and (rn.cpu()[[1, 3, 6]] == 9.0).all()


def _tied_reference(q, k, rn, scale, slopes, chunk):
    """Per sequence: every head's read-out of raw keys under the scores of keys times their own number.  (T, heads * dim)."""
    heads, kvh = q.shape[1], k.shape[1]
    pos = torch.arange(q.shape[0])
    of = lambda h: h // (heads // kvh)
    return torch.cat([zo.chunk_softmax_readout(q[:, h].double(), k[:, of(h)].double() * rn[:, of(h), None].double(), k[:, of(h)].double(), pos, pos, scale,
                                               float(slopes[h]), chunk) for h in range(heads)], -1)


def _cached(keys, rns, n_slots, seed):
    perm = torch.randperm(n_slots, generator=torch.Generator().manual_seed(seed)).tolist()
    g, d = keys[0].shape[1], keys[0].shape[2]
    kc, rc = torch.zeros(n_slots, g * d), torch.zeros(n_slots, g)
    lists = []
    for k, r in zip(keys, rns):
        s = [perm.pop() for _ in range(k.shape[0])]
        kc[s], rc[s] = k.reshape(len(s), -1), r
        lists.append(s)
    return kc, rc, lists


def _attend(ops, q_rows, lens, totals, lists, kc, vc, rc, fmt, decode, **kw):
    """ops.softcap_attn for a step that brings the last lens[b] tokens of the first totals[b] of sequence b."""
    flat = torch.tensor([s for b, l in enumerate(lists) for s in l[:totals[b]]], dtype=torch.int32).cuda()
    start = torch.tensor(np.concatenate([[0], np.cumsum(totals)[:-1]]), dtype=torch.int64).cuda()
    kv_len = torch.tensor(totals, dtype=torch.int32).cuda()
    lay = step_layout(ops, lens, [n - l for n, l in zip(totals, lens)], list(range(len(lens))), decode)
    return ops.softcap_attn(q_rows.to(fmt).cuda(), kc, vc, flat, start, kv_len, lay, cap=0.0, k_rn=rc, **kw).float().cpu()


@pytest.mark.parametrize("heads,kvh,dim", [(6, 2, 24), (4, 1, 64), (5, 5, 7), (3, 1, 200), (2, 1, 300)])
@pytest.mark.parametrize("chunk,loud", [(0, 0), (50, 50), (64, 63), (1, 0), (1000, 0), (13, 26)])
def test_attention_over_tied_rows_in_chunks(heads, kvh, dim, chunk, loud):
    """Two sequences of unequal length at scattered slots; every query asks loudly for key `loud`, the first key of a chunk or the last of
    the one before, so a chunk that is one key off shows; gentle slopes, so far keys count; portions and single tokens that end
    just inside and just outside a chunk, with and without the key split; the kernel that reads a row once and (through a copy of the
    cache as values) the general one."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(dim + chunk)
    scale = 0.3
    n = [200, 77]
    slopes = torch.tensor([0.02 * 2.0 ** -h for h in range(heads)])
    q = [torch.randn(t, heads, dim, generator=g) for t in n]
    k = [torch.randn(t, kvh, dim, generator=g) for t in n]
    rn = [torch.rand(t, kvh, generator=g) + 0.5 for t in n]
    for b in range(2):
        for h in range(heads):
            k0 = k[b][loud, h // (heads // kvh)]
            q[b][:, h] = q[b][:, h] * 0.3 + 24.0 * k0 / k0.norm() ** 2
    want = [_tied_reference(q[b], k[b], rn[b], scale, slopes, chunk or None) for b in range(2)]
    kc, rc, lists = _cached(k, rn, 300, 3)
    kc, rc = kc.cuda(), rc.cuda()
    kw = dict(scale=scale, heads=heads, kv_heads=kvh, dim=dim, vdim=dim, slopes=slopes.cuda(), chunk=chunk)
    for lens, totals, decode in (([200, 77], [200, 77], False), ([3, 30], [103, 77], False), ([1, 1], [51, 50], True), ([1, 1], [200, 2], True),
                                 ([2, 1], [65, 2], False), ([1, 1], [1, 64], True), ([14, 13], [64, 26], False)):
        rows = torch.cat([q[b][totals[b] - lens[b]:totals[b]].reshape(lens[b], -1) for b in range(2)])
        ref = torch.cat([want[b][totals[b] - lens[b]:totals[b]] for b in range(2)])
        for split in (1, 4):
            for vc in (kc, kc.clone()):
                got = _attend(ops, rows, lens, totals, lists, kc, vc, rc, torch.float32, decode, n_split=split, **kw)
                close(got, ref, 1e-4, f"lens {lens} of {totals}, split {split}")
    if chunk > 1 and chunk < 200:      # the restatement itself depends on where the chunks begin
        other = _tied_reference(q[0], k[0], rn[0], scale, slopes, chunk + 1)
        assert (other - want[0]).abs().max() > 0.2


@pytest.mark.parametrize("dim", [64, 96, 128])
@pytest.mark.parametrize("chunk,loud", [(0, 0), (100, 100), (100, 99), (33, 66), (64, 128)])
def test_tied_rows_in_chunks_on_the_matrix_cores(dim, chunk, loud):
    """Steps of many tokens in bfloat16 take the tile kernel: ragged prompts that end in the middle of a key tile, portions that start in
    the middle of a chunk, chunks that begin inside a tile and inside a block of queries; against the restatement on the same bfloat16
    values, and the kernels for few tokens beside it."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(dim)
    heads, kvh, scale = 4, 2, 0.2
    n = [200, 77, 300, 1]
    bf = lambda x: x.to(torch.bfloat16).float()
    slopes = torch.tensor([0.03, 0.01, 0.003, 0.2])
    q = [bf(torch.randn(t, heads, dim, generator=g) * 0.3) for t in n]
    k = [bf(torch.randn(t, kvh, dim, generator=g)) for t in n]
    rn = [torch.rand(t, kvh, generator=g) + 0.5 for t in n]
    for b in (0, 2):
        for h in range(heads):
            k0 = k[b][loud, h // (heads // kvh)]
            q[b][:, h] = bf(q[b][:, h] * 0.3 + 36.0 * k0 / k0.norm() ** 2)
    want = [_tied_reference(q[b], k[b], rn[b], scale, slopes, chunk or None) for b in range(len(n))]
    kc, rc, lists = _cached(k, rn, 700, 5)
    kc, rc = kc.to(torch.bfloat16).cuda(), rc.cuda()
    kw = dict(scale=scale, heads=heads, kv_heads=kvh, dim=dim, vdim=dim, slopes=slopes.cuda(), chunk=chunk, n_split=1)
    for lens, totals in ((n, n), ([70, 3, 130, 1], [200, 77, 300, 1]), ([129, 77, 1, 1], [130, 77, 65, 1])):
        rows = torch.cat([q[b][totals[b] - lens[b]:totals[b]].reshape(lens[b], -1) for b in range(len(n))])
        ref = torch.cat([want[b][totals[b] - lens[b]:totals[b]] for b in range(len(n))])
        for cores, vc, what in ((True, kc, "matrix cores"), (False, kc, "a row read once"), (False, kc.clone(), "vector units")):
            got = _attend(ops, rows, lens, totals, lists, kc, vc, rc, torch.bfloat16, False, matrix_cores=cores, **kw)
            err = ((got.double() - ref).abs() / (ref.abs() + 0.05 * ref.std())).max().item()
            assert err < 8e-3, f"{what}, lens {lens} of {totals}: {err:.2e}"


@pytest.mark.parametrize("power", [1.0, 0.0625, 0.3])
def test_decays_of_the_channels(power):
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(4)
    for t, n_out, k_in in ((9, 30, 5), (3, 70, 300), (1, 7, 16)):
        x, w, b = torch.randn(t, k_in, generator=g), torch.randn(n_out, k_in, generator=g), torch.randn(n_out, generator=g) * 20.0
        got = ops.skinny_proj(x.cuda(), w.cuda(), bias=b.cuda(), out_act="sigmoid_pow", power=power).cpu()
        want = zo.channel_decay(x.double() @ w.double().T + b.double(), 1.0 / power)
        assert torch.allclose(got.double(), want, atol=1e-6, rtol=2e-5)
        assert torch.allclose(ops.skinny_proj(x.cuda(), w.cuda(), bias=b.cuda()).cpu().double(), x.double() @ w.double().T + b.double(), atol=1e-4)


LONG_ORDER = [[0, 1]] * 4 + [[0]] * 6 + [[1]] * 5 + [[2, 1]] * 5 + [[2]] * 4
LONG_CUTS = {0: [1, 2, 9, 8, 1, 1, 280, 1, 1, 300], 1: [5, 1, 1, 2, 8], 2: [2, 1, 6]}


@pytest.mark.parametrize("chunk", [None, 0, 5, 64])
@pytest.mark.parametrize("heads,dim,vdim", [(2, 40, 70), (1, 3, 5), (3, 128, 33), (1, 300, 20), (2, 32, 300)])
def test_channel_decay_memory_over_cuts_and_reused_slots(chunk, heads, dim, vdim):
    """Slots that are not in order, steps of 1, 2 and hundreds of tokens (those of 256 and more in chunks side by side unless `chunk` says
    otherwise), a sequence that takes over a used slot.  Channels whose decay is close to one keep the first token for hundreds of
    steps, others forget at once."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(dim)
    hd, he = heads * dim, heads * vdim
    n = {0: 604, 1: 17, 2: 9}
    full = {i: torch.randn(t, 2 * hd + he + 3 + hd, generator=g) for i, t in n.items()}
    for x in full.values():
        x[:, -hd:] = torch.sigmoid(x[:, -hd:] * 4.0 + 4.0) ** 0.1
        x[:, -hd] = 0.9999                          # the first channel remembers
        if dim > 2:
            x[:, -hd + 1] = 1e-30                    # the second one forgets (products of decays underflow to zero)

    def ref(x):
        x = x.double()
        q, k, v = x[:, 3:3 + hd].view(-1, heads, dim), x[:, 3 + hd:3 + 2 * hd].view(-1, heads, dim), x[:, 3 + 2 * hd:3 + 2 * hd + he].view(-1, heads, vdim)
        a = x[:, -hd:].view(-1, heads, dim)
        return [zo.channel_decay_memory(q[:, h] * 0.25, k[:, h], v[:, h], a[:, h]) for h in range(heads)]
    want = {i: torch.cat([o for o, _ in ref(x)], 1) for i, x in full.items()}
    mem = torch.full((3, heads, dim, vdim), 7.0).cuda()

    def run(x, lens, pos0, slots, decode):
        x = x.cuda()
        o = ops.gla_scan(x, (3, 3 + hd, 3 + 2 * hd), x[:, -hd:].contiguous(), mem, step_layout(ops, lens, pos0, slots, decode), heads, dim, vdim, q_mul=0.25,
                         chunk=chunk)
        return o.reshape(len(x), he).cpu()
    got = _walk(full, {i: list(c) for i, c in LONG_CUTS.items()}, {0: 2, 1: 0, 2: 2}, LONG_ORDER, run)
    for i in full:
        close(got[i], want[i], 1e-4, f"sequence {i}")
    close(mem[2].cpu(), torch.stack([s for _, s in ref(full[2])]), 1e-4, "memory of the last sequence in slot 2")


@pytest.mark.parametrize("chunk", [None, 0, 5, 64])
@pytest.mark.parametrize("heads,dim,vdim", [(2, 40, 70), (1, 3, 5), (1, 300, 20), (2, 32, 300)])
def test_exponentially_gated_memory_in_chunks(chunk, heads, dim, vdim):
    """The same for the matrix memory with a running maximum: input gates that jump by twenty and more, so that the maximum moves in the
    middle of a chunk and long after one."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(dim + 1)
    hd, he, cap = heads * dim, heads * vdim, 15.0
    n = {0: 604, 1: 17, 2: 9}
    full = {i: torch.randn(t, 2 * hd + he + 2 * heads, generator=g) for i, t in n.items()}
    for x in full.values():
        x[:, -2 * heads:-heads] *= 3.0
        x[::41, -2 * heads:-heads] += 25.0
        x[:, -heads:] = x[:, -heads:] * 2.0 + 4.0
    bias = torch.randn(2 * heads, generator=g) * 0.3

    def ref(x):
        x = x.double()
        q, k, v = x[:, :hd].view(-1, heads, dim), x[:, hd:2 * hd].view(-1, heads, dim), x[:, 2 * hd:2 * hd + he].view(-1, heads, vdim)
        i = cap * torch.tanh((x[:, -2 * heads:-heads] + bias[:heads].double()) / cap)
        f = torch.nn.functional.logsigmoid(cap * torch.tanh((x[:, -heads:] + bias[heads:].double()) / cap))
        return [zo.exp_gated_memory(q[:, h] * dim ** -0.5, k[:, h], v[:, h], i[:, h], f[:, h]) for h in range(heads)]
    refs = {i: ref(x) for i, x in full.items()}
    mem, nrm, peak = torch.full((3, heads, dim, vdim), 7.0).cuda(), torch.full((3, heads, dim), 7.0).cuda(), torch.full((3, heads), 7.0).cuda()

    def run(x, lens, pos0, slots, decode):
        x = x.cuda()
        o = ops.mlstm_scan(x, (0, hd, 2 * hd), x[:, -2 * heads:].contiguous(), bias.cuda(), cap, mem, nrm, peak, step_layout(ops, lens, pos0, slots, decode),
                           heads, dim, vdim, chunk=chunk)
        return o.reshape(len(x), he).cpu()
    got = _walk(full, {i: list(c) for i, c in LONG_CUTS.items()}, {0: 2, 1: 0, 2: 2}, LONG_ORDER, run)
    for i in full:
        want = torch.cat([o for o, _ in refs[i]], 1)
        err = ((got[i].double() - want).abs() / (want.abs() + want.std())).max().item()
        assert err < 1e-3, f"sequence {i}: {err:.2e}"
    for h in range(heads):
        s, nn, m = refs[2][h][1]
        assert abs(peak[2, h].item() - m) < 1e-4
        close(mem[2, h].cpu(), s, 1e-4, "memory in slot 2")
        assert torch.allclose(nrm[2, h].cpu().double(), nn, atol=1e-4 * (nn.abs().max().item() + 1e-3))


@pytest.mark.parametrize("experts,top,groups,keep", [(6, 3, 3, 2), (20, 5, 4, 3), (4, 1, 0, 0), (8, 3, 4, 4), (12, 6, 2, 1), (5, 5, 0, 0), (9, 2, 9, 2), (200, 7, 100, 9),
                                                     (64, 64, 2, 2), (130, 3, 0, 0)])
def test_sigmoid_router_with_groups_and_a_correction(experts, top, groups, keep):
    """Corrections large enough to make choice scores negative (an excluded group must not win with zero) and to choose other experts than
    the scores alone would; the weights ignore them."""
    from nano_vllm_x_amd import ops
    g = torch.Generator().manual_seed(experts)
    z, corr = torch.randn(150, experts, generator=g) * 2.0, torch.randn(experts, generator=g) * 0.4 - 1.2
    router = {"experts": experts, "top": top, "scale": 2.5, "groups": {"count": groups, "keep": keep} if groups else None}
    got_i, got_w = ops.moe_route_sigmoid(z.cuda(), corr.cuda(), top, groups, keep, 2.5)
    got_i, got_w = got_i.cpu().tolist(), got_w.cpu().double()
    differs = [0, 0, 0]
    for t in range(150):
        ids, wts = zo.route_logits(z[t].tolist(), corr.tolist(), router)
        assert sorted(got_i[t]) == sorted(ids), t
        by_id = dict(zip(ids, wts))
        assert all(abs(got_w[t, k].item() - by_id[e]) < 1e-6 for k, e in enumerate(got_i[t]))
        differs[0] += sorted(zo.route_logits(z[t].tolist(), [0.0] * experts, router)[0]) != sorted(ids)
        differs[1] += sorted(zo.route_logits(z[t].tolist(), corr.tolist(), {**router, "groups": None})[0]) != sorted(ids)
    if top < experts:
        assert differs[0] > 0, "the correction moves no choice"
    if groups and keep < min(top, groups):
        assert differs[1] > 0, "the groups move no choice"


@pytest.mark.parametrize("fmt", [torch.float32, torch.bfloat16, torch.float16])
@pytest.mark.parametrize("rows,ff", [(37, 64), (5, 12), (1, 8), (300, 1536), (3, 7)])
def test_gelu_gate(fmt, rows, ff):
    from nano_vllm_x_amd import ops
    gu = (torch.randn(rows, 2 * ff, generator=torch.Generator().manual_seed(rows + ff)) * 2.0).to(fmt)
    got = ops.gelu_glu(gu.cuda())
    assert got.dtype == fmt and got.shape == (rows, ff)
    near(got.float().cpu(), zo.gelu_tanh(gu[:, :ff].double()) * gu[:, ff:].double(), 1e-4 if fmt == torch.float32 else 5e-3 if fmt == torch.bfloat16 else 1e-3)


@pytest.mark.parametrize("experts,top,groups,keep,shared", [(6, 3, 3, 2, 30), (3, 3, 0, 0, None), (4, 1, 2, 1, 24), (70, 4, 10, 3, 8)])
def test_experts_by_rows_and_by_expert_order_beside_a_shared_one(experts, top, groups, keep, shared):
    from nano_vllm_x_amd.layers.moe import DenseGLU, GroupedSigmoidMoE
    g = torch.Generator().manual_seed(top)
    width, ff, t, limit = 40, 24, 50, 0.9
    p = {f"e{j}.{s}": torch.randn((ff, width) if s != "down" else (width, ff), generator=g) * 0.3 for j in range(experts) for s in ("gate", "up", "down")}
    p["router"], p["correction"] = torch.randn(experts, width, generator=g) * 0.5, torch.randn(experts, generator=g)
    for s in ("gate", "up", "down") if shared else ():
        p["shared." + s] = torch.randn((shared, width) if s != "down" else (width, shared), generator=g) * 0.3
    moe = GroupedSigmoidMoE(width, experts, top, ff, limit, 1.702, 1.0, groups=groups or None, keep=keep or None, scale=1.7,
                            shared=DenseGLU(width, shared, 2.1, 1.702) if shared else None).float().cuda()
    with torch.no_grad():
        for j in range(experts):
            moe.w_gu[j, :ff], moe.w_gu[j, ff:], moe.w_d[j] = p[f"e{j}.gate"].cuda(), p[f"e{j}.up"].cuda(), p[f"e{j}.down"].cuda()
        moe.router.copy_(p["router"])
        moe.correction.copy_(p["correction"])
        if shared:
            moe.shared.gu_proj.weight.copy_(torch.cat([p["shared.gate"], p["shared.up"]]))
            moe.shared.down.weight.copy_(p["shared.down"])
    h = torch.randn(t, width, generator=g)
    mlp = {"expert": {"ff": ff, "limit": limit}, "shared": {"ff": shared, "limit": 2.1} if shared else None,
           "router": {"experts": experts, "top": top, "scale": 1.7, "groups": {"count": groups, "keep": keep} if groups else None}}
    want = zo.moe_ff(h.double(), {k: v.double() for k, v in p.items()}, "", mlp)
    total = lambda r: (r[0] if r[1] is None else r[0] + r[1]).cpu()
    with torch.inference_mode():
        close(total(moe(h.cuda(), decode_step=False)), want, 1e-4, "expert order")
        close(total(moe(h.cuda(), decode_step=True)), want, 1e-4, "rows")
        close(total(moe(h[:3].cuda())), want[:3], 1e-4, "few tokens")


# ---- one mechanism at a time ---------------------------------------------------------------------------------------------
def _att(mlp=None, **changes):
    return {"type": "attention", "mixer": dict(ATT["mixer"], **changes), "mlp": mlp}


def _no_mask(layer):
    m = dict(layer["mixer"])
    m.pop("mask")
    return {**layer, "mixer": m}


BARE = dict(GLA, mlp=None)
ONE = {
    "attention in chunks": ([_att()], {}),
    "attention, all keys": ([_no_mask(_att())], {}),
    "attention, chunks of one position": ([_att(mask={"size": 1})], {}),
    "attention, chunks of a page": ([_att(mask={"size": 64})], {}),
    "attention, one head, a size of nothing": ([_att(heads=1, kv_heads=1, dim=3, vdim=3, scale=0.9)], {}),
    "attention, five heads on one key": ([_att(DENSE, heads=5, kv_heads=1, dim=16, vdim=16)], {}),
    "gated linear attention": ([BARE], {}),
    "gated linear attention, tau of one, wide inner decay": ([dict(GLA, mlp=None, mixer=dict(GLA["mixer"], tau=1.0, decay_rank=33, vdim=3))], {}),
    "matrix memory": ([dict(MLS, mlp=None)], {}),
    "matrix memory, one head, a low cap": ([{"type": "mlstm", "mixer": {"heads": 1, "dim": 5, "vdim": 5, "gate_cap": 0.7}, "mlp": None}], {}),
    "dense feed-forward": ([dict(BARE, mlp=DENSE)], {}),
    "experts in groups beside a shared one": ([dict(BARE, mlp=MOE)], {}),
    "experts, all of all, no shared one": ([dict(BARE, mlp={"kind": "moe", "expert": {"ff": 8, "limit": 0.5}, "router": {"experts": 3, "top": 3}})], {}),
    "experts, groups of one": ([dict(BARE, mlp={"kind": "moe", "expert": {"ff": 8, "limit": 3.0}, "shared": {"ff": 5, "limit": 0.2},
                                               "router": {"experts": 5, "top": 2, "scale": 0.5, "groups": {"count": 5, "keep": 3}}})], {}),
    "no pair table": ([BARE], {"pair": None}),
    "a pair table of one bucket": ([BARE], {"pair": {"buckets": 1, "mul_prev": 9, "mul_cur": 4}}),
    "a pass from the first layer to the last": ([ATT, MLS], {"loop": {"start": 0, "stop": 2, "times": 3}}),
    "one layer three times": ([GLA, ATT, MLS], {"loop": {"start": 1, "stop": 2, "times": 3}}),
    "one pass": ([GLA, MLS], {"loop": {"start": 1, "stop": 2, "times": 1}}),
    "the last layers twice": ([GLA, MLS, ATT], {"loop": LOOP}),
    "the first layers four times": ([GLA, ATT, MLS], {"loop": {"start": 0, "stop": 2, "times": 4}}),
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
    close(replay(eng, {"c": toks}, [[("c", 1)]] * 80)["c"], want, F32_TOL, "token by token")
    eng.shutdown()


def test_residual_after_every_layer_run(tmp_path):
    """The stream after each run of a layer (every pass counts), as the model can record it, against the restatement's."""
    cfg = make_cfg([ATT, GLA, MLS, dict(ATT, mlp=MOE)], loop=LOOP)
    w = weights_of(cfg, 5)
    eng = make_engine(model_dir(tmp_path, cfg, w), pool=128)
    toks = tokens(23, cfg["vocab"], 1)
    streams = []
    zo.forward(cfg, w, toks, streams)
    model = eng.model_runner.model
    model.layer_streams = []
    replay(eng, {"a": toks}, [[("a", 23)]])
    got, model.layer_streams = model.layer_streams, None
    assert len(got) == len(streams) == 6
    for i, (a, b) in enumerate(zip(got, streams)):
        close(a.float().cpu(), b, 5e-5, f"after layer run {i}")
    eng.shutdown()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sizes_that_fit_no_vector_width(tmp_path, dtype):
    """A width, head sizes, feed-forward sizes and a vocabulary that are multiples of nothing useful (no 16-byte rows anywhere), three
    query heads on one key/value head, experts in the first layer and none in the last."""
    odd = [{"type": "attention", "mixer": {"heads": 3, "kv_heads": 1, "dim": 10, "vdim": 10, "scale": 0.3, "mask": {"size": 21}},
            "mlp": {"kind": "moe", "expert": {"ff": 9, "limit": 1.1}, "shared": {"ff": 5, "limit": 0.6},
                    "router": {"experts": 9, "top": 3, "scale": 1.9, "groups": {"count": 3, "keep": 1}}}},
           {"type": "gla", "mixer": {"heads": 5, "dim": 3, "vdim": 7, "tau": 3.0, "decay_rank": 3}, "mlp": {"kind": "dense", "ff": 11}},
           {"type": "mlstm", "mixer": {"heads": 3, "dim": 5, "vdim": 9, "gate_cap": 4.0}, "mlp": None}]
    cfg = make_cfg(odd, width=49, vocab=37, loop={"start": 0, "stop": 2, "times": 2}, pair={"buckets": 101, "mul_prev": 53, "mul_cur": 1}, positions=77)
    w = weights_of(cfg, 4)
    eng = make_engine(model_dir(tmp_path, cfg, w), dtype=dtype, pool=256)
    toks = tokens(45, 37, 8)
    want = forward(cfg, w, toks)
    got = replay(eng, {"a": toks}, [[("a", 33)], [("a", 2)]] + [[("a", 1)]] * 10)["a"]
    if dtype == "float32":
        close(got, want, F32_TOL, "float32")
        close(replay(eng, {"b": toks}, [[("b", 45)]])["b"], want, F32_TOL, "whole")
    else:
        err = (got.double() - want).abs().amax(dim=1) / want.std()
        assert err.median() < 0.08 and err.max() < 0.4, (err.median().item(), err.max().item())
    eng.shutdown()


def test_first_tokens_page_borders_and_chunk_edges_in_prompts_and_decoding(tmp_path):
    """Prompts of 1, 2, 63, 64, 65, 128, 129 tokens; pages of 64, key tiles and chunks of 50 crossed token by token and by portions that
    start, end and turn at them; sharpened scores."""
    cfg = make_cfg([_att(DENSE, mask={"size": 50}), GLA, _att(MOE, mask={"size": 64}), MLS], loop={"start": 0, "stop": 3, "times": 2})
    w = sharpen(weights_of(cfg, 12))
    eng = make_engine(model_dir(tmp_path, cfg, w), pool=1024)
    toks = tokens(200, cfg["vocab"], 6)
    want = forward(cfg, w, toks)
    for n in (1, 2, 3, 49, 50, 51, 63, 64, 65, 128, 129):
        close(replay(eng, {f"p{n}": toks[:n]}, [[(f"p{n}", n)]])[f"p{n}"], want[:n], F32_TOL, f"prompt of {n}")
    sched = [[("a", 1)]] * 3 + [[("a", 45)]] + [[("a", 1)]] * 5 + [[("a", 2)], [("a", 8)], [("a", 2)], [("a", 32)]] + [[("a", 1)]] * 9 + \
            [[("a", 40)]] + [[("a", 1)]] * 6 + [[("a", 48)]]
    assert sum(n for step in sched for _, n in step) == 200
    close(replay(eng, {"a": toks}, sched)["a"], want, F32_TOL, "edges crossed token by token")
    # the chunks count: the same model with chunks one longer is another function
    other = json.loads(json.dumps(cfg))
    other["layers"][0]["mixer"]["mask"]["size"] = 51
    moved = (forward(other, w, toks) - want).abs().amax(dim=1)
    assert moved[:50].max() == 0 and moved[50] > 8 * F32_TOL * want.std()
    eng.shutdown()


def drawn_configuration(rnd):
    """A configuration drawn at random: 2 to 6 layers of any kind in any order, a run of them repeated or not, sizes from small and odd to
    those the matrix-core kernels take, any feed-forward or none."""
    def mlp():
        kind = rnd.choice(["dense", "moe", "moe", None])
        if kind is None:
            return None
        if kind == "dense":
            return {"kind": "dense", "ff": rnd.choice([24, 50, 128])}
        count, per = rnd.choice([1, 2, 4]), rnd.choice([1, 2, 3])
        keep = rnd.randint(1, count)
        router = {"experts": count * per, "top": rnd.randint(1, min(keep * per, 4)), "scale": rnd.choice([1.0, 2.5])}
        if rnd.random() < 0.8:
            router["groups"] = {"count": count, "keep": keep}
        out = {"kind": "moe", "expert": {"ff": rnd.choice([8, 20, 32]), "limit": rnd.choice([0.7, 2.0, 9.0])}, "router": router}
        if rnd.random() < 0.8:
            out["shared"] = {"ff": rnd.choice([7, 40]), "limit": rnd.choice([0.5, 1.0, 6.0])}
        return out

    layers = []
    for _ in range(rnd.randint(2, 6)):
        kind = rnd.choice(["attention", "gla", "mlstm"])
        if kind == "attention":
            kvh, dim = rnd.choice([1, 2, 3]), rnd.choice([6, 16, 64, 40, 96])
            m = {"heads": kvh * rnd.choice([1, 2, 4]), "kv_heads": kvh, "dim": dim, "vdim": dim, "scale": dim ** -0.5 * rnd.choice([1.0, 2.0])}
            if rnd.random() < 0.8:
                m["mask"] = {"size": rnd.choice([3, 17, 64, 100])}
        elif kind == "gla":
            m = {"heads": rnd.choice([1, 2, 5]), "dim": rnd.choice([4, 16, 40]), "vdim": rnd.choice([6, 32, 80]), "tau": rnd.choice([1.0, 4.0, 16.0]),
                 "decay_rank": rnd.choice([1, 8, 20])}
        else:
            m = {"heads": rnd.choice([1, 2, 5]), "dim": rnd.choice([4, 16, 40]), "vdim": rnd.choice([6, 32, 80]), "gate_cap": rnd.choice([2.0, 15.0])}
        layers.append({"type": kind, "mixer": m, "mlp": mlp()})
    loop = None
    if rnd.random() < 0.8:
        start = rnd.randint(0, len(layers) - 1)
        loop = {"start": start, "stop": rnd.randint(start + 1, len(layers)), "times": rnd.choice([1, 2, 3])}
    return make_cfg(layers, width=rnd.choice([24, 50, 96, 160]), vocab=rnd.choice([37, 130, 301]), eps=rnd.choice([1e-5, 1e-6]), loop=loop,
                    pair=rnd.choice([None, PAIR, {"buckets": 1000, "mul_prev": 77, "mul_cur": 13}]), positions=rnd.choice([200, 333]))


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
STACK = [ATT, MLS, GLA, dict(ATT, mlp=MOE)]


def test_batches_of_unequal_requests_in_a_small_pool(tmp_path):
    """Four live requests at most in a pool smaller than the sum of all: portions beside single tokens, a request that
    pauses for some steps, token slots and state slots that change hands (six requests, four state slots)."""
    cfg = make_cfg(STACK, loop=LOOP)
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


def test_far_tokens_and_old_state_count(tmp_path):
    """330 tokens, the first of them still seen at the end: through attention layers without chunks (gentle slopes of many heads, one of
    which asks for the first key), through channels that decay slowly and through the matrix memory."""
    layers = [_no_mask(_att(DENSE, heads=8, kv_heads=2)), dict(GLA, mixer=dict(GLA["mixer"], tau=64.0)), MLS]
    cfg = make_cfg(layers, loop=LOOP)
    w = sharpen(weights_of(cfg, 7), 2.0)
    w["l2.mix.f.b"] = (w["l2.mix.f.b"] + 4.0).to(torch.bfloat16).float()
    eng = make_engine(model_dir(tmp_path, cfg, w), pool=512)
    toks = tokens(330, cfg["vocab"], 2)
    want = forward(cfg, w, toks)
    got = replay(eng, {"a": toks}, [[("a", 255)], [("a", 1)], [("a", 1)], [("a", 2)], [("a", 30)]] + [[("a", 1)]] * 41)["a"]
    close(got, want, F32_TOL, "far tokens")
    close(replay(eng, {"b": toks}, [[("b", 330)]])["b"], want, F32_TOL, "whole, the recurrences in chunks side by side")
    other = forward(cfg, w, [(toks[0] + 1) % 61] + toks[1:])
    assert (other[-1] - want[-1]).abs().max() > 8 * F32_TOL * want.std()
    eng.shutdown()


def test_bfloat16_stays_within_rounding(tmp_path):
    """Dense feed-forwards: a router's close call may go either way in 16 bits, which says nothing about the kernels."""
    cfg = make_cfg([dict(layer, mlp=DENSE) for layer in STACK], loop=LOOP)
    toks = tokens(90, cfg["vocab"], 4)
    want = forward(cfg, weights_of(cfg, 2), toks)
    eng = make_engine(model_dir(tmp_path, cfg), dtype="bfloat16", seed=2)
    got = replay(eng, {"a": toks}, [[("a", 50)], [("a", 2)]] + [[("a", 1)]] * 38)["a"]
    err = (got.double() - want).abs().amax(dim=1) / want.std()
    assert err.median() < 0.08 and err.max() < 0.5, (err.median().item(), err.max().item())
    eng.shutdown()


def test_bfloat16_with_heads_for_the_matrix_cores(tmp_path):
    """Head sizes the tile kernel is built for, prompts long enough to take it, in bfloat16: whole prompts against portions and single
    tokens, and both against the restatement within rounding."""
    att = {"type": "attention", "mixer": {"heads": 8, "kv_heads": 4, "dim": 64, "vdim": 64, "scale": 0.125, "mask": {"size": 150}}, "mlp": DENSE}
    gla = {"type": "gla", "mixer": {"heads": 2, "dim": 64, "vdim": 96, "tau": 16.0}, "mlp": None}
    mls = {"type": "mlstm", "mixer": {"heads": 4, "dim": 48, "vdim": 64, "gate_cap": 15.0}, "mlp": DENSE}
    cfg = make_cfg([att, mls, gla], width=128, vocab=97, loop={"start": 0, "stop": 2, "times": 2})
    w = weights_of(cfg, 3)
    eng = make_engine(model_dir(tmp_path, cfg, w), dtype="bfloat16", pool=1024)
    toks = tokens(400, 97, 9)
    want = forward(cfg, w, toks)
    whole = replay(eng, {"a": toks}, [[("a", 400)]])["a"]
    cut = replay(eng, {"b": toks}, [[("b", 230)], [("b", 100)], [("b", 2)], [("b", 63)]] + [[("b", 1)]] * 5)["b"]
    for got, what in ((whole, "whole"), (cut, "cut")):
        err = (got.double() - want).abs().amax(dim=1) / want.std()
        assert err.median() < 0.08 and err.max() < 0.5, (what, err.median().item(), err.max().item())
    eng.shutdown()


def test_checkpoint_with_a_missing_or_misshapen_tensor_is_refused(tmp_path):
    cfg = make_cfg(STACK, loop=LOOP)
    w = weights_of(cfg, 0)
    for gone in ("l0.mix.k.b", "l1.mlp.correction", "l1.mlp.shared.down", "l2.mix.a2", "loop.step", "bigram", "l3.mix.k.norm"):
        bad = dict(w)
        del bad[gone]
        with pytest.raises(KeyError):
            make_engine(model_dir(tmp_path, cfg, bad, name="missing_" + gone.replace(".", "_")))
    for k, (name, shape) in enumerate((("bigram", (23, 40)), ("loop.in", (40, 40)), ("l2.mix.a1", (16, 41)), ("pos", (511, 40)))):
        bad = dict(w)
        bad[name] = torch.zeros(*shape)
        with pytest.raises(ValueError):
            make_engine(model_dir(tmp_path, cfg, bad, name=f"shape{k}"))
    bad = dict(w)
    bad["l2.mix.a1"] = torch.zeros(7, 40)          # fits the model, but not its second half
    with pytest.raises(ValueError):
        make_engine(model_dir(tmp_path, cfg, bad, name="rank"))


# ---- generation: the scheduler's own choices ---------------------------------------------------------------------------
def oracle_greedy(w, cfg, prompt, n_new):
    return greedy(lambda t: forward(cfg, w, t), prompt, n_new)


@pytest.mark.parametrize("chunked", [False, True], ids=["whole prompts", "chunked prefill"])
def test_greedy_generation_through_the_engine(tmp_path, chunked):
    """Prompts of unequal length admitted together, decoded as one batch; more requests than state slots, so the later ones wait
    for a slot that an earlier one gives back; with chunked prefill the prompts are computed in portions of seven tokens.  Long
    decoding (70 tokens, across a page of 64 and two chunks) for one of them."""
    from nano_vllm_x_amd.core.common import SamplingParams
    cfg = make_cfg(STACK, loop=LOOP)
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
    cfg = make_cfg(STACK, loop=LOOP)
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
    cfg = make_cfg(STACK, vocab=300, loop=LOOP)
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


def test_no_sequence_runs_past_the_table_of_positions(tmp_path):
    """A request without a length of its own ends where the learned positions do; given input beyond them is refused."""
    from nano_vllm_x_amd.core.common import SamplingParams
    cfg = make_cfg([GLA, ATT], positions=30)
    eng = make_engine(model_dir(tmp_path, cfg), pool=256, max_bs=2, seed=8)
    assert eng.context_len == 30
    prompt = tokens(21, cfg["vocab"], 1)
    eng.add_sequence("a", list(prompt), SamplingParams(temperature=0.0, ignore_eos=True))
    out = []
    while eng.has_unfinished_sequences():
        out += [o.new_token_id for o in eng.step()]
    assert out == oracle_greedy(weights_of(cfg, 8), cfg, prompt, 9)
    eng.add_sequence("b", list(prompt), SamplingParams(ignore_eos=True))
    with pytest.raises(ValueError):
        eng.extend_sequence("b", [1] * 10)
    eng.shutdown()


def test_preempted_sequence_starts_again_from_an_empty_state(tmp_path):
    from nano_vllm_x_amd.core.common import SamplingParams
    cfg = make_cfg(STACK, loop=LOOP)
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
    cfg = make_cfg(STACK, vocab=90, loop=LOOP)
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
    cfg = make_cfg(STACK, vocab=80, loop=LOOP)
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
