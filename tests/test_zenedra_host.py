"""Host side of the Zenedra family, without a device: configuration, registry, checkpoint names and where their tensors land in
the fused parameters, the order of layer runs, and properties of the restatement that the GPU tests lean on."""
import json
import math

import pytest
import torch

from oracle import zenedra_oracle as zo

LAYERS = [{"type": "gla", "mixer": {"heads": 2, "dim": 6, "vdim": 10, "tau": 8.0, "decay_rank": 4}, "mlp": None},
          {"type": "attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 10, "vdim": 10, "scale": 0.3, "mask": {"size": 5}}, "mlp": {"kind": "dense", "ff": 22}},
          {"type": "mlstm", "mixer": {"heads": 3, "dim": 4, "vdim": 8, "gate_cap": 7.0},
           "mlp": {"kind": "moe", "expert": {"ff": 18, "limit": 1.5}, "shared": {"ff": 14, "limit": 2.5},
                   "router": {"experts": 6, "top": 2, "scale": 1.25, "groups": {"count": 3, "keep": 1}}}},
          {"type": "attention", "mixer": {"heads": 2, "kv_heads": 2, "dim": 8, "vdim": 8, "scale": 0.1},
           "mlp": {"kind": "moe", "expert": {"ff": 4, "limit": 9.0}, "router": {"experts": 3, "top": 1}}}]
CFG = {"architecture": "Zenedra", "vocab": 53, "width": 36, "norm": {"eps": 1e-6}, "max_positions": 90, "layers": LAYERS,
       "embedding": {"bigram": {"buckets": 11, "mul_prev": 3, "mul_cur": 8}}, "loop": {"start": 1, "stop": 3, "times": 3}}


def test_registry_reads_the_configuration_from_a_directory(tmp_path):
    from nano_vllm_x_amd.registry import load_config, model_class_of
    from nano_vllm_x_amd.zenedra import ZenedraConfig, ZenedraForCausalLM
    (tmp_path / "config.json").write_text(json.dumps(CFG))
    cfg = load_config(str(tmp_path))
    assert isinstance(cfg, ZenedraConfig) and model_class_of(cfg) is ZenedraForCausalLM and ZenedraForCausalLM.family == "seq_state"
    assert (cfg.vocab_size, cfg.width, cfg.hidden_size, cfg.eps, cfg.max_positions) == (53, 36, 36, 1e-6, 90)
    assert cfg.bigram == {"buckets": 11, "mul_prev": 3, "mul_cur": 8} and cfg.loop == {"start": 1, "stop": 3, "times": 3}
    assert cfg.layers[1]["mixer"]["chunk"] == 5 and cfg.layers[3]["mixer"]["chunk"] is None and cfg.layers[0]["mlp"] is None
    assert cfg.layers[2]["mlp"]["shared"] == {"ff": 14, "limit": 2.5} and cfg.layers[3]["mlp"]["shared"] is None
    assert cfg.layers[3]["mlp"]["router"] == {"experts": 3, "top": 1, "scale": 1.0, "groups": None}
    again = ZenedraConfig.from_dict(json.loads(json.dumps(cfg.to_dict())))
    assert again == cfg
    plain = ZenedraConfig.from_dict({k: v for k, v in CFG.items() if k not in ("loop", "embedding")})
    assert plain.loop is None and plain.bigram is None and [r[:2] for r in plain.runs()] == [(i, (i, 0)) for i in range(4)]
    assert ZenedraConfig.from_dict(plain.to_dict()) == plain
    with pytest.raises(ValueError):
        ZenedraConfig.from_dict({**CFG, "layers": [{"type": "conv", "mixer": {"heads": 1, "dim": 1}, "mlp": None}]})
    with pytest.raises(ValueError):      # values are keys
        ZenedraConfig.from_dict({**CFG, "layers": [{**LAYERS[1], "mixer": {**LAYERS[1]["mixer"], "vdim": 8}}]})
    with pytest.raises(ValueError):
        ZenedraConfig.from_dict({**CFG, "layers": [{**LAYERS[1], "mlp": {"kind": "glu", "ff": 4}}]})
    for loop in ({"start": 2, "stop": 2, "times": 1}, {"start": 1, "stop": 5, "times": 1}, {"start": 0, "stop": 1, "times": 0}):
        with pytest.raises(ValueError):
            ZenedraConfig.from_dict({**CFG, "loop": loop})


def test_order_of_layer_runs_and_what_each_run_keeps():
    from nano_vllm_x_amd.zenedra import ZenedraConfig, ZenedraForCausalLM
    cfg = ZenedraConfig.from_dict(CFG)
    runs = cfg.runs()
    assert [i for i, _, _ in runs] == [0, 1, 2, 1, 2, 1, 2, 3] == [i for i, _ in zo.layer_order(4, CFG["loop"])]
    assert [p for _, _, p in runs] == [None, 0, None, 1, None, 2, None, None] and len({n for _, n, _ in runs}) == len(runs)
    model = ZenedraForCausalLM(cfg)
    f32 = torch.float32
    assert model.latent_ranks() == {**{((1, t), "k"): 20 for t in range(3)}, **{((1, t), "rn"): (2, f32) for t in range(3)},
                                    ((3, 0), "k"): 16, ((3, 0), "rn"): (2, f32)}
    shapes = model.state_shapes()
    assert shapes["prev_id"] == (1,) and shapes[((0, 0), "S")] == (2, 6, 10)
    assert all(shapes[((2, t), "S")] == (3, 4, 8) and shapes[((2, t), "n")] == (3, 4) and shapes[((2, t), "m")] == (3,) for t in range(3)) and len(shapes) == 11
    from nano_vllm_x_amd.core.kv_cache import LatentCachePool
    assert LatentCachePool.bytes_per_token(model.latent_ranks(), torch.bfloat16) == 3 * (40 + 8) + 32 + 8
    pool = LatentCachePool(torch.bfloat16, torch.device("cpu"), 5, model.latent_ranks())
    assert pool.get(((1, 2), "k")).dtype == torch.bfloat16 and pool.get(((1, 2), "rn")).dtype == f32 and pool.get(((1, 2), "rn")).shape == (5, 2)


def test_checkpoint_tensors_land_in_the_fused_parameters():
    from nano_vllm_x_amd.zenedra import ZenedraConfig, ZenedraForCausalLM, checkpoint_shapes, random_checkpoint
    cfg = ZenedraConfig.from_dict(CFG)
    w = dict(random_checkpoint(cfg, 3))
    assert {k: tuple(v.shape) for k, v in w.items()} == checkpoint_shapes(cfg)
    assert "l0.norm2" not in w and "l1.mix.v" not in w and "l3.mlp.shared.up" not in w and w["bigram"].shape == (12, 36) and w["loop.step"].shape == (3, 36)
    w["l0.mix.a1"], w["l0.mix.a2"] = torch.randn(7, 36), torch.randn(12, 7)          # the inner size of the decay is the checkpoint's
    model = ZenedraForCausalLM(cfg).float()
    model.load_weights(w.items())
    gla, att, mls, att2 = (l.mixer for l in model.layers)
    assert torch.equal(model.pair, w["bigram"]) and torch.equal(model.pos, w["pos"]) and torch.equal(model.head, w["head"])
    assert torch.equal(model.loop_in[0], w["loop.in"][:, :36]) and torch.equal(model.loop_in[1], w["loop.in"][:, 36:]) and torch.equal(model.loop_step, w["loop.step"])
    assert torch.equal(model._join_w[1], w["loop.in"][:, 36:])
    # norms of the stream are kept as the factor itself; the others are stored so
    assert torch.equal(model.layers[1].norm2, 1.0 + w["l1.norm2"]) and torch.equal(model.final_norm, 1.0 + w["final.norm"])
    assert torch.equal(att.q_norm, w["l1.mix.q.norm"]) and torch.equal(gla.norm, w["l0.mix.norm"]) and gla.norm.shape == (10,) and mls.norm.shape == (24,)
    assert gla.a1.shape == (7, 36) and torch.equal(gla.a2, w["l0.mix.a2"]) and torch.equal(gla.a2_b, w["l0.mix.a2.b"])
    rows = gla.qkvg_proj.weight
    assert rows.shape[0] == 2 * 12 + 2 * 20 and torch.equal(rows[12:24], w["l0.mix.k"]) and torch.equal(rows[44:], w["l0.mix.g"])
    rows = att.in_proj
    assert rows.weight.shape[0] == 60 and torch.equal(rows.weight[40:], w["l1.mix.k"]) and torch.equal(rows.bias[40:], w["l1.mix.k.b"]) and torch.equal(att.o_proj.bias, w["l1.mix.o.b"])
    assert torch.allclose(att.slopes.double(), zo.distance_slopes(4)) and att.chunk == 5 and att2.chunk == 0 and att2.window == 0
    assert torch.equal(mls.gate_w[3:], w["l2.mix.f"]) and torch.equal(mls.gate_b[:3], w["l2.mix.i.b"])
    moe = model.layers[2].mlp
    assert torch.equal(moe.w_gu[2, 18:], w["l2.mlp.e2.up"]) and torch.equal(moe.w_d[0], w["l2.mlp.e0.down"]) and torch.equal(moe.correction, w["l2.mlp.correction"])
    assert torch.equal(moe.shared.gu_proj.weight[14:], w["l2.mlp.shared.up"]) and moe.shared.limit == 2.5 and moe.limit == 1.5 and moe.scale == 1.25
    assert (moe.groups, moe.keep, moe.top, model.layers[3].mlp.groups, model.layers[3].mlp.shared) == (3, 1, 2, 0, None)
    dense = model.layers[1].mlp
    assert torch.equal(dense.gu_proj.weight[:22], w["l1.mlp.gate"]) and torch.equal(dense.down.weight, w["l1.mlp.down"])
    with pytest.raises(KeyError):
        model.load_weights([(k, v) for k, v in w.items() if k != "l1.mix.k.b"])
    with pytest.warns(UserWarning, match="does not use"):      # a tensor that nothing reads is left out, and said so
        model.load_weights(list(w.items()) + [("l1.mix.v", torch.zeros(20, 36))])
    half = ZenedraForCausalLM(cfg).to(torch.bfloat16)
    half.pack_decode_weights()
    assert half._join_w[0].shape == (36, 72) and torch.equal(half._join_w[0][:, :36], half._join_w[0][:, 36:])


def test_restatement_is_causal_and_its_parts_have_the_stated_form():
    from nano_vllm_x_amd.zenedra import ZenedraConfig, random_checkpoint
    cfg = ZenedraConfig.from_dict(CFG)
    w = dict(random_checkpoint(cfg, 1))
    toks = torch.randint(0, 53, (12,), generator=torch.Generator().manual_seed(0)).tolist()
    streams = []
    full = zo.forward(CFG, w, toks, streams)
    assert len(streams) == 8 and streams[0].shape == (12, 36)
    assert torch.allclose(zo.forward(CFG, w, toks[:7]), full[:7], atol=1e-12)
    assert (zo.forward(CFG, w, [(toks[0] + 1) % 53] + toks[1:])[-1] - full[-1]).abs().max() > 1e-6
    # pairs: the first token has the extra row; the hash is of the two ids in order
    assert zo.bigram_rows([4, 5, 4], 11, 3, 8) == [11, (12 + 40) % 11, (15 + 32) % 11]
    # one slope per head, whatever their number
    assert zo.distance_slopes(8).tolist() == [2.0 ** -(h + 1) for h in range(8)] and abs(zo.distance_slopes(3)[1].item() - 2.0 ** (-16 / 3)) < 1e-15
    g = torch.Generator().manual_seed(2)
    pos = torch.arange(6)
    v = torch.randn(6, 3, generator=g).double()
    zero = torch.zeros(6, 4).double()
    # with equal scores the weights fall by the slope alone; a chunk's first position sees itself only
    o = zo.chunk_softmax_readout(zero, zero, v, pos, pos, 1.0, math.log(2.0), None)
    assert torch.allclose(o[2], (v[0] / 4 + v[1] / 2 + v[2]) / 1.75)
    o = zo.chunk_softmax_readout(zero, zero, v, pos, pos, 1.0, 0.0, 4)
    assert torch.allclose(o[3], v[:4].mean(0)) and torch.allclose(o[4], v[4]) and torch.allclose(o[5], (v[4] + v[5]) / 2)
    # the decayed memory: decays act on key channels, a token's own write is read
    q, k = torch.ones(2, 2).double(), torch.tensor([[1.0, 0.0], [0.0, 1.0]]).double()
    o, s = zo.channel_decay_memory(q, k, torch.tensor([[1.0], [10.0]]).double(), torch.tensor([[0.1, 0.2], [0.5, 0.25]]).double())
    assert o[:, 0].tolist() == [1.0, 10.5] and s[:, 0].tolist() == [0.5, 10.0]
    # the gated memory: the running maximum starts at 0, not at minus infinity: a first input gate far below zero writes almost nothing
    one = torch.ones(1, 1).double()
    o, (s, n, m) = zo.exp_gated_memory(one, one, one, torch.tensor([-20.0]), torch.tensor([-1.0]))
    assert m == -1.0 and abs(s.item() - math.exp(-19.0)) < 1e-12 and abs(o.item() - math.exp(-19.0) / (math.exp(1.0) + 1e-6)) < 1e-12
    # the router: choice scores may be negative and a struck-out expert never wins; weights ignore the correction
    z, corr = [0.0, 0.0, 3.0, 3.0], [-5.0, -5.0, -9.0, -9.0]
    ids, wts = zo.route_logits(z, corr, {"experts": 4, "top": 2, "scale": 2.0, "groups": {"count": 2, "keep": 1}})
    assert sorted(ids) == [0, 1] and wts == [1.0, 1.0]
    # a group counts as the sum of its two best, not as its best
    ids, _ = zo.route_logits([9.0, -9.0, 0.5, 0.5], [0.0] * 4, {"experts": 4, "top": 1, "groups": {"count": 2, "keep": 1}})
    assert ids[0] in (2, 3)


def test_configurations_of_the_device_tests_are_read_alike_by_both_sides():
    """Every configuration the device tests use parses in the package and runs through the restatement with the package's random
    weights (names and shapes agree)."""
    import importlib.util
    import os
    spec = importlib.util.spec_from_file_location("gpu_zenedra", os.path.join(os.path.dirname(os.path.abspath(__file__)), "test_gpu_zenedra.py"))
    mod = importlib.util.module_from_spec(spec)
    spec.loader.exec_module(mod)
    for name, (layers, kw) in mod.ONE.items():
        cfg = mod.make_cfg(layers, **kw)
        out = zo.forward(cfg, mod.weights_of(cfg, 0), [1, 5, 2, 60, 0])
        assert out.shape == (5, 61) and torch.isfinite(out).all(), name
