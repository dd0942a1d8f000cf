"""Dagavik's configuration reader, checkpoint names, ranks taken from tensors, and cache shapes (no GPU),
and the float64 reference against itself: causality, windows, sinks, the two recurrences against
their unrolled sums, the choice among groups, the first token's pair row."""
import math

import pytest
import torch

from tests import dagavik_oracle as R
from vllm_legacy_amd.model.dagavik import ANY, DagavikConfig, DagavikForCausalLM
from vllm_legacy_amd.model.registry import resolve, supported_architectures


def small():
    return R.make_config([
        R.delta_layer(4, 2, 8, 12, 3, (5, 9), mlp=R.moe_mlp(6, 2, 10, (3, 2), 0.7)),
        R.latent_layer(3, 10, 6, 20, 0.4, mlp=R.moe_mlp(3, 1, 14)),
        R.parallel_layer((4, 2, 12, 10, 5, 6, 500.0, 0.3), (2, 6, 14, 9.0), (1.3, 0.2), mlp=None),
        R.latent_layer(2, 4, 8, 20, kv_from=1, mlp=R.moe_mlp(4, 3, 6, (2, 2)))], vocab=50, width=32, bigram=(19, 11, 3))


def test_registry_and_config():
    assert "Dagavik" in supported_architectures()
    model_cls, config_cls = resolve("Dagavik")
    assert model_cls is DagavikForCausalLM and config_cls is DagavikConfig
    cfg = DagavikConfig.from_dict(R.public_config(small()))
    d, c, p, e = (layer.mixer for layer in cfg.layers)
    assert (d.heads, d.kv_heads, d.dim, d.vdim, d.taps) == (4, 2, 8, 12, 3)
    assert (c.heads, c.dim, c.vdim, c.kv_rank, c.scale, c.kv_from) == (3, 10, 6, 20, 0.4, None)
    assert (e.heads, e.dim, e.vdim, e.kv_rank, e.scale, e.kv_from) == (2, 4, 8, 20, 0.5, 1)
    le, ri = p.left, p.right
    assert (le.heads, le.kv_heads, le.dim, le.vdim, le.window, le.rot_dims, le.rot_base, le.scale) == \
        (4, 2, 12, 10, 5, 6, 500.0, 0.3)
    assert (ri.heads, ri.dim, ri.vdim, ri.gate_cap, p.left_scale, p.right_scale) == (2, 6, 14, 9.0, 1.3, 0.2)
    m = cfg.layers[0].mlp
    assert (m.experts, m.top, m.ff, m.scale, m.groups, m.keep_groups) == (6, 2, 10, 0.7, 3, 2) and cfg.layers[2].mlp is None
    assert (cfg.vocab, cfg.width, cfg.eps, cfg.buckets, cfg.mul_prev, cfg.mul_cur) == (50, 32, 1e-5, 19, 11, 3)
    raw = R.public_config(small())
    del raw["layers"][2]["mixer"]["left"]["mask"], raw["layers"][2]["mixer"]["left"]["rot"]
    del raw["layers"][0]["mlp"]["router"]["groups"]
    cfg = DagavikConfig.from_dict(raw)
    assert (cfg.layers[2].mixer.left.window, cfg.layers[2].mixer.left.rot_dims) == (0, 0)
    assert (cfg.layers[0].mlp.groups, cfg.layers[0].mlp.keep_groups) == (1, 1)


def test_checkpoint_names_ranks_and_cache_shapes():
    raw = small()
    model = DagavikForCausalLM(DagavikConfig.from_dict(R.public_config(raw)), torch.float32, "cpu")
    assert model.tensor_shapes()["l0.mix.a1"] == (ANY, 32) and model.tensor_shapes()["l0.mix.g2"] == (48, ANY)
    W = R.random_tensors(raw, 0)
    assert model.load_weights(W) == len(W)
    assert {k: tuple(v.shape) for k, v in W.items()} == model.tensor_shapes()       # now with the ranks
    assert set(model.random_weights(1)) == set(W)
    # the projections that read h are one matrix, every part on a multiple of eight rows; a second step's
    # columns are padded to where its first step's part ends
    layer = model.layers[0]
    assert all(s % 8 == 0 for s in layer.in_starts) and layer.w_in.shape[0] % 8 == 0
    for (name, n, _), s in zip(layer.in_parts, layer.in_starts):
        assert torch.equal(layer.w_in.data[s:s + n], W["l0." + name].float()), name
    assert layer.w_decay.shape == (32, 8) and layer.w_gate.shape == (48, 16)
    assert torch.equal(layer.w_decay.data[:, :5], W["l0.mix.a2"].float()) and not layer.w_decay.data[:, 5:].any()
    assert torch.equal(layer.norm1.data, 1.0 + W["l0.norm1"].float())
    assert layer.recur.norm_weight.shape == (48, ) and torch.equal(layer.recur.norm_weight.data[12:24], W["l0.mix.norm"].float())
    caches = model.allocate_caches(5, 4, 2)
    assert len(caches) == 5 and caches[4]["last_token"].shape == (2, )
    assert caches[0]["state"].shape == (2, 4, 12, 8) and caches[0]["conv"].shape == (2, 2, 16 + 16 + 48)
    assert caches[1]["latent"].shape == (5, 4, 20) and caches[3] is caches[1]       # one latent cache, two readers
    assert caches[2]["keys"].shape == (5, 4, 2, 12) and caches[2]["values"].shape == (5, 4, 2, 10)
    assert caches[2]["memory"].shape == (2, 2, 6 * 15) and caches[2]["maximum"].shape == (2, 2)
    assert {caches[i][k].dtype for i, k in ((0, "state"), (0, "conv"), (2, "memory"), (2, "maximum"))} == {torch.float32}
    assert model.cache_spec()[3] == {}
    for name, change in (("l2.mix.left.v.b", None), ("l0.mix.a2", torch.zeros(32, 6)), ("l3.mix.uk", torch.zeros(8, 19))):
        bad = dict(W)
        if change is None:
            del bad[name]
        else:
            bad[name] = change
        with pytest.raises((KeyError, ValueError)):
            model.load_weights(bad)


def test_bad_configs_are_refused():
    for change in (lambda r: r["layers"][0].update(type="lstm"),
                   lambda r: r["layers"][0]["mlp"]["router"].update(top=5),             # two groups of two can be chosen
                   lambda r: r["layers"][0]["mlp"]["router"].update(groups={"count": 4, "keep": 2}),
                   lambda r: r["layers"][0]["mlp"]["router"].update(groups={"count": 3, "keep": 4}),
                   lambda r: r["layers"][0]["mlp"].update(kind="dense"),
                   lambda r: r["layers"][0]["mixer"].update(kv_heads=3),
                   lambda r: r["layers"][0]["mixer"].update(conv=0),
                   lambda r: r["layers"][2]["mixer"]["left"].update(kv_heads=3),
                   lambda r: r["layers"][2]["mixer"]["left"]["rot"].update(dims=14),
                   lambda r: r["layers"][2]["mixer"]["left"]["rot"].update(dims=5),
                   lambda r: r["layers"][2]["mixer"]["right"].update(gate_cap=0),
                   lambda r: r["layers"][3]["mixer"].update(kv_from=0),
                   lambda r: r["layers"][3]["mixer"].update(kv_from=3),
                   lambda r: r["layers"][3]["mixer"].update(kv_rank=24),
                   lambda r: r["layers"][1]["mixer"].update(kv_from=3)):
        raw = R.public_config(small())
        change(raw)
        with pytest.raises(ValueError):
            DagavikConfig.from_dict(raw)


def test_reference_is_causal_and_windowed():
    raw = small()
    W = R.random_tensors(raw, 1)
    toks = torch.randint(0, 50, (12, ), generator=torch.Generator().manual_seed(0)).tolist()
    full, part = R.forward(raw, W, toks), R.forward(raw, W, toks[:7])
    assert float((full[:7] - part).abs().max()) < 1e-9
    vis = R.visible(8, 3)
    assert vis[5].tolist() == [False] * 3 + [True] * 3 + [False] * 2 and vis[1].tolist() == [True] * 2 + [False] * 6
    assert torch.equal(R.visible(8, 3, 4), vis[4:])


def test_sink_joins_the_denominator():
    s = torch.tensor([[-2.0, 0.5, 3.0], [900.0, 1.0, -math.inf]], dtype=R.F)
    sink = torch.tensor([[1.5], [-3.0]], dtype=R.F)
    w = R.sink_softmax(s, sink)
    assert torch.allclose(w[0], torch.exp(s[0]) / (torch.exp(sink[0]) + torch.exp(s[0]).sum()))
    assert torch.allclose(w[1], torch.tensor([1.0, 0.0, 0.0], dtype=R.F))
    assert torch.allclose(R.sink_softmax(s), torch.softmax(s, -1))


def test_first_token_takes_the_last_pair_row():
    e, p = torch.arange(6, dtype=R.F)[:, None], 100 * torch.arange(5, dtype=R.F)[:, None]
    got = R.pair_embedding([3, 5, 1], e, p, 3, 2)
    assert got[:, 0].tolist() == [3 + 400, 5 + 100 * ((3 * 3 + 5 * 2) % 4), 1 + 100 * ((5 * 3 + 1 * 2) % 4)]


def test_matrix_memory_is_the_unrolled_sum():
    """The stabilized walk against sums of e^(sum f + i): the running maximum cancels, but for the floor."""
    g = torch.Generator().manual_seed(0)
    n, H, D, V = 7, 2, 3, 4
    q, k = (torch.randn((n, H, D), dtype=R.F, generator=g) for _ in range(2))
    v = torch.randn((n, H, V), dtype=R.F, generator=g)
    i, f = 3 * torch.randn((n, H), dtype=R.F, generator=g), -torch.rand((n, H), dtype=R.F, generator=g)
    o = R.matrix_memory_walk(q, k, v, i, f)
    m = torch.zeros(H, dtype=R.F)
    for t in range(n):
        m = torch.maximum(f[t] + m, i[t])
        w = torch.stack([torch.exp(f[j + 1:t + 1].sum(0) + i[j]) for j in range(t + 1)])            # [t + 1, H]
        dots = torch.stack([(k[j] * q[t]).sum(-1) for j in range(t + 1)])
        num, den = ((w * dots)[:, :, None] * v[:t + 1]).sum(0), (w * dots).sum(0)
        want = num / (torch.clamp(den.abs(), min=1.0) + 1e-6 * torch.exp(m))[:, None]
        assert torch.allclose(o[t], want), t


def test_delta_walk_overwrites_what_a_key_holds():
    """With beta = 1 and no decay, reading a key right after writing it returns its value, whatever the
    key held before; a decay acts on the key's channels."""
    k = torch.zeros((3, 1, 4), dtype=R.F)
    k[:, 0, 1] = 1.0
    v = torch.arange(6, dtype=R.F).view(3, 1, 2)
    g, beta = torch.ones((3, 1, 4), dtype=R.F), torch.ones((3, 1), dtype=R.F)
    o, S = R.delta_walk(k, k, v, g, beta)
    assert torch.equal(o, v)
    g[2, 0, 1] = 0.25
    beta[2] = 0.0
    o, _ = R.delta_walk(k, k, v, g, beta)
    assert torch.equal(o[2], 0.25 * v[1])
    z, a, b = torch.zeros((1, 1, 2), dtype=R.F), torch.zeros(1, dtype=R.F), torch.tensor([[0.0, -50.0]], dtype=R.F)
    assert torch.allclose(R.channel_decay(z, a, b), torch.tensor([[[0.5, 1.0]]], dtype=R.F))


def test_choice_among_groups():
    s = torch.tensor([0.05, 0.30, 0.28, 0.01, 0.26, 0.10], dtype=R.F)
    assert R.choose(s, 2, 3, 2).tolist() == [1, 2] and R.choose(s, 2, 1, 1).tolist() == [1, 2]
    assert R.choose(s, 3, 3, 2).tolist() == [1, 2, 0]                # 4 and 5 sit in the third-best group
    assert R.choose(s, 2, 3, 1).tolist() == [1, 0]
