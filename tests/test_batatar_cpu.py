"""Batatar's configuration reader, checkpoint names, order of layer runs and cache shapes (no GPU), and
the float64 reference against itself: causality, chunks, the sink, the recurrence against its
unrolled sum, the experts' weighted inputs."""
import math

import pytest
import torch

from tests import batatar_oracle as R
from vllm_legacy_amd.model.batatar import BatatarConfig, BatatarForCausalLM
from vllm_legacy_amd.model.registry import resolve, supported_architectures


def small():
    return R.make_config([
        R.lightning_layer(3, 8, 12, [0.5, 0.9, 0.99], mlp=R.moe_mlp(5, 2, 10)),
        R.parallel_layer((4, 2, 8, 12, 5, 15.0, 0.3), (6, 10, 7, 3, 2, 4), mlp=R.moe_mlp(3, 1, 14)),
        R.lightning_layer(2, 6, mlp=None)], vocab=50, width=32, residual_mult=0.4, loop=(1, 3, 3))


def test_registry_and_config():
    assert "Batatar" in supported_architectures()
    model_cls, config_cls = resolve("Batatar")
    assert model_cls is BatatarForCausalLM and config_cls is BatatarConfig
    cfg = BatatarConfig.from_dict(small())
    a, p, b = (layer.mixer for layer in cfg.layers)
    assert (a.heads, a.dim, a.vdim, a.decay) == (3, 8, 12, [0.5, 0.9, 0.99]) and (b.heads, b.dim, b.vdim) == (2, 6, 6)
    le, ri = p.left, p.right
    assert (le.heads, le.kv_heads, le.dim, le.vdim, le.chunk, le.softcap, le.scale) == (4, 2, 8, 12, 5, 15.0, 0.3)
    assert (ri.heads, ri.vdim, ri.state, ri.groups, ri.norm_groups, ri.taps) == (6, 10, 7, 3, 2, 4)
    assert (cfg.layers[0].mlp.experts, cfg.layers[0].mlp.top, cfg.layers[0].mlp.ff) == (5, 2, 10) and cfg.layers[2].mlp is None
    assert (cfg.vocab, cfg.width, cfg.residual_mult, cfg.eps) == (50, 32, 0.4, 1e-5)
    assert cfg.layer_runs() == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None)] == R.layer_order(small())
    raw = small()
    del raw["loop"], raw["layers"][1]["mixer"]["left"]["mask"], raw["layers"][1]["mixer"]["left"]["softcap"]
    raw["layers"][2]["mixer"]["decay"] = 0.75           # one number for all heads
    cfg = BatatarConfig.from_dict(raw)
    assert cfg.layer_runs() == [(0, None), (1, None), (2, None)] and not cfg.loops
    assert (cfg.layers[1].mixer.left.chunk, cfg.layers[1].mixer.left.softcap) == (0, 0.0)
    assert cfg.layers[2].mixer.decay == [0.75, 0.75]


def test_checkpoint_names_and_cache_shapes():
    raw = small()
    model = BatatarForCausalLM(BatatarConfig.from_dict(raw), torch.float32, "cpu")
    W = R.random_tensors(raw, 0)
    assert {k: tuple(v.shape) for k, v in W.items()} == model.tensor_shapes()
    assert model.load_weights(W) == len(W)
    assert set(model.random_weights(1)) == set(W)
    # the projections that read h are one matrix, every part on a multiple of eight rows
    layer = model.layers[1]
    assert all(s % 8 == 0 for s in layer.in_starts) and layer.w_in.shape[0] % 8 == 0
    inner = 60
    z, xbc, dt = (W["l1.mix.right.in"][a:b].float() for a, b in ((0, inner), (inner, 2 * inner + 42), (2 * inner + 42, None)))
    for part, want in zip((4, 5, 6), (z, xbc, dt)):
        s = layer.in_starts[part]
        assert torch.equal(layer.w_in.data[s:s + want.shape[0]], want)
    assert torch.equal(layer.b_in.data[layer.in_starts[1]:layer.in_starts[1] + 16], W["l1.mix.left.k.b"].float())
    assert not layer.b_in.data[layer.in_starts[3]:].any()
    caches = model.allocate_caches(5, 4, 2)
    assert len(caches) == 7                             # one per layer run
    assert caches[0]["state"].shape == (2, 3, 8, 12) and set(caches[0]) == {"state"}
    for run in (1, 3, 5):
        assert caches[run]["keys"].shape == (5, 4, 2, 8) and caches[run]["values"].shape == (5, 4, 2, 12)
        assert caches[run]["state"].shape == (2, 6, 7, 10) and caches[run]["conv"].shape == (2, 3, inner + 42)
    assert all(c["state"].dtype == torch.float32 for c in caches)
    assert caches[1]["state"].data_ptr() != caches[3]["state"].data_ptr()
    del W["l1.mix.left.v.b"]
    with pytest.raises(KeyError):
        model.load_weights(W)


def test_bad_configs_are_refused():
    for change in (lambda r: r["layers"][0].update(type="lstm"),
                   lambda r: r["layers"][0]["mlp"]["router"].update(top=9),
                   lambda r: r["layers"][0]["mlp"].update(kind="dense"),
                   lambda r: r["layers"][0]["mixer"].update(decay=[0.5]),
                   lambda r: r["layers"][1]["mixer"]["left"].update(kv_heads=3),
                   lambda r: r["layers"][1]["mixer"]["right"].update(groups=4),
                   lambda r: r["layers"][1]["mixer"]["right"].update(norm_groups=7),
                   lambda r: r["loop"].update(stop=9)):
        raw = small()
        change(raw)
        with pytest.raises(ValueError):
            BatatarConfig.from_dict(raw)
    raw = small()
    raw["layers"][0]["mixer"]["decay"] = [0.5, 0.9, 1.5]
    with pytest.raises(ValueError):
        BatatarForCausalLM(BatatarConfig.from_dict(raw), torch.float32, "cpu")


def test_log_decays():
    from vllm_legacy_amd.attention.recurrent import ConstantDecayRecurrence
    r = ConstantDecayRecurrence(4, 8, 8, [0.0, 0.25, 0.999, 1.0], 1e-5)
    logs = r.log_decay.tolist()
    assert logs[0] == -1e4 and math.exp(logs[0]) == 0.0 and logs[3] == 0.0
    assert logs[1] == pytest.approx(math.log(0.25), rel=1e-7) and logs[2] == pytest.approx(math.log(0.999), rel=1e-6)


def test_reference_is_causal_and_chunked():
    raw = small()
    W = R.random_tensors(raw, 1)
    toks = torch.randint(0, 50, (12, ), generator=torch.Generator().manual_seed(0)).tolist()
    full, part = R.forward(raw, W, toks), R.forward(raw, W, toks[:7])
    assert float((full[:7] - part).abs().max()) < 1e-9
    vis = R.visible(8, 3)
    assert vis[5].tolist() == [False] * 3 + [True] * 3 + [False] * 2 and vis[6].tolist() == [False] * 6 + [True, False]
    assert R.visible(8, 0)[5].tolist() == [True] * 6 + [False] * 2
    assert torch.equal(R.visible(8, 3, 4), vis[4:])


def test_sink_softmax_sums_to_less_than_one():
    s = torch.tensor([[-2.0, 0.5, 3.0], [-900.0, -901.0, -math.inf], [900.0, 1.0, -math.inf]], dtype=R.F)
    w = R.sink_softmax(s)
    e = torch.exp(s[0])
    assert torch.allclose(w[0], e / (1 + e.sum()))
    assert float(w[1].sum()) < 1e-300 and abs(float(w[2].sum()) - 1.0) < 1e-12
    assert torch.allclose(R.sink_softmax(s, False), torch.softmax(s, -1))


def test_decayed_walk_is_the_unrolled_sum():
    g = torch.Generator().manual_seed(0)
    n, H, D, V = 9, 2, 3, 4
    q, k = (torch.randn((n, H, D), dtype=R.F, generator=g) for _ in range(2))
    v, a = torch.randn((n, H, V), dtype=R.F, generator=g), torch.rand((n, H), dtype=R.F, generator=g)
    o, S = R.decayed_walk(q, k, v, a)
    t = 6
    want = sum((a[j + 1:t + 1].prod(0) * (q[t] * k[j]).sum(-1))[:, None] * v[j] for j in range(t + 1))
    assert torch.allclose(o[t], want)
    o1, S1 = R.decayed_walk(q[:4], k[:4], v[:4], a[:4])
    o2, S2 = R.decayed_walk(q[4:], k[4:], v[4:], a[4:], S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)


def test_expert_weights_multiply_the_inputs():
    g = torch.Generator().manual_seed(1)
    t = {"gate": torch.randn((5, 4), dtype=R.F, generator=g), "up": torch.randn((5, 4), dtype=R.F, generator=g),
         "down": torch.randn((4, 5), dtype=R.F, generator=g)}
    layer = {"router": torch.randn((1, 4), dtype=R.F, generator=g), **{f"e0.{k}": v for k, v in t.items()}}
    h = torch.randn((3, 4), dtype=R.F, generator=g)
    s = torch.sigmoid(h @ layer["router"].T)
    got = R.routed_ff(h, layer, R.moe_mlp(1, 1, 5))
    assert torch.allclose(got, R.expert(s * h, t))
    assert float((got - s * R.expert(h, t)).abs().max()) > 1e-2
