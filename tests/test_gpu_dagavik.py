"""Dagavik through the framework -- registry, checkpoint loader, cache manager, model runner,
scheduler, sampler -- and its mechanisms one by one, against the float64 reference of
tests/dagavik_oracle.py on small random models and inputs.

Mechanisms alone: the stream's update with several branches and two readers; the delta rule with a decay
per channel (token by token, in blocks, mixed runs, decays of 0 and 1, slots that hold anything, a
write that is read far behind); the matrix memory (gates, normalizer and floor, blocks and pieces, gates
at their caps, a token that outlives hundreds of others); head norms with a factor per head; windowed
attention with rotated and unrotated dimensions (one planted key just inside and just outside the window, at
page borders, in prompts and in decoding); latent attention with sinks (one planted key among hundreds,
shares of keys, sinks above and below the scores, a cache another layer fills); routing among groups.
Whole models: prompts whole, in portions down to two tokens and token by token; mixed batches with
pages and slots used again; long decoding; a batch does not change a request; greedy generation
through LLMEngine and the command line; the trace replayer as a program.  The float32 bar is
float32 rounding through the stack and is the one that finds faults of cutting, batching and
reuse; the bfloat16 runs cover the matrix-core kernels with a looser bar."""
import json
import os
import subprocess
import sys

import pytest
import torch

from tests import dagavik_oracle as R

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F = R.F
BAR = {torch.float32: 1e-4, torch.bfloat16: 0.2}
MEAN_BAR = {torch.float32: 1e-4, torch.bfloat16: 0.06}


def configs():
    D, P, L, E = R.delta_layer, R.parallel_layer, R.latent_layer, R.moe_mlp
    return {
        "plain": R.make_config([
            D(4, 2, 16, 24, 4, (8, 16), mlp=E(6, 2, 24, (3, 2))),
            L(4, 16, 16, 32, mlp=E(4, 1, 32, (2, 1), 0.8)),
            P((4, 2, 16, 24, 9, 8, 1000.0), (2, 16, 24, 15.0), mlp=E(4, 2, 40, (2, 2))),
            L(2, 24, 16, 32, kv_from=1, mlp=None)]),
        # sizes that are neither equal nor powers of two, one key head, vdim != dim, scales that are not
        # dim^-1/2, no feed-forward at the start, every dimension rotated, large eps
        "odd": R.make_config([
            P((3, 1, 12, 20, 7, 12, 100.0, 0.5), (3, 10, 14, 4.0), (1.4, 0.3), mlp=None),
            D(6, 3, 12, 20, 3, (3, 11), mlp=E(9, 3, 20, (3, 1), 3.0)),
            L(3, 10, 14, 28, 0.7, mlp=E(5, 2, 14)),
            L(5, 6, 10, 28, 0.2, kv_from=2, mlp=E(7, 7, 14)),
            L(2, 8, 8, 20, mlp=E(3, 1, 20, (3, 2)))], vocab=131, width=40, eps=1e-3, bigram=(7, 5, 3)),
        # key heads = heads, one expert, every expert chosen, one tap, a scale of one for both branches
        "equal": R.make_config([P((2, 2, 16, 16, 16, 4, 10000.0), (2, 16, 16, 8.0), (1.0, 1.0), mlp=E(3, 3, 16, scale=1.0)),
                                D(2, 2, 16, 16, 1, (16, 16), mlp=E(2, 2, 16, (2, 2), 1.0)),
                                L(4, 8, 8, 16, 1.0, mlp=E(1, 1, 16))]),
        # a window of one token and of more tokens than any request has, one head, nothing rotated, one bucket
        "edges": R.make_config([P((2, 1, 8, 8, 1, 2, 50.0), (1, 32, 4, 1.5), mlp=E(2, 1, 24, (2, 1))),
                                P((1, 1, 40, 12, 500, 0, 10.0), (3, 4, 20, 30.0), mlp=E(3, 2, 20)),
                                D(1, 1, 40, 8, 6, (1, 1), mlp=None),
                                L(1, 8, 40, 48, mlp=None)], width=48, bigram=(1, 3, 5)),
        # nothing a multiple of four: widths, head sizes, ranks, vocabulary, expert sizes
        "ragged": R.make_config([
            D(5, 5, 9, 14, 5, (6, 3), mlp=E(5, 2, 18)),
            P((3, 3, 10, 14, 11, 6, 77.0), (5, 7, 9, 12.0), mlp=E(6, 4, 6, (2, 2))),
            L(3, 7, 5, 22, mlp=E(3, 1, 30)),
            D(6, 2, 7, 11, 2, (10, 5), mlp=None),
            L(6, 22, 9, 22, kv_from=2, mlp=E(4, 2, 10, (4, 3)))], vocab=101, width=50),
        # sizes for the matrix-core kernels: multiples of 32, many heads, wide values, wide latents
        "mfma": R.make_config([
            D(4, 2, 64, 128, 4, (32, 24), mlp=E(8, 2, 32, (4, 2))),
            P((8, 2, 32, 64, 45, 16, 5000.0), (4, 96, 32, 15.0), mlp=E(8, 1, 64)),
            L(8, 32, 64, 96, mlp=E(4, 3, 32, (2, 2))),
            P((4, 4, 64, 32, 70, 64, 5000.0), (2, 64, 128, 20.0), mlp=None),
            L(4, 64, 32, 96, kv_from=2, mlp=E(4, 1, 64)),
            D(2, 2, 160, 32, 3, (8, 8), mlp=E(4, 2, 32))], width=128),
    }


class Served:
    """A checkpoint on disk, loaded through the registry, with the engine's cache manager and
    model runner around it."""

    def __init__(self, tmp_path, name, dtype, num_blocks=64, block_size=4, num_slots=3, seed=0):
        from vllm_legacy_amd.engine.cache_manager import CacheManager
        from vllm_legacy_amd.engine.model_runner import ModelRunner
        from vllm_legacy_amd.model.registry import load_model
        self.cfg = configs()[name]
        self.W = R.random_tensors(self.cfg, seed)
        self.folder = R.write_checkpoint(str(tmp_path / name), self.cfg, self.W)
        self.dtype = dtype
        self.model = load_model(self.folder, dtype, DEV)
        self.cache = CacheManager(num_blocks, block_size, num_slots)
        self.runner = ModelRunner(self.model, self.cache, DEV)
        self.done = {}

    def step(self, entries):
        """entries: [(id, tokens)]; logits of every token come back per id."""
        batch, want = [], []
        for sid, tokens in entries:
            if not self.cache.is_live(sid):
                self.cache.admit(sid)
                self.done[sid] = 0
            self.cache.grow(sid, self.done[sid] + len(tokens))
            batch.append((sid, list(tokens), self.done[sid]))
            want.append(list(range(len(tokens))))
        logits = self.runner.execute(batch, want).cpu()
        out, at = {}, 0
        for sid, tokens in entries:
            out[sid] = logits[at:at + len(tokens)]
            at += len(tokens)
            self.done[sid] += len(tokens)
        return out

    def end(self, sid):
        self.cache.free(sid)
        del self.done[sid]

    def reference(self, tokens):
        return R.forward(self.cfg, self.W, tokens)

    def check(self, got, tokens, what=""):
        within(logit_error(got, self.reference(tokens)), self.dtype, what)


def logit_error(got, want):
    return R.row_errors(got, want) / R.spread(want.to(F))


def within(err, dtype, what=""):
    # in bfloat16 a router's close call can go the other way than in the float64 reference and move
    # that token's logits: one row in ten may be out; float32 rows must all be in
    worst = float(err.max()) if dtype == torch.float32 else float(torch.quantile(err, 0.9))
    assert worst <= BAR[dtype] and float(err.mean()) <= MEAN_BAR[dtype], (what, float(err.max()), float(err.mean()))


def tokens_of(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n, ), generator=g).tolist()


def rnd(shape, seed, std=1.0):
    return torch.randn(shape, generator=torch.Generator().manual_seed(seed)) * std


def make_batch(query_lens, context_lens, block_size=4, tables=None, slots=None):
    from vllm_legacy_amd.attention.batch import SequenceBatch
    if tables is None:
        tables, at = [], 0
        for n, c in zip(query_lens, context_lens):
            need = (n + c + block_size - 1) // block_size
            tables.append(list(range(at, at + need)))
            at += need
    slots = list(range(len(query_lens))) if slots is None else slots
    return SequenceBatch.build(query_lens, context_lens, tables, slots, block_size, DEV)


def close(got, want, tol, what=""):
    err = float((got.detach().cpu().to(F) - want).abs().max() / want.abs().max().clamp_min(1e-30))
    assert err <= tol, (what, err)


def run_plan(plan, lens, slots, call, block_size=4):
    """Feeds sequences through `call(batch, {key: (first row, rows)})` -> output rows, step by step; a plan's
    step is [(key, tokens)].  Returns every key's rows in order.  `slots` says which slot a key has."""
    at, got = {k: 0 for k in lens}, {k: [] for k in lens}
    for step in plan:
        batch = make_batch([n for _, n in step], [at[k] for k, _ in step], block_size, slots=[slots[k] for k, _ in step])
        out = call(batch, [(k, at[k], n) for k, n in step]).float().cpu()
        lo = 0
        for k, n in step:
            got[k].append(out[lo:lo + n])
            at[k] += n
            lo += n
    assert at == lens, (at, lens)
    return {k: torch.cat(v) for k, v in got.items()}


MIXED_PLAN = [[("a", 70), ("b", 2)], [("b", 1), ("a", 1), ("c", 5)], [("c", 1), ("b", 4), ("a", 9)],
              [("a", 1), ("c", 1), ("d", 1)], [("d", 1)], [("d", 17), ("c", 33), ("a", 16)], [("d", 2), ("a", 3)]]
MIXED_LENS = {"a": 100, "b": 7, "c": 40, "d": 21}
MIXED_SLOTS = {"a": 0, "b": 1, "c": 2, "d": 1}          # d takes the slot that b leaves


def rows_of(seqs, parts):
    return torch.cat([seqs[k][lo:lo + n] for k, lo, n in parts]).to(DEV)


# ----------------------------------------------------------------------------- the stream's update
@pytest.mark.parametrize("width", [40, 50, 256, 2500, 5000])
@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
def test_branch_sums_and_their_readers_norms(width, out_dtype):
    """Up to three scaled terms and a token's expert rows (one choice without a row) join the stream; none,
    one or two readers get their normed copies."""
    from vllm_legacy_amd import _seq_ops as ops
    T = 5
    x = rnd((T, width), 1)
    ys = [(rnd((T, width), 2 + i, 1.0 + i), f) for i, f in enumerate((0.7, -1.3, 1.0))]
    ye, wts = rnd((9, width), 7, 2.0), rnd((T, 3), 8)
    pair = torch.tensor([[0, 3, 8], [1, -1, 2], [4, 4, 4], [7, 6, 5], [-1, -1, 0]], dtype=torch.int32)
    esum = torch.stack([sum(wts[t, k].to(F) * ye[pair[t, k]].to(F) for k in range(3) if pair[t, k] >= 0) for t in range(T)])
    ws = [1 + 0.3 * rnd((width, ), 11), 1 + 0.3 * rnd((width, ), 12)]
    for nt in range(4):
        for experts in (False, True):
            for readers in range(3):
                want = x.to(F) + sum(f * y.to(F) for y, f in ys[:nt]) + (esum if experts else 0)
                xs = x.to(DEV).clone()
                outs = [(torch.empty((T, width), dtype=out_dtype, device=DEV), w.to(DEV)) for w in ws[:readers]]
                ops.branch_sum_norms(xs, [(y.to(DEV), f) for y, f in ys[:nt]],
                                     (ye.to(DEV), pair.to(DEV), wts.to(DEV)) if experts else None, outs, 1e-3)
                close(xs, want, 3e-6, (nt, experts, readers))
                for (o, _), w in zip(outs, ws):
                    close(o, R.rms_norm(want, w.to(F), 1e-3), 3e-6 if out_dtype == torch.float32 else 6e-3, (nt, readers))


# ----------------------------------------------------------------------------- delta rule, a decay per channel
DELTA_SHAPES = [(2, 2, 16, 16), (4, 2, 20, 12), (3, 1, 64, 40), (6, 3, 96, 64), (2, 1, 130, 33), (1, 1, 256, 16),
                (2, 2, 7, 9), (1, 1, 300, 8), (4, 4, 128, 128), (1, 1, 1, 1)]


def delta_inputs(n, shape, seed, dtype, spread=2.0):
    H, G, D, V = shape
    q, k, v = rnd((n, G * D), seed).to(dtype), rnd((n, G * D), seed + 1).to(dtype), rnd((n, H * V), seed + 2).to(dtype)
    return q, k, v, rnd((n, H), seed + 3, 2.0).to(dtype), rnd((n, H * D), seed + 4, spread)


def delta_reference(x, shape, a_log, dt_bias):
    H, G, D, V = shape
    q, k, v, b, z = (t.to(F) for t in x)
    n = q.shape[0]
    q = (R.unit_vector(q.view(n, G, D)) * D**-0.5).repeat_interleave(H // G, 1)
    k = R.unit_vector(k.view(n, G, D)).repeat_interleave(H // G, 1)
    g = R.channel_decay(z.view(n, H, D), a_log.to(F), dt_bias.to(F).view(H, D))
    return R.delta_walk(q, k, v.view(n, H, V), g, torch.sigmoid(b))


def delta_call(shape, seqs, state, a_log, dt_bias):
    from vllm_legacy_amd import _seq_ops as ops
    H, G, D, V = shape

    def call(batch, parts):
        # rows are slices of a wider matrix, as a merged projection leaves them
        q, k, v, b, z = (rows_of({key: s[i] for key, s in seqs.items()}, parts) for i in range(5))
        wide = torch.cat([q, k, v, b], 1)
        q, k, v, b = wide.split([G * D, G * D, H * V, H], 1)
        o = torch.full((q.shape[0], H * V), 7.0, device=DEV)
        ops.channel_delta_scan(o, q, k, v, b, z, dt_bias.to(DEV), a_log.to(DEV), state, batch.query_start_loc,
                               batch.context_lens, batch.state_slots, G, batch.max_query_len)
        return o

    return call


@pytest.mark.parametrize("shape", DELTA_SHAPES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_channel_delta_rule(shape, dtype):
    """Mixed runs of four sequences (one takes over a slot), all three kernel choices; slots start as NaN."""
    from vllm_legacy_amd import _seq_ops as ops
    H, G, D, V = shape
    a_log, dt_bias = rnd((H, ), 1, 0.7), rnd((H * D, ), 2) - 2.0
    seqs = {k: delta_inputs(n, shape, 10 * i, dtype) for i, (k, n) in enumerate(MIXED_LENS.items())}
    want = {k: delta_reference(x, shape, a_log, dt_bias) for k, x in seqs.items()}
    for mode in (0, 1, 2):
        ops.set_channel_delta_kernel(mode)
        try:
            state = torch.full((4, H, V, D), float("nan"), device=DEV)
            got = run_plan(MIXED_PLAN, MIXED_LENS, MIXED_SLOTS, delta_call(shape, seqs, state, a_log, dt_bias))
        finally:
            ops.set_channel_delta_kernel(0)
        for k, (o, S) in want.items():
            close(got[k], o.reshape(MIXED_LENS[k], H * V), 2e-5, (mode, k))
            if k != "b":
                close(state[MIXED_SLOTS[k]], S.transpose(1, 2), 2e-5, (mode, k, "state"))
        assert bool(torch.isnan(state[3]).all())            # nobody's slot


def test_channel_delta_rule_at_extreme_decays():
    """Channels that forget everything at every token beside channels that forget nothing, and tokens whose
    decay underflows to 0 for all channels; keys that repeat exactly with beta near 1."""
    from vllm_legacy_amd import _seq_ops as ops
    shape, n = (2, 1, 32, 16), 75
    H, G, D, V = shape
    q, k, v, b, z = delta_inputs(n, shape, 5, torch.float32, 0.5)
    z[:, ::3] = -60.0                   # g = 1
    z[:, 1::3] = 200.0                  # g = 0
    z[20], z[21], z[50] = 3000.0, -60.0, 90.0
    k[30:40] = k[29]
    b[28:45] = 30.0
    a_log, dt_bias = torch.tensor([0.3, -0.2]), torch.zeros(H * D)
    x = (q, k, v, b, z)
    want, _ = delta_reference(x, shape, a_log, dt_bias)
    assert bool(torch.isfinite(want).all())
    for mode in (1, 2):
        ops.set_channel_delta_kernel(mode)
        try:
            got = run_plan([[("a", 47)], [("a", 2)], [("a", 26)]], {"a": n}, {"a": 0},
                           delta_call(shape, {"a": x}, torch.zeros((1, H, V, D), device=DEV), a_log, dt_bias))["a"]
        finally:
            ops.set_channel_delta_kernel(0)
        close(got, want.reshape(n, H * V), 2e-5, mode)


def test_channel_delta_rule_reads_a_far_write():
    """One key is written once and nothing else touches its channel; 600 tokens later a query along it
    still finds the value, through prompts in portions and decoded tokens."""
    shape, n = (1, 1, 32, 16), 640
    H, G, D, V = shape
    q, k, v, b, z = delta_inputs(n, shape, 9, torch.float32, 0.1)
    k[:, 0], q[:, 0] = 0.0, 0.0
    k[3] = torch.eye(D)[0]
    q[635] = torch.eye(D)[0]
    b[3], z[:, 0], z[:, 1:] = 40.0, -12.0, -1.0
    x, a_log, dt_bias = (q, k, v, b, z), torch.zeros(H), torch.zeros(H * D)
    want, _ = delta_reference(x, shape, a_log, dt_bias)
    assert float((want[635, 0] - v[3].to(F) * D**-0.5).abs().max()) < 0.01 * float(v[3].abs().max())
    for plan in ([n], [300, 2, 330] + [1] * 8, [17] * 37 + [11]):
        got = run_plan([[("a", c)] for c in plan], {"a": n}, {"a": 1},
                       delta_call(shape, {"a": x}, torch.zeros((2, H, V, D), device=DEV), a_log, dt_bias))["a"]
        close(got, want.reshape(n, V), 3e-5, plan[:2])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("shape", [(4, 2, 16, 24), (3, 3, 9, 14), (2, 1, 64, 128)])
def test_channel_delta_layer(dtype, shape):
    """With its head norm and output gate."""
    from vllm_legacy_amd.attention.recurrent import ChannelDeltaRule
    H, G, D, V = shape
    n = 45
    layer = ChannelDeltaRule(H, G, D, V, 1e-4, DEV)
    a_log, dt_bias, nw = rnd((H, ), 1, 0.5), rnd((H * D, ), 2) - 2.0, 1 + 0.3 * rnd((V, ), 3)
    layer.set_weights(a_log, dt_bias, nw)
    x = delta_inputs(n, shape, 4, dtype)
    gate = rnd((n, H * V), 30, 2.0).to(dtype)
    o, _ = delta_reference(x, shape, a_log, dt_bias)
    want = R.rms_norm(o, nw.to(F), 1e-4).reshape(n, H * V) * torch.sigmoid(gate.to(F))
    state, at, outs = torch.full(ChannelDeltaRule.get_state_shape(2, H, D, V), 3.0, device=DEV), 0, []
    for c in (20, 1, 2, 21, 1):
        q, k, v, b, z = (t[at:at + c].to(DEV) for t in x)
        out = torch.empty((c, H * V), dtype=dtype, device=DEV)
        layer(out, q, k, v, gate[at:at + c].to(DEV), b, z, state, make_batch([c], [at], 4, slots=[1]))
        outs.append(out.float().cpu())
        at += c
    close(torch.cat(outs), want, 3e-5 if dtype == torch.float32 else 1e-2)
    assert bool((state[0] == 3.0).all())


# ----------------------------------------------------------------------------- matrix memory
MEMORY_SHAPES = [(2, 8, 8), (4, 16, 24), (3, 10, 7), (3, 32, 96), (2, 128, 128), (1, 96, 200), (2, 20, 300), (1, 160, 16), (5, 1, 1)]


def memory_inputs(n, shape, seed, dtype, spread=3.0):
    H, D, V = shape
    return rnd((n, H * D), seed).to(dtype), rnd((n, H * D), seed + 1).to(dtype), rnd((n, H * V), seed + 2).to(dtype), \
        rnd((n, H), seed + 3, spread), rnd((n, H), seed + 4, spread) + 1.0


def memory_reference(x, shape, bi, bf, cap):
    H, D, V = shape
    q, k, v, zi, zf = (t.to(F) for t in x)
    n = q.shape[0]
    eye = torch.eye(H, dtype=F)
    i, _ = R.memory_gates(zi, {"i": eye, "i.b": bi.to(F), "f": eye, "f.b": bf.to(F)}, cap)
    _, f = R.memory_gates(zf, {"i": eye, "i.b": bi.to(F), "f": eye, "f.b": bf.to(F)}, cap)
    return R.matrix_memory_walk(q.view(n, H, D) * D**-0.5, k.view(n, H, D), v.view(n, H, V), i, f).reshape(n, H * V)


def memory_call(shape, seqs, state, maximum, bi, bf, cap):
    from vllm_legacy_amd import _seq_ops as ops
    H, D, V = shape

    def call(batch, parts):
        q, k, v, zi, zf = (rows_of({key: s[i] for key, s in seqs.items()}, parts) for i in range(5))
        at = (batch.query_start_loc, batch.context_lens, batch.state_slots)
        rl, rw, rf = ops.matrix_memory_gates(zi, zf, bi.to(DEV), bf.to(DEV), cap, maximum, *at, batch.max_query_len)
        assert float(rl.max()) <= 1e-5 and float(rw.max()) <= 1.0 + 1e-6
        o, ns = torch.empty((q.shape[0], H * V), device=DEV), torch.empty((q.shape[0], H), device=DEV)
        ops.decay_scan(o, q, k, v, state, *at, H, batch.max_query_len, row_log=rl, row_weight=rw, row_floor=rf,
                       norm_scale=ns, norm_eps=1e-6, q_scale=D**-0.5, sizes=(D, V))
        return (o.view(-1, H, V) * ns[:, :, None]).view(-1, H * V)

    return call


@pytest.mark.parametrize("shape", MEMORY_SHAPES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_matrix_memory(shape, dtype):
    """Mixed runs of four sequences (one takes over a slot), all three kernel choices; slots start as NaN."""
    from vllm_legacy_amd import _seq_ops as ops
    from vllm_legacy_amd.attention.recurrent import MatrixMemory
    H, D, V = shape
    bi, bf, cap = rnd((H, ), 1), 1.0 + rnd((H, ), 2), 6.0
    seqs = {k: memory_inputs(n, shape, 10 * i, dtype) for i, (k, n) in enumerate(MIXED_LENS.items())}
    want = {k: memory_reference(x, shape, bi, bf, cap) for k, x in seqs.items()}
    for mode in (0, 1, 2):
        ops.set_decay_scan_kernel(mode)
        try:
            state, maximum = (torch.full(s, float("nan"), device=DEV) for s in MatrixMemory.get_state_shapes(4, H, D, V))
            got = run_plan(MIXED_PLAN, MIXED_LENS, MIXED_SLOTS, memory_call(shape, seqs, state, maximum, bi, bf, cap))
        finally:
            ops.set_decay_scan_kernel(0)
        for k in want:
            # where n . q nearly cancels above the floor, rounding is magnified: rows relative to the largest
            close(got[k], want[k], 1e-4, (mode, k))
        assert bool(torch.isnan(state[3]).all()) and bool(torch.isnan(maximum[3]).all())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("lens", [(257, 3), (700, 258), (1100, 1)])
def test_matrix_memory_in_pieces(dtype, lens):
    """Long runs are cut into pieces that are walked at once; the normalizer travels with them.  The running
    maximum passes several stretches of the gates' scan."""
    from vllm_legacy_amd.attention.recurrent import MatrixMemory
    shape = (2, 24, 40)
    H, D, V = shape
    bi, bf, cap = rnd((H, ), 1), 3.0 + rnd((H, ), 2), 15.0
    seqs = {k: memory_inputs(n + 30, shape, 7 * i, dtype) for i, (k, n) in enumerate(zip("ab", lens))}
    # queries and keys of one sign: n . q does not cancel, so the outputs are as exact as their sums
    seqs = {k: (x[0].abs(), x[1].abs()) + x[2:] for k, x in seqs.items()}
    state, maximum = (torch.full(s, float("nan"), device=DEV) for s in MatrixMemory.get_state_shapes(2, H, D, V))
    plan = [[("a", lens[0]), ("b", lens[1])], [("b", 29), ("a", 1)], [("a", 29), ("b", 1)]]
    got = run_plan(plan, {k: n + 30 for k, n in zip("ab", lens)}, {"a": 1, "b": 0},
                   memory_call(shape, seqs, state, maximum, bi, bf, cap))
    for k in seqs:
        close(got[k], memory_reference(seqs[k], shape, bi, bf, cap), 3e-5, k)


@pytest.mark.parametrize("cap", [1.5, 15.0, 40.0])
def test_matrix_memory_at_its_gates_limits(cap):
    """Input gates at plus and minus the cap, forget gates that drop everything and that keep everything, and
    a first token whose weight lies far below the starting maximum of 0 (the floor decides)."""
    from vllm_legacy_amd import _seq_ops as ops
    from vllm_legacy_amd.attention.recurrent import MatrixMemory
    shape, n = (2, 16, 12), 150
    H, D, V = shape
    q, k, v, zi, zf = memory_inputs(n, shape, 3, torch.float32, 1.0)
    zi[0], zi[5], zi[70:75], zi[100] = -1000.0, 1000.0, -1000.0, 1000.0
    zf[6:60], zf[60], zf[61:90], zf[130] = 1000.0, -1000.0, 1000.0, -1000.0
    x, bi, bf = (q, k, v, zi, zf), torch.zeros(H), torch.zeros(H)
    want = memory_reference(x, shape, bi, bf, cap)
    for mode in (1, 2):
        ops.set_decay_scan_kernel(mode)
        try:
            state, maximum = (torch.zeros(s, device=DEV) for s in MatrixMemory.get_state_shapes(1, H, D, V))
            got = run_plan([[("a", 3)], [("a", 100)], [("a", 2)], [("a", 45)]], {"a": n}, {"a": 0},
                           memory_call(shape, {"a": x}, state, maximum, bi, bf, cap))["a"]
        finally:
            ops.set_decay_scan_kernel(0)
        for lo, hi in ((0, 1), (1, 6), (6, 70), (70, 101), (101, n)):
            close(got[lo:hi], want[lo:hi], 2e-4, (mode, lo))


def test_matrix_memory_keeps_a_far_token():
    """A token written with a large input gate outweighs 600 later ones while the forget gates stay open."""
    from vllm_legacy_amd.attention.recurrent import MatrixMemory
    shape, n = (1, 16, 8), 620
    H, D, V = shape
    q, k, v, zi, zf = memory_inputs(n, shape, 3, torch.float32, 0.2)
    zi[4], zf[5:], k[4], q[615] = 14.0, 30.0, 3 * torch.eye(D)[2], 3 * torch.eye(D)[2]
    x, bi, bf = (q, k, v, zi, zf), torch.zeros(H), torch.zeros(H)
    want = memory_reference(x, shape, bi, bf, 15.0)
    assert float((want[615] - v[4].to(F)).abs().max()) < 0.05 * float(v[4].abs().max())
    for plan in ([n], [300, 2, 310] + [1] * 8, [9] * 68 + [8]):
        state, maximum = (torch.zeros(s, device=DEV) for s in MatrixMemory.get_state_shapes(1, H, D, V))
        got = run_plan([[("a", c)] for c in plan], {"a": n}, {"a": 0},
                       memory_call(shape, {"a": x}, state, maximum, bi, bf, 15.0))["a"]
        close(got, want, 1e-4, plan[:2])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n,groups", [(48, 3), (50, 5), (4096, 32), (1024, 4), (600, 2), (6, 6)])
def test_head_norms_with_a_factor_per_head(dtype, n, groups):
    """o times a factor per (token, head), then its root mean square per head, the weights, the gate: heads
    of up to 256 numbers (lanes of a wave share one), longer ones and unaligned rows."""
    from vllm_legacy_amd import _seq_ops as ops
    T = 5
    o, w, factor = rnd((T, n), 1), 1 + 0.2 * rnd((n, ), 2), torch.exp(2 * rnd((T, groups), 3))
    wide = rnd((T, n + 8), 4, 1.5).to(dtype)
    for first in (0, 1, 8):
        z = wide[:, first:first + n]
        u = o.to(F).view(T, groups, -1) * factor.to(F)[:, :, None]
        for gate_first in (False, True):
            gv = torch.sigmoid(z.to(F)).view(T, groups, -1)
            want = R.unit_rms(u * gv if gate_first else u, 1e-2)
            want = (want if gate_first else want * gv).reshape(T, n) * w.to(F)
            out = torch.full((T, n + 8), 7.0, dtype=dtype, device=DEV)
            ops.gated_group_rms_norm(out[:, first:first + n], o.to(DEV), w.to(DEV), wide.to(DEV)[:, first:first + n], "sigmoid",
                                     gate_first, groups, 1e-2, factor.to(DEV))
            close(out[:, first:first + n], want, 5e-6 if dtype == torch.float32 else 6e-3, (first, gate_first))
            assert bool((out[:, :first] == 7.0).all()) and bool((out[:, first + n:] == 7.0).all())


# ----------------------------------------------------------------------------- windowed attention
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("shape", [(4, 2, 16, 24, 9, 8), (6, 2, 64, 192, 40, 16), (3, 1, 10, 7, 33, 10), (8, 2, 64, 128, 64, 32),
                                   (2, 1, 32, 320, 20, 8), (2, 2, 300, 400, 17, 16), (6, 3, 128, 160, 50, 64)])
def test_window_edges_by_one_planted_key(dtype, shape):
    """One key matches one query through an unrotated (or, where all turn, the slowest) dimension; it is
    seen at a distance of window - 1 and not at a distance of window, in a prompt, in portions and
    decoded, wherever it lies on a page."""
    from vllm_legacy_amd.attention.backends.rotary_kv import RotaryKVAttention
    H, G, D, V, window, dims = shape
    BS = 4
    attn = RotaryKVAttention(H, G, D, V, D**-0.5, dims, 1e6, interleaved=False, window=window, device=DEV)
    spot = D - 1                                    # with every dimension turned: the second half of the slowest pair
    for j in (0, 3, 4, 9):
        for inside in (True, False):
            i = j + window - (1 if inside else 0)
            n = i + 3
            q, k, v = rnd((n, H, D), 1, 0.1), rnd((n, G, D), 2, 0.1), rnd((n, G, V), 3)
            q[i, :, spot], k[j, :, spot], v[j] = 12.0, 12.0 * D**0.5, 50.0
            q, k, v = (t.to(dtype) for t in (q, k, v))
            rq, rk = (R.rotate_half(t.to(F), dims, 1e6) for t in (q, k))
            want = R.attention_core(rq, rk, v.to(F), D**-0.5, window).reshape(n, H * V)
            assert (float(want[i].abs().min()) > 40.0) == inside
            for cuts in ([n], [i - 1, 4] if i > 1 else [n], [n - 4] + [1] * 4):
                kc, vc = (torch.full(s, float("nan"), dtype=dtype, device=DEV)
                          for s in RotaryKVAttention.get_cache_shapes(40, BS, G, D, V))
                table = torch.randperm(40, generator=torch.Generator().manual_seed(j))[:(n + BS - 1) // BS].tolist()
                at, outs = 0, []
                for c in cuts:
                    batch = make_batch([c], [at], BS, [table])
                    out = torch.empty((c, H * V), dtype=dtype, device=DEV)
                    qq, kk, vv = (t[at:at + c].reshape(c, -1).to(DEV) for t in (q, k, v))
                    attn(out, qq.clone(), kk, vv, None, kc, vc, batch)
                    outs.append(out.float().cpu())
                    at += c
                close(torch.cat(outs), want, 2e-5 if dtype == torch.float32 else 2e-2, (j, inside, cuts[:2]))


# ----------------------------------------------------------------------------- latent attention
def latent_case(n, H, D, V, rank, seed, dtype, sink):
    t = {"uk": rnd((H * D, rank), seed, rank**-0.5), "uv": rnd((H * V, rank), seed + 1, rank**-0.5), "dkv.norm": 1 + 0.2 * rnd((rank, ), seed + 2),
         "sink": sink}
    t = {k: v.to(torch.bfloat16) for k, v in t.items()}
    return t, rnd((n, H * D), seed + 3).to(dtype), rnd((n, rank), seed + 4).to(dtype)


def latent_want(t, q, kv, H, D, V, scale, eps=1e-5):
    n = q.shape[0]
    tf = {k: v.to(F) for k, v in t.items()}
    c = R.rms_norm(kv.to(F), tf["dkv.norm"], eps)
    k, v = (c @ tf["uk"].T).view(n, H, D), (c @ tf["uv"].T).view(n, H, V)
    return R.attention_core(q.to(F).view(n, H, D), k, v, scale, sink=tf["sink"]).reshape(n, H * V)


def latent_run(attns, t, q, kv, cuts, block_size=4, splits=None):
    """attns: (layer with its own latents, layer that reads them); both see the same queries."""
    own, reader = attns
    n, dtype = q.shape[0], q.dtype
    need = (n + block_size - 1) // block_size
    cache = torch.full((need + 5, block_size, own.rank), float("nan"), dtype=dtype, device=DEV)
    table = torch.randperm(need + 5, generator=torch.Generator().manual_seed(n))[:need].tolist()
    outs, at = [], 0
    for c in cuts:
        batch = make_batch([c], [at], block_size, [table])
        # a wider row, as a merged projection leaves it
        wide = torch.cat([q[at:at + c], kv[at:at + c]], 1).to(DEV)
        a = own(wide[:, :q.shape[1]], wide[:, q.shape[1]:], cache, batch)
        b = reader(wide[:, :q.shape[1]], None, cache, batch)
        assert torch.equal(a, b)
        outs.append(a.float().cpu())
        at += c
    return torch.cat(outs)


def latent_layers(H, D, V, rank, scale, dtype, t):
    from vllm_legacy_amd.attention.backends.latent_kv import LatentKVAttention
    own = LatentKVAttention(H, D, 0, V, rank, scale, 0, 1.0, None, 1e-5, dtype, DEV, sinks=True)
    reader = LatentKVAttention(H, D, 0, V, rank, scale, 0, 1.0, None, 1e-5, dtype, DEV, sinks=True, own_latent=False)
    own.set_weights(t["uk"], t["uv"], t["dkv.norm"], t["sink"])
    reader.set_weights(t["uk"], t["uv"], None, t["sink"])
    return own, reader


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("shape", [(4, 16, 16, 32, 0.25), (3, 10, 14, 28, 0.7), (8, 32, 64, 96, 0.2), (33, 8, 8, 64, 0.3),
                                   (2, 24, 40, 512, 0.2), (5, 7, 3, 22, 1.1), (1, 64, 16, 160, 0.1)])
def test_latent_attention_with_sinks(dtype, shape):
    """Sinks far below, around and far above the scores; prompts, portions, decoded tokens; a second layer
    reads the same cache; cache places nobody wrote are NaN."""
    H, D, V, rank, scale = shape
    sink = torch.linspace(-8.0, 8.0, H) if H > 1 else torch.tensor([1.5])
    t, q, kv = latent_case(50, H, D, V, rank, 1, dtype, sink)
    want = latent_want(t, q, kv, H, D, V, scale)
    plain = latent_want({**t, "sink": torch.full((H, ), -1e4)}, q, kv, H, D, V, scale)
    assert float((want - plain).abs().max()) > 0.2 * float(plain.abs().max())
    layers = latent_layers(H, D, V, rank, scale, dtype, t)
    for cuts in ([50], [2, 3, 1, 30, 14], [45] + [1] * 5, [33, 17]):
        close(latent_run(layers, t, q, kv, cuts), want, 2e-5 if dtype == torch.float32 else 3e-2, cuts[:2])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_latent_attention_finds_one_far_key(dtype):
    """One latent among a thousand matches one query, which is decoded (its keys shared out to several
    workgroups) or in a prompt; the sink takes what the match leaves."""
    H, D, V, rank, scale, n = 4, 32, 32, 64, 0.2, 1050
    t, q, kv = latent_case(n, H, D, V, rank, 3, dtype, torch.tensor([-4.0, 0.0, 4.0, 9.0]))
    q = q * 0.1
    t["uk"][:, 7] *= 4.0
    for j in (0, 15, 16, 511, 1040):
        qq, kk = q.clone(), kv.clone()
        kk[:, 7], kk[j] = 0.0, 0.02
        kk[j, 7] = 9.0
        c = R.rms_norm(kk[j].to(F), t["dkv.norm"].to(F), 1e-5)
        key = (t["uk"].to(F) @ c).view(H, D)
        qq[n - 1] = (key / key.norm(dim=1, keepdim=True)**2 * 75).reshape(-1).to(dtype)       # a score of 15
        want = latent_want(t, qq, kk, H, D, V, scale)
        val = (t["uv"].to(F) @ c).view(H, V)
        assert float((want[n - 1].view(H, V) - val)[:3].abs().max()) < 0.1 * float(val.abs().max())
        layers = latent_layers(H, D, V, rank, scale, dtype, t)
        for cuts in ([n], [n - 1, 1], [600, n - 602, 2]):
            got = latent_run(layers, t, qq, kk, cuts, 16)
            close(got[n - 20:], want[n - 20:], 2e-5 if dtype == torch.float32 else 3e-2, (j, cuts))


# ----------------------------------------------------------------------------- experts
@pytest.mark.parametrize("experts,groups,keep,top", [(15, 5, 2, 4), (8, 8, 3, 3), (6, 1, 1, 2), (9, 3, 1, 3), (70, 7, 4, 5),
                                                     (128, 64, 2, 4), (5, 5, 5, 5), (256, 8, 4, 8)])
def test_router_among_groups(experts, groups, keep, top):
    """Only experts of the best groups can be chosen; weights are the scores over all experts times the
    scale.  Formed by the kernel (aligned and unaligned rows) and from given logits."""
    from vllm_legacy_amd import _seq_ops as ops
    T = 40
    for W in (64, 50):
        h, router = rnd((T, W), 0), rnd((experts, W), 1, 2 * W**-0.5)
        z = h.to(F) @ router.to(F).T
        s = torch.softmax(z, -1)
        idx = torch.stack([R.choose(s[i], top, groups, keep) for i in range(T)])
        for logits in (None, z.float().to(DEV)):
            e, w, _ = ops.moe_route(h.to(DEV), router.to(DEV), None, None, top, logits, renormalize=False, groups=groups,
                                    keep_groups=keep, weight_scale=1.9)
            assert torch.equal(e.cpu().long(), idx)
            close(w, 1.9 * s.gather(1, idx), 3e-6)
    if keep < groups and keep * (experts // groups) > top:
        assert not torch.equal(idx, torch.topk(s, top, -1).indices)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows", [3, 300])
def test_grouped_experts_block(dtype, rows):
    from vllm_legacy_amd.routed_experts import RoutedExperts
    W, E, top, ff = 64, 6, 2, 24
    moe = RoutedExperts(W, E, 0, top, ff, act="silu", dtype=dtype, device=DEV, gated=True, renormalize=False, groups=3,
                        keep_groups=2, weight_scale=1.7)
    t = {"router": rnd((E, W), 1, 2 * W**-0.5)}
    for e in range(E):
        t.update({f"e{e}.gate": rnd((ff, W), 10 + e, W**-0.5), f"e{e}.up": rnd((ff, W), 20 + e, W**-0.5),
                  f"e{e}.down": rnd((W, ff), 30 + e, ff**-0.5)})
    t = {k: v.to(torch.bfloat16) for k, v in t.items()}
    moe.set_weights(t)
    h = rnd((rows, W), 5).to(dtype)
    want = R.routed_ff(h.to(F), {k: v.to(F) for k, v in t.items()}, R.moe_mlp(E, top, ff, (3, 2), 1.7))
    err = (moe(h.to(DEV)).cpu().to(F) - want).abs().amax(1) / want.abs().max()
    if dtype == torch.float32:
        assert float(err.max()) <= 2e-5
    else:       # a close call of the router may go the other way for a few rows
        assert float(torch.quantile(err, 0.9)) <= 2e-2
    with pytest.raises(ValueError):
        RoutedExperts(W, E, 0, 3, ff, dtype=dtype, device=DEV, groups=3, keep_groups=1)


# ----------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("name", list(configs()))
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_whole_prompt_portions_and_decoding_agree_with_the_reference(tmp_path, name, dtype):
    s = Served(tmp_path, name, dtype)
    n = 90 if name == "mfma" else 41
    toks = tokens_of(s.cfg, n, 1)
    want = s.reference(toks)

    def run(sizes, sid):
        got, lo, i = [], 0, 0
        while lo < n:
            c = min(sizes[i % len(sizes)], n - lo)
            got.append(s.step([(sid, toks[lo:lo + c])])[sid])
            lo += c
            i += 1
        s.end(sid)
        return torch.cat(got)

    for sid, sizes in (("whole", [n]), ("portions", [2, 3, 4, 5, 1, 7, 2]), ("prefill+decode", [n - 12] + [1] * 12),
                       ("long portions", [33, 40, 5]), ("tokens", [1])):
        within(logit_error(run(sizes, sid), want), dtype, sid)


@pytest.mark.parametrize("name", ["plain", "odd", "equal", "edges", "ragged"])
def test_layer_by_layer_against_the_reference(tmp_path, name):
    """The stream after every layer, float32."""
    s = Served(tmp_path, name, torch.float32)
    toks = tokens_of(s.cfg, 17, 4)
    taps = []
    R.forward(s.cfg, s.W, toks, taps)
    s.cache.admit("a")
    s.cache.grow("a", 17)
    batch = make_batch([17], [0], 4, tables=[s.cache.block_table("a")], slots=[s.cache.state_slot("a")])
    got = []
    with torch.inference_mode():
        s.model(torch.tensor(toks, device=DEV), batch.positions, s.runner.caches, batch,
                tap=lambda i, x: got.append(x.detach().cpu().clone()))
    assert len(got) == len(taps) == len(s.cfg["layers"])
    for i, (a, b) in enumerate(zip(got, taps)):
        assert float((a.to(F) - b).abs().max() / b.abs().max()) <= 2e-5, i


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_mixed_batches_with_pages_and_slots_used_again(tmp_path, dtype):
    """Three slots, a pool that cannot hold all five requests at once: requests end, their
    pages and slots go to later ones; every step mixes portions and single tokens."""
    s = Served(tmp_path, "plain", dtype, num_blocks=30, block_size=4, num_slots=3)
    reqs = {k: tokens_of(s.cfg, n, i) for i, (k, n) in enumerate([("a", 45), ("b", 9), ("c", 30), ("d", 38), ("e", 2)])}
    plan = [
        [("a", 5), ("b", 2)],
        [("a", 16), ("b", 1), ("c", 2)],
        [("b", 1), ("c", 7), ("a", 1)],
        [("a", 9), ("b", 5), ("c", 1)],          # b ends here (9 tokens)
        [("d", 3), ("a", 1), ("c", 13)],         # d takes b's slot and pages
        [("d", 1), ("a", 13), ("c", 7)],         # a and c end
        [("d", 30), ("e", 1)],
        [("e", 1), ("d", 1)],
        [("d", 3)],
    ]
    got = {k: [] for k in reqs}
    at = {k: 0 for k in reqs}
    used_slots = {}
    for step in plan:
        entries = [(k, reqs[k][at[k]:at[k] + n]) for k, n in step]
        out = s.step(entries)
        for k, n in step:
            used_slots.setdefault(k, s.cache.state_slot(k))
            got[k].append(out[k])
            at[k] += n
            if at[k] == len(reqs[k]):
                s.end(k)
    assert at == {k: len(v) for k, v in reqs.items()}
    assert used_slots["d"] == used_slots["b"] and len(set(used_slots.values())) == 3
    for k in reqs:
        s.check(torch.cat(got[k]), reqs[k], k)


@pytest.mark.parametrize("name", ["plain", "edges"])
def test_long_decoding_over_many_pages(tmp_path, name):
    """Windows and pages begin and end many times among decoded tokens."""
    s = Served(tmp_path, name, torch.float32, num_blocks=80, block_size=4)
    toks = tokens_of(s.cfg, 200, 8)
    got = [s.step([("a", toks[:3])])["a"]]
    for t in range(3, 200):
        got.append(s.step([("a", toks[t:t + 1])])["a"])
    s.check(torch.cat(got), toks)


def test_long_prompts_beside_a_decoding_request(tmp_path):
    """Prompts of several hundred tokens (blocks and pieces of the recurrences, windows well inside), whole and in large
    portions beside a decoding request, in bfloat16 on the matrix cores."""
    s = Served(tmp_path, "mfma", torch.bfloat16, num_blocks=100, block_size=16)
    a, b = tokens_of(s.cfg, 300, 5), tokens_of(s.cfg, 560, 6)
    got_a = [s.step([("a", a[:290])])["a"]] + [s.step([("a", a[t:t + 1])])["a"] for t in range(290, 300)]
    s.check(torch.cat(got_a), a, "whole + decode")
    s.end("a")
    got_b = [s.step([("b", b[:257])])["b"], s.step([("b", b[257:554]), ("a", a[:3])])["b"]]
    got_b += [s.step([("b", b[t:t + 1])])["b"] for t in range(554, 560)]
    s.check(torch.cat(got_b), b, "portions + decode")


def test_a_batch_does_not_change_a_request(tmp_path):
    """The same request alone and beside two others: equal beyond rounding (float32)."""
    s = Served(tmp_path, "odd", torch.float32)
    a, b, c = (tokens_of(s.cfg, n, i) for i, n in enumerate((33, 12, 50)))
    alone = torch.cat([s.step([("a", a[:20])])["a"], s.step([("a", a[20:])])["a"]])
    s.end("a")
    s.step([("c", c[:41])])
    first = s.step([("b", b[:5]), ("a", a[:20]), ("c", c[41:42])])["a"]
    second = s.step([("c", c[42:43]), ("a", a[20:]), ("b", b[5:])])["a"]
    both = torch.cat([first, second])
    assert float(logit_error(both, alone).max()) <= 1e-5


def greedy_reference(s, prompt, n):
    """(tokens, how clear each choice was): a choice closer than the bar is a tie."""
    toks, margins = list(prompt), []
    for _ in range(n):
        last = s.reference(toks)[-1]
        top = torch.topk(last, 2).values
        margins.append(float(top[0] - top[1]))
        toks.append(int(torch.argmax(last)))
    return toks[len(prompt):], margins


@pytest.mark.parametrize("num_blocks,preempt", [(64, False), (9, True)])
def test_greedy_generation_through_the_engine(tmp_path, num_blocks, preempt):
    from vllm_legacy_amd.engine import EngineConfig, LLMEngine, SamplingParams
    s = Served(tmp_path, "plain", torch.float32)
    engine = LLMEngine(s.model, EngineConfig(block_size=4, num_blocks=num_blocks, max_num_seqs=3,
                                             max_num_batched_tokens=7), DEV)
    prompts = [tokens_of(s.cfg, n, 20 + n) for n in (11, 3, 6, 1)]
    outs = engine.generate(prompts, SamplingParams(max_tokens=8))
    assert (engine.scheduler.num_preemptions > 0) == preempt
    assert engine.cache.free_blocks == num_blocks and engine.cache.free_slots == 3
    for p, o in zip(prompts, outs):
        want, margins = greedy_reference(s, p, 8)
        assert o.finished and o.finish_reason == "length" and len(o.token_ids) == 8
        for t, (a, b, m) in enumerate(zip(o.token_ids, want, margins)):
            if m < 1e-3:
                break                      # a tie within rounding: what follows may differ
            assert a == b, (t, a, b)


def test_generation_from_a_folder_and_the_command_line(tmp_path):
    """LLMEngine.from_pretrained picks the model class by config.json; the command line prints the
    same greedy tokens."""
    from vllm_legacy_amd.engine import EngineConfig, LLMEngine, SamplingParams
    s = Served(tmp_path, "equal", torch.float32)
    engine = LLMEngine.from_pretrained(s.folder, torch.float32, EngineConfig(block_size=4, num_blocks=40, max_num_seqs=2), DEV)
    assert type(engine.runner.model).__name__ == "DagavikForCausalLM"
    p = tokens_of(s.cfg, 7, 3)
    first = engine.generate([p], SamplingParams(max_tokens=6))[0].token_ids
    out = engine.generate([p], SamplingParams(max_tokens=6, stop_token_ids=[first[2]]))[0]
    assert out.finish_reason == "stop" and out.token_ids == first[:first.index(first[2]) + 1]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, "-m", "vllm_legacy_amd.engine.cli", "generate", "--model", s.folder, "--dtype",
                        "float32", "--prompt", ",".join(map(str, p)), "--max-tokens", "6", "--num-blocks", "64"],
                       cwd=root, capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert json.loads(r.stdout.strip().splitlines()[-1])["token_ids"] == first


def test_trace_replayer_as_a_program(tmp_path):
    """bin/trace_run fed four steps (two requests, a portion beside a single token, a request that
    ends and whose id comes back as a new request) writes the logits the reference gives."""
    s = Served(tmp_path, "odd", torch.float32)
    a, b = tokens_of(s.cfg, 9, 1), tokens_of(s.cfg, 4, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:6], "want": [0, 5]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[6:7], "want": []}, {"id": "b", "tokens": b[:3], "want": [2]}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[3:], "want": [0]}, {"id": "a", "tokens": a[7:], "want": [1]}], "end": ["a", "b"]},
        {"step": 3, "entries": [{"id": "a", "tokens": b, "want": [3]}], "end": ["a"]},
    ]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", s.folder, "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "128"], input="\n".join(json.dumps(x) for x in steps) + "\n",
                       capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    import numpy as np
    ra, rb = s.reference(a), s.reference(b)
    V = s.cfg["vocab"]
    want = {0: ra[[0, 5]], 1: rb[[2]], 2: torch.stack([rb[3], ra[8]]), 3: rb[[3]]}
    for n, w in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, V))
        assert got.shape == w.shape and float(logit_error(got, w).max()) <= 1e-4, n
