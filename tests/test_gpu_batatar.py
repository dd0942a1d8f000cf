"""Batatar through the framework -- registry, checkpoint loader, cache manager, model runner,
scheduler, sampler -- and its mechanisms one by one, against the float64 reference of
tests/batatar_oracle.py on small random models and inputs.

Mechanisms alone: the stream update with a scale, without a norm and with two normed branches; head
norms in the cache write; chunked attention with a sink and a score cap (random inputs in many sizes
and cuts; one planted key just inside and just outside a chunk, at page borders, in prompts and in
decoding; the plain kernel against the matrix-core kernels; chunks together with windows and kept
tokens); the recurrence with constant and with per-token decays (token by token, in blocks and in
pieces, mixed runs, far tokens, decays near 0 and 1, slots that hold anything); the gated norm over
parts; the state-space layer with its convolution across cuts; experts with sigmoid scores and
weighted inputs.
Whole models: prompts whole, in portions down to two tokens and token by token; mixed batches with
pages and slots used again; long decoding; a batch does not change a request; greedy generation
through LLMEngine and the command line; the trace replayer as a program.  The float32 bar is
float32 rounding through the stack and is the one that finds faults of cutting, batching and
reuse: both number formats run the same code paths except the matrix-core attention kernels, which
the bfloat16 runs cover with a looser bar."""
import json
import os
import subprocess
import sys

import pytest
import torch

from tests import batatar_oracle as R

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F = R.F
BAR = {torch.float32: 1e-4, torch.bfloat16: 0.2}
MEAN_BAR = {torch.float32: 1e-4, torch.bfloat16: 0.06}


def configs():
    L, P, E = R.lightning_layer, R.parallel_layer, R.moe_mlp
    return {
        "plain": R.make_config([
            L(4, 16, mlp=E(6, 2, 24)),
            P((4, 2, 16, 16, 9, 12.0), (4, 16, 8, 2, 2, 4), mlp=E(4, 1, 32)),
            L(2, 16, 24, [0.9, 0.995], mlp=E(3, 1, 40)),
            P((2, 1, 24, 16, 14, 30.0), (2, 24, 16, 1, 1, 3), mlp=None)], loop=(1, 3, 2)),
        # sizes that are neither equal nor powers of two; one key head, vdim != dim, groups and the norm's
        # parts unequal, a scale that is not dim^-1/2, three passes over everything but the last layer,
        # a feed-forward missing, the parallel layer first, one decay for all heads
        "odd": R.make_config([
            P((3, 1, 12, 20, 7, 6.0, 0.5), (6, 10, 14, 3, 5, 3), mlp=E(5, 3, 20)),
            L(3, 12, 20, [0.25, 0.8, 0.999], mlp=None),
            L(5, 6, 10, 0.93, mlp=E(7, 2, 14))], vocab=131, width=40, eps=1e-3, residual_mult=1.3, loop=(0, 2, 3)),
        # key heads = heads, a group per head, one part, every expert chosen, no loop, a convolution of one
        # tap, a multiplier of one, decays of 0 and 1
        "equal": R.make_config([P((2, 2, 16, 16, 16, 8.0), (2, 16, 16, 2, 1, 1), mlp=E(3, 3, 16)),
                                L(2, 16, 16, [0.0, 1.0], mlp=E(2, 2, 16)),
                                P((4, 4, 8, 8, 8, 4.0), (4, 8, 8, 4, 4, 2), mlp=E(1, 1, 16))], residual_mult=1.0),
        # chunks of one token and of more tokens than any request has; one pass; one head
        "edges": R.make_config([P((2, 1, 8, 8, 1, 5.0), (1, 32, 4, 1, 8, 6), mlp=E(2, 1, 24)),
                                P((1, 1, 40, 12, 500, 25.0), (3, 4, 20, 1, 3, 4), mlp=E(3, 2, 20)),
                                L(1, 8, 40, [0.97], mlp=None)], width=48, loop=(1, 2, 1)),
        # nothing a multiple of four: widths, head sizes, state sizes, vocabulary, expert sizes
        "ragged": R.make_config([
            P((3, 3, 10, 14, 11, 9.0), (5, 6, 9, 5, 2, 3), mlp=E(5, 2, 18)),
            L(3, 7, 11, mlp=E(4, 4, 6)),
            P((6, 2, 22, 5, 6, 20.0), (3, 7, 5, 1, 3, 5), mlp=E(3, 1, 30))], vocab=101, width=50, loop=(1, 3, 2)),
        # sizes for the matrix-core kernels: multiples of 32, many heads, wide values
        "mfma": R.make_config([
            L(4, 64, 128, mlp=E(6, 2, 32)),
            P((8, 2, 32, 64, 45, 15.0), (4, 96, 32, 2, 4, 4), mlp=E(8, 1, 64)),
            P((4, 4, 64, 32, 70, 30.0), (2, 64, 128, 1, 1, 4), mlp=None),
            L(2, 96, 32, [0.9, 0.998], mlp=E(4, 3, 32))], width=128, loop=(2, 4, 2)),
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


# ----------------------------------------------------------------------------- row-wise layers
@pytest.mark.parametrize("width", [40, 256, 2500])
@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
def test_stream_update_scaled_and_with_two_branches(width, out_dtype):
    """x += m y (no norm), and x += m (N(y) w + N(y2) w2), each followed by the next norm; a row added in
    the same launch; rows of the branches are views of wider matrices."""
    from vllm_legacy_amd import _seq_ops as ops
    x, y, y2, row = rnd((5, width), 1), rnd((5, width), 2, 3.0), rnd((5, width), 3, 0.2), rnd((width, ), 4)
    w, w2, wn = (1 + 0.3 * rnd((width, ), s) for s in (5, 6, 7))
    tol = 3e-6 if out_dtype == torch.float32 else 6e-3
    for branches in (1, 2):
        if branches == 1:
            want = x.to(F) + 0.7 * y.to(F) + row.to(F)
        else:
            want = x.to(F) + 0.35 * (R.rms_norm(y.to(F), w.to(F), 1e-3) + R.rms_norm(y2.to(F), w2.to(F), 1e-3)) + row.to(F)
        xs, h = x.to(DEV).clone(), torch.empty((5, width), dtype=out_dtype, device=DEV)
        both = torch.cat([y, y2], 1).to(DEV)
        if branches == 1:
            ops.residual_norms(xs, both[:, :width], add_row=row.to(DEV), out=h, pre_weight=wn.to(DEV), eps=1e-3, y_scale=0.7)
        else:
            ops.residual_norms(xs, both[:, :width], None, w.to(DEV), None, row.to(DEV), h, wn.to(DEV), 1e-3, 0.35,
                               both[:, width:], w2.to(DEV))
        close(xs, want, 3e-6, branches)
        close(h, R.rms_norm(want, wn.to(F), 1e-3), tol, branches)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n,groups", [(48, 1), (48, 3), (50, 5), (4096, 8), (9000, 1), (6, 6), (2052, 3)])
@pytest.mark.parametrize("gate_first", [True, False])
def test_gated_norm_over_parts(dtype, n, groups, gate_first):
    """silu(gate) ahead of the norm or sigmoid(gate) behind it; parts of unequal size of values (a norm over
    the whole row would give something else); aligned rows and rows that are not."""
    from vllm_legacy_amd import _seq_ops as ops
    o = rnd((3, n), 1) * (1 + torch.arange(groups).repeat_interleave(n // groups).float())
    w = 1 + 0.2 * rnd((n, ), 2)
    wide = rnd((3, n + 9), 3, 1.5).to(dtype)
    for first in (0, 1, 8):
        z = wide[:, first:first + n]
        zf = z.to(F)
        want = R.grouped_gated_norm(o.to(F), zf, w.to(F), groups, 1e-5) if gate_first else \
            R.unit_rms(o.to(F).view(3, groups, -1), 1e-5).reshape(3, n) * w.to(F) * torch.sigmoid(zf)
        out = torch.full((3, n + 16), 7.0, dtype=dtype, device=DEV)
        ops.gated_group_rms_norm(out[:, first:first + n], o.to(DEV), w.to(DEV), wide.to(DEV)[:, first:first + n],
                                 "silu" if gate_first else "sigmoid", gate_first, groups, 1e-5)
        close(out[:, first:first + n], want, 3e-6 if dtype == torch.float32 else 6e-3, first)
        assert bool((out[:, :first] == 7.0).all()) and bool((out[:, first + n:] == 7.0).all())


# ----------------------------------------------------------------------------- chunked attention with a sink
def attention_spec(H, G, D, V, chunk, softcap=0.0, scale=None):
    return {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": D**-0.5 if scale is None else scale,
            "softcap": softcap, "mask": {"size": chunk}}


def attention_reference(spec, q, k, v, sink=True, eps=1e-5, norm=True):
    q, k = q.to(F), k.to(F)
    if norm:
        q, k = R.unit_rms(q, eps), R.unit_rms(k, eps)
    return R.attention_core(q, k, v.to(F), spec["scale"], spec["softcap"], spec["mask"]["size"], sink), k


def run_attention(spec, q, k, v, cuts, dtype, block_size=4, keys_out=None, norm=True, sink=0.0):
    """One sequence through RotaryKVAttention in steps of the given sizes; pages in a scrambled
    order.  Returns [n, H, V] fp32 on the CPU."""
    from vllm_legacy_amd.attention.backends.rotary_kv import RotaryKVAttention
    H, G, D, V = spec["heads"], spec["kv_heads"], spec["dim"], spec["vdim"]
    n = q.shape[0]
    layer = RotaryKVAttention(H, G, D, V, spec["scale"], 0, 1.0, device=DEV, softcap=spec["softcap"], norm_eps=1e-5,
                              norm_heads=norm, chunk=spec["mask"]["size"] or None, sink_score=sink)
    pages = (n + block_size - 1) // block_size
    order = torch.randperm(pages + 3, generator=torch.Generator().manual_seed(1)).tolist()
    ks, vs = RotaryKVAttention.get_cache_shapes(pages + 3, block_size, G, D, V)
    kc = torch.full(ks, float("nan"), dtype=dtype, device=DEV)      # a read of an unwritten place shows
    vc = torch.full(vs, float("nan"), dtype=dtype, device=DEV)
    outs, at = [], 0
    for c in cuts:
        c = min(c, n - at)
        if c <= 0:
            break
        batch = make_batch([c], [at], block_size, tables=[order[:pages]])
        qq = q[at:at + c].reshape(c, H * D).to(dtype).to(DEV).clone()
        kk = k[at:at + c].reshape(c, G * D).to(dtype).to(DEV)
        vv = v[at:at + c].reshape(c, G * V).to(dtype).to(DEV)
        out = torch.empty((c, H * V), dtype=dtype, device=DEV)
        layer(out, qq, kk, vv, None, kc, vc, batch)
        outs.append(out.float().cpu().view(c, H, V))
        at += c
    assert at == n
    if keys_out is not None:
        rows = torch.tensor([order[j // block_size] * block_size + j % block_size for j in range(n)])
        keys_out.append(kc.view(-1, G, D)[rows.to(DEV)].float().cpu())
    return torch.cat(outs)


ATTN_SHAPES = [
    # H, G, D, V, chunk, softcap
    (4, 2, 16, 16, 9, 10.0),
    (3, 1, 24, 12, 5, 0.0),
    (6, 3, 8, 20, 70, 4.0),
    (2, 2, 40, 6, 1, 25.0),
    (5, 1, 7, 9, 16, 3.0),
    (10, 2, 32, 64, 20, 12.0),
    (2, 1, 96, 64, 33, 8.0),
    (8, 1, 64, 32, 64, 0.0),
    (5, 5, 128, 128, 17, 30.0),
    (4, 2, 32, 96, 0, 6.0),
    (6, 2, 64, 32, 60, 18.0),
    (40, 1, 32, 32, 32, 5.0),
]


@pytest.mark.parametrize("shape", ATTN_SHAPES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_attention_prompt_portions_and_decoding(shape, dtype):
    """Scores around zero, so that the sink takes a visible share; every key has a value level of its
    own, so a chunk that is one off moves the output."""
    H, G, D, V, chunk, cap = shape
    spec = attention_spec(H, G, D, V, chunk, cap, 1.3 * D**-0.5)
    n = 75
    q, k, v = rnd((n, H, D), 0, 1.7), rnd((n, G, D), 1, 1.7), rnd((n, G, V), 2)
    q[:, 0] *= 4.0               # heads of unequal size: a norm of the whole row would give something else
    k[:, -1] *= 5.0
    v += (torch.arange(n).float() % 7)[:, None, None] * 3.0
    if dtype == torch.bfloat16:
        q, k, v = (t.to(dtype).float() for t in (q, k, v))
    want, want_k = attention_reference(spec, q, k, v)
    if chunk:
        for other in (chunk + 1, chunk - 1):
            off, _ = attention_reference(attention_spec(H, G, D, V, other, cap, spec["scale"]), q, k, v)
            assert other == 0 or float((want - off).abs().max()) > 0.05
    plain, _ = attention_reference(spec, q, k, v, sink=False)
    assert float((want - plain).abs().max()) > 0.3           # the sink shows
    bar = 3e-5 if dtype == torch.float32 else 0.03
    for cuts in ([n], [2, 3, 4, 5, 1, 7, 2] * 5, [40] + [1] * 35, [33, 35, 7], [1] * n):
        keys = []
        got = run_attention(spec, q, k, v, cuts, dtype, keys_out=keys)
        assert float((got - want).abs().max()) <= bar * float(want.abs().max()), (cuts[:3], float((got - want).abs().max()))
        close(keys[0], want_k, 1e-5 if dtype == torch.float32 else 1e-2, "keys")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_scores_far_below_and_above_the_sink(dtype):
    """Keys whose scores are all far below the sink's leave almost nothing; a sink with a score of its
    own; a row whose scores are far above it is a plain softmax."""
    n, H, D = 40, 2, 32
    spec = attention_spec(H, 1, D, D, 0)
    q, k, v = rnd((n, H, D), 0, 0.2), rnd((n, 1, D), 1, 0.2), 1 + rnd((n, 1, D), 2, 0.1)
    q[:, :, 0], k[:, :, 0] = 10.0, -3.0         # every score about -5.3
    q[20:, :, 0] = -90.0                        # and about 47 from row 20 on
    if dtype == torch.bfloat16:
        q, k, v = (t.to(dtype).float() for t in (q, k, v))
    want, _ = attention_reference(spec, q, k, v, norm=False)
    assert 0.0 < float(want[0].max()) < 0.02 and float(want[20:].min()) > 0.5
    bar = 3e-5 if dtype == torch.float32 else 0.03
    for cuts in ([n], [17, 2, 9] + [1] * 12):
        got = run_attention(spec, q, k, v, cuts, dtype, norm=False)
        assert float((got - want).abs().max()) <= bar
        assert float((got[:20] - want[:20]).abs().max()) <= bar * float(want[:20].abs().max())
    # a sink of score s is the same as all other scores lowered by s (no cap)
    s = attention_reference(spec, q, k, v, norm=False)[0]
    kk, qq = torch.cat([k, torch.ones(n, 1, 1)], 2), torch.cat([q, torch.full((n, H, 1), -2.0 * D**0.5)], 2)
    lowered = R.attention_core(qq.to(F), kk.to(F), v.to(F), D**-0.5)
    got = run_attention(spec, q, k, v, [n - 3, 1, 1, 1], dtype, norm=False, sink=2.0)
    assert float((got - lowered).abs().max()) <= bar and float((lowered - s).abs().max()) > 0.05


def planted(spec, n, rows, key, dtype, seed=0):
    """Random q, k, v in which the queries `rows` and the key `key` share one large coordinate, and the
    key's value is a level nobody else has: if the key is visible it takes the whole weight, if not
    the output stays with the others."""
    H, G, D, V = spec["heads"], spec["kv_heads"], spec["dim"], spec["vdim"]
    q, k, v = rnd((n, H, D), seed, 0.3), rnd((n, G, D), seed + 1, 0.3), rnd((n, G, V), seed + 2)
    q[rows, :, D - 1] = 30.0
    k[key, :, D - 1] = 30.0
    v[key] = 40.0
    if dtype == torch.bfloat16:
        q, k, v = (t.to(dtype).float() for t in (q, k, v))
    return q, k, v


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("dim,block_size", [(16, 4), (64, 16)])
@pytest.mark.parametrize("case", ["chunk_first", "chunk_before", "chunk_last", "page_edge", "start"])
def test_one_key_at_the_edges_of_a_chunk(dtype, dim, block_size, case):
    """A chunk's first key seen by all of the chunk's rows and by none of the next chunk's; the key right
    before a chunk (not seen from it); a chunk's last key seen by itself only; a key on a page's last
    place; the sequence's first token.  In a prompt, in portions and in decoded rows; 16-bit runs take
    the matrix-core kernels at dim 64."""
    chunk, n = 37, 300
    spec = attention_spec(4, 2, dim, dim, chunk, 50.0, 2.0)
    edge = 7 * chunk                    # 259: the last whole chunk starts here
    key, rows = {"chunk_first": (edge, range(edge, n)), "chunk_before": (edge - 1, range(edge - 6, n)),
                 "chunk_last": (edge + chunk - 1, range(edge + chunk - 8, n)),
                 "page_edge": (n - 20 - (n - 20) % block_size - 1, range(n - 20, n)), "start": (0, range(0, n))}[case]
    rows = list(rows)
    q, k, v = planted(spec, n, rows, key, dtype)
    want, _ = attention_reference(spec, q, k, v)
    seen = 0
    for r in rows:
        vis = key <= r and r // chunk == key // chunk
        seen += vis
        assert (float(want[r].mean(-1).min()) > 35.0) == vis and (float(want[r].mean(-1).max()) < 8.0) == (not vis), (case, r)
    assert 0 < seen < len(rows) or case == "page_edge"
    bar = 3e-5 if dtype == torch.float32 else 0.03
    for cuts in ([n], [n - 45] + [1] * 45, [100, 3, 155, 2, 2, 38], [edge - 1, 2, 2] + [17] + [1] * 30, [edge, n - edge]):
        got = run_attention(spec, q, k, v, cuts, dtype, block_size=block_size)
        assert float((got - want).abs().max()) <= bar * float(want.abs().max()), (case, cuts[:2])


def test_plain_and_matrix_core_kernels_agree():
    """bfloat16 through the kernel every dtype can take and through the matrix-core kernels."""
    from vllm_legacy_amd import _seq_ops as ops
    spec = attention_spec(8, 2, 96, 64, 45, 9.0)
    n = 131
    q, k, v = (t.to(torch.bfloat16).float() for t in (rnd((n, 8, 96), 0, 1.5), rnd((n, 2, 96), 1, 1.5), rnd((n, 2, 64), 2)))
    fast = run_attention(spec, q, k, v, [90, 3] + [1] * 38, torch.bfloat16)
    ops.set_kv_attention_kernel(1)
    try:
        plain = run_attention(spec, q, k, v, [90, 3] + [1] * 38, torch.bfloat16)
    finally:
        ops.set_kv_attention_kernel(0)
    assert float((fast - plain).abs().max()) <= 0.03 * float(plain.abs().max())
    assert not torch.equal(fast, plain)          # two kernels did run


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_chunks_beside_windows_kept_tokens_rotation_and_gates(dtype):
    """The terms of the attention layer together: a row sees its chunk's keys of its window and the
    sequence's first tokens; heads are normed ahead of a rotation; one gate per head."""
    from vllm_legacy_amd.attention.backends.rotary_kv import RotaryKVAttention
    n, H, G, D, chunk, window, keep = 70, 4, 2, 32, 23, 9, 2
    q, k, v, gate = rnd((n, H, D), 0, 2.0), rnd((n, G, D), 1, 2.0), rnd((n, G, D), 2), rnd((n, H), 3)
    if dtype == torch.bfloat16:
        q, k, v, gate = (t.to(dtype).float() for t in (q, k, v, gate))
    ang = torch.arange(n).to(F)[:, None] * 100.0**(-torch.arange(0, 16, 2).to(F) / 16)
    c, s = torch.cos(ang)[:, None], torch.sin(ang)[:, None]

    def turned(u):                       # pairs (2i, 2i + 1) of the first 16 elements
        u = R.unit_rms(u.to(F), 1e-5)
        a, b = u[..., 0:16:2], u[..., 1:16:2]
        return torch.cat([torch.stack([a * c - b * s, b * c + a * s], -1).flatten(-2), u[..., 16:]], -1)

    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    ok = (j <= i) & (((i - j < window) & (i // chunk == j // chunk)) | (j < keep))
    qq, kk, vv = turned(q), turned(k).repeat_interleave(2, 1), v.to(F).repeat_interleave(2, 1)
    sc = (torch.einsum("ihd,jhd->hij", qq, kk) * 0.4).masked_fill(~ok, float("-inf"))
    want = torch.einsum("hij,jhv->ihv", R.sink_softmax(sc), vv) * torch.sigmoid(gate.to(F))[:, :, None]
    layer = RotaryKVAttention(H, G, D, D, 0.4, 16, 100.0, window=window, device=DEV, keep_first=keep, norm_eps=1e-5,
                              norm_heads=True, chunk=chunk, sink_score=0.0)
    for cuts in ([n], [30, 2, 20] + [1] * 18):
        ks, vs = RotaryKVAttention.get_cache_shapes(20, 4, G, D, D)
        kc, vc = (torch.full(t, float("nan"), dtype=dtype, device=DEV) for t in (ks, vs))
        at, outs = 0, []
        for m in cuts:
            batch = make_batch([m], [at], 4, tables=[list(range(18, 0, -1))])
            out = torch.empty((m, H * D), dtype=dtype, device=DEV)
            layer(out, q[at:at + m].reshape(m, -1).to(dtype).to(DEV), k[at:at + m].reshape(m, -1).to(dtype).to(DEV),
                  v[at:at + m].reshape(m, -1).to(dtype).to(DEV), gate[at:at + m].to(dtype).to(DEV), kc, vc, batch)
            outs.append(out.float().cpu().view(m, H, D))
            at += m
        got = torch.cat(outs)
        assert float((got - want).abs().max()) <= (3e-5 if dtype == torch.float32 else 0.03) * float(want.abs().max())


# ----------------------------------------------------------------------------- recurrences
@pytest.fixture(params=[0, 1, 2], ids=["by_run", "token_by_token", "in_blocks"])
def scan_kernel(request):
    from vllm_legacy_amd import _seq_ops as ops
    ops.set_decay_scan_kernel(request.param)
    yield request.param
    ops.set_decay_scan_kernel(0)


def run_scan(shape, seqs, plan, dtype, act, decay=None, dt=None, dt_bias=None, a_log=None, skip=None, slots=None):
    """seqs: name -> (q [n, G, D], k, v [n, H, V]); plan: steps of [(name, rows)]; slots of the state start
    as NaN (or hold what an earlier sequence left).  Returns name -> [n, H, V]."""
    from vllm_legacy_amd import _seq_ops as ops
    H, G, D, V = shape
    names = list(seqs)
    slots = slots or {k: i for i, k in enumerate(names)}
    state = torch.full((max(slots.values()) + 1, H, D, V), float("nan"), device=DEV)
    at, got = {k: 0 for k in names}, {k: [] for k in names}

    def rows(i, step):
        return torch.cat([seqs[k][i][at[k]:at[k] + n].reshape(n, -1) for k, n in step]).to(dtype)

    for step in plan:
        batch = make_batch([n for _, n in step], [at[k] for k, _ in step], 4, slots=[slots[k] for k, _ in step])
        q, k, v = (rows(i, step) for i in range(3))
        wide = torch.cat([q, k, v], 1).to(DEV)          # views of one projection
        T = wide.shape[0]
        dts = None if dt is None else torch.cat([dt[k][at[k]:at[k] + n] for k, n in step]).to(dtype).to(DEV)
        o = torch.full((T, H * V), float("nan"), device=DEV)
        ops.decay_scan(o, wide[:, :G * D], wide[:, G * D:2 * G * D], wide[:, 2 * G * D:], state, batch.query_start_loc,
                       batch.context_lens, batch.state_slots, G, batch.max_query_len,
                       None if decay is None else torch.log(decay.to(F)).float().to(DEV), dts,
                       None if dt_bias is None else dt_bias.to(DEV), None if a_log is None else a_log.to(DEV),
                       None if skip is None else skip.to(DEV), act)
        o = o.cpu().view(T, H, V)
        lo = 0
        for k_, n in step:
            got[k_].append(o[lo:lo + n])
            lo += n
            at[k_] += n
    assert all(at[k] == seqs[k][0].shape[0] for k in names)
    return {k: torch.cat(v) for k, v in got.items()}


SCAN_SHAPES = [(4, 4, 16, 16), (3, 3, 12, 20), (6, 2, 9, 14), (2, 2, 64, 64), (4, 1, 32, 48), (2, 2, 96, 128),
               (2, 1, 128, 100), (1, 1, 5, 3), (2, 2, 200, 24), (3, 3, 48, 65)]


@pytest.mark.parametrize("shape", SCAN_SHAPES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_recurrence_with_constant_decays(shape, dtype, scan_kernel):
    """Sequences of unequal lengths, portions and single tokens together, a slot taken over from a
    sequence that ended; the inputs pass silu."""
    H, G, D, V = shape
    decay = torch.linspace(0.3, 0.999, H) if H > 1 else torch.tensor([0.9])
    lens = {"a": 83, "b": 5, "c": 70, "d": 66}
    seqs = {k: tuple(rnd((n, h, d), 10 * i + j).to(dtype).float() for j, (h, d) in enumerate(((G, D), (G, D), (H, V))))
            for i, (k, n) in enumerate(lens.items())}
    plan = [[("a", 64), ("b", 3)], [("b", 1), ("a", 1), ("c", 2)], [("a", 5), ("b", 1), ("c", 65)],
            [("d", 66), ("c", 1), ("a", 4)], [("a", 9), ("c", 2)]]
    got = run_scan(shape, seqs, plan, dtype, "silu", decay, slots={"a": 2, "b": 0, "c": 1, "d": 0})
    for k, (q, kk, v) in seqs.items():
        q, kk, v = R.silu(q.to(F)), R.silu(kk.to(F)), R.silu(v.to(F))
        want, _ = R.decayed_walk(q.repeat_interleave(H // G, 1), kk.repeat_interleave(H // G, 1), v,
                                 decay.to(F).expand(q.shape[0], H))
        close(got[k], want, 1e-5, k)


@pytest.mark.parametrize("shape", SCAN_SHAPES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_recurrence_with_per_token_decays(shape, dtype, scan_kernel):
    """Step sizes through softplus, decays between nearly 1 and nearly 0 (nothing overflows), a skip."""
    H, G, D, V = shape
    lens = {"a": 150, "b": 4, "c": 61}
    seqs = {k: tuple(rnd((n, h, d), 10 * i + j).to(dtype).float() for j, (h, d) in enumerate(((G, D), (G, D), (H, V))))
            for i, (k, n) in enumerate(lens.items())}
    dt = {k: rnd((n, H), 70 + i, 2.0).to(dtype).float() for i, (k, n) in enumerate(lens.items())}
    dt["a"][20:24] = 30.0               # steps beyond the softplus's bend
    dt["a"][90:92] = 3072.0             # and so large that sums of their logarithms swallow the others'
    dt_bias, a_log, skip = rnd((H, ), 1), rnd((H, ), 2, 1.5), rnd((H, ), 3)
    plan = [[("b", 2), ("a", 130)], [("a", 1), ("c", 60), ("b", 1)], [("c", 1), ("b", 1), ("a", 19)]]
    got = run_scan(shape, seqs, plan, dtype, "none", None, dt, dt_bias, a_log, skip)
    for k, (q, kk, v) in seqs.items():
        want = R.ssd_walk(v.to(F), kk.to(F), q.to(F), dt[k].to(F), a_log.to(F), dt_bias.to(F), skip.to(F))
        close(got[k], want, 2e-5, k)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("lens", [(257, ), (600, 3, 256, 1000), (2, 512, 1, 259)])
def test_long_runs_walk_in_pieces(dtype, lens):
    """Runs of more than 256 rows beside short ones, fresh and continued, per-token decays slow enough to
    carry a token over several pieces."""
    H, G, D, V = 3, 1, 24, 40
    seqs = {str(i): tuple(rnd((n + 7, h, d), 10 * i + j).to(dtype).float() for j, (h, d) in enumerate(((G, D), (G, D), (H, V))))
            for i, n in enumerate(lens)}
    dt = {k: (-3.0 + rnd((s[0].shape[0], H), 70, 1.0)).to(dtype).float() for k, s in seqs.items()}
    dt_bias, a_log, skip = rnd((H, ), 1, 0.3), torch.tensor([-4.0, -2.0, 1.0]), rnd((H, ), 3)
    whole = [(k, s[0].shape[0] - 7) for k, s in seqs.items()]
    for plan in ([whole, [(k, 5) for k in seqs], [(k, 2) for k in seqs]], [[(k, 7) for k in seqs], whole]):
        got = run_scan((H, G, D, V), seqs, plan, dtype, "none", None, dt, dt_bias, a_log, skip)
        for k, (q, kk, v) in seqs.items():
            want = R.ssd_walk(v.to(F), kk.to(F), q.to(F), dt[k].to(F), a_log.to(F), dt_bias.to(F), skip.to(F))
            close(got[k], want, 3e-5, (k, len(plan)))


@pytest.mark.parametrize("cuts", [[700], [300, 400], [255, 2, 443], [640] + [1] * 60])
def test_a_far_token_is_carried_by_a_slow_decay(cuts):
    """One token with a large key and value, everything else orthogonal to the last query: what the query
    reads 690 tokens later is that token's value times decay^690, and nothing where the decay is fast."""
    H, D, V, n, at = 2, 32, 32, 700, 9
    q, k, v = (rnd((n, H, D), i, 0.5) for i in range(3))
    k[..., 0] = 0.0
    k[at, :, 0] = 20.0
    q[-1] = 0.0
    q[-1, :, 0] = 3.0
    decay = torch.tensor([0.999, 0.9])
    plan = [[("a", c)] for c in cuts]
    got = run_scan((H, H, D, V), {"a": (q, k, v)}, plan, torch.float32, "none", decay)["a"]
    want, _ = R.decayed_walk(q.to(F), k.to(F), v.to(F), decay.to(F).expand(n, H))
    close(got, want, 2e-5)
    expect = 60.0 * 0.999**(n - 1 - at) * v[at, 0].to(F)
    assert float((got[-1, 0].to(F) - expect).abs().max()) <= 1e-4 * float(expect.abs().max())
    assert float(got[-1, 1].abs().max()) < 1e-6


@pytest.mark.parametrize("dtypes", [(torch.float32, torch.float32), (torch.bfloat16, torch.bfloat16), (torch.float32, torch.bfloat16),
                                    (torch.bfloat16, torch.float32)])
@pytest.mark.parametrize("channels,taps", [(48, 4), (64, 3), (24, 2), (40, 1), (50, 4), (32, 7), (2056, 4)])
def test_short_convolution_across_cuts_and_batches(dtypes, channels, taps):
    """Aligned rows (runs of rows per thread) and any others; sequences of unequal lengths, single rows beside
    portions, more than a thousand rows at once, a slot taken over; both kernels agree with the reference."""
    from vllm_legacy_amd import _seq_ops as ops
    from vllm_legacy_amd.layers import ShortConv
    din, dout = dtypes
    conv = ShortConv(channels, taps, True, "silu", DEV)
    w, b = rnd((channels, taps), 1), rnd((channels, ), 2)
    conv.weight.data, conv.bias.data = w.to(DEV), b.to(DEV)
    lens = {"a": 1200 if channels == 48 else 60, "b": 7, "c": 33, "d": 12}
    seqs = {k: rnd((n, channels), 3 + i).to(din) for i, (k, n) in enumerate(lens.items())}
    want = {k: R.short_conv(u.to(F), w.to(F), b.to(F)) for k, u in seqs.items()}
    slots = {"a": 0, "b": 1, "c": 2, "d": 1}
    plan = [[("a", lens["a"] - 20), ("b", 2)], [("b", 1), ("a", 1), ("c", 1)], [("c", 1), ("b", 4), ("a", 9)],
            [("a", 1), ("c", 1), ("d", 1)], [("d", 1)], [("d", 8), ("c", 30), ("a", 9)], [("d", 2)]]
    for mode in (0, 1):
        ops.set_short_conv_kernel(mode)
        try:
            state = torch.full((3, max(taps - 1, 0), channels), 5.0, device=DEV)
            at, got = {k: 0 for k in seqs}, {k: [] for k in seqs}
            for step in plan:
                batch = make_batch([n for _, n in step], [at[k] for k, _ in step], 4, slots=[slots[k] for k, _ in step])
                wide = torch.zeros((sum(n for _, n in step), channels + 8), dtype=din)
                wide[:, 8:] = torch.cat([seqs[k][at[k]:at[k] + n] for k, n in step])
                out = torch.empty((wide.shape[0], channels), dtype=dout, device=DEV)
                conv(out, wide.to(DEV)[:, 8:], state if taps > 1 else None, batch)
                lo = 0
                for k, n in step:
                    got[k].append(out[lo:lo + n].float().cpu())
                    at[k] += n
                    lo += n
            assert at == lens
            for k in seqs:
                close(torch.cat(got[k]), want[k], 1e-6 if dout == torch.float32 else 6e-3, (mode, k))
        finally:
            ops.set_short_conv_kernel(0)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("shape", [(4, 16, 8, 2, 2, 4), (6, 10, 14, 3, 5, 3), (3, 7, 5, 1, 7, 1), (2, 64, 32, 1, 1, 4)])
def test_state_space_layer_across_cuts(dtype, shape):
    """Convolution, recurrence and gated norm of the state-space layer, cut anywhere; both states live in
    slots that another sequence used before."""
    from vllm_legacy_amd.attention.recurrent import StateSpaceRecurrence
    H, V, N, G, parts, taps = shape
    layer = StateSpaceRecurrence(H, V, N, G, parts, taps, 1e-5, DEV)
    inner, chan = layer.inner, layer.channels
    t = {"conv": rnd((chan, taps), 1), "conv.b": rnd((chan, ), 2), "dt_bias": rnd((H, ), 3) - 2, "A_log": rnd((H, ), 4, 0.5),
         "D": rnd((H, ), 5), "norm": 1 + 0.2 * rnd((inner, ), 6)}
    layer.conv.weight.data, layer.conv.bias.data = t["conv"].to(DEV), t["conv.b"].to(DEV)
    layer.dt_bias.data, layer.a_log.data, layer.skip.data = t["dt_bias"].to(DEV), t["A_log"].to(DEV), t["D"].to(DEV)
    layer.norm_weight.data = t["norm"].to(DEV)
    n = 90
    spec = {"heads": H, "vdim": V, "state": N, "groups": G, "norm_groups": parts}
    p = rnd((n, inner + chan + H), 7).to(dtype)
    eye = torch.eye(inner + chan + H, dtype=F)
    want = R.ssd_branch(p.to(F), {**{k: v.to(F) for k, v in t.items()}, "in": eye, "o": torch.eye(inner, dtype=F)}, spec, 1e-5)
    ss, cs = StateSpaceRecurrence.get_state_shapes(3, H, V, N, G, taps)
    state, conv = torch.full(ss, 9.0, device=DEV), torch.full(cs, -9.0, device=DEV)
    for cuts in ([n], [2, 3, 1, 64, 2, 18], [70] + [1] * 20):
        at, outs = 0, []
        for c in cuts:
            batch = make_batch([c], [at], 4, slots=[1])
            pp = p[at:at + c].to(DEV)
            out = torch.empty((c, inner), dtype=dtype, device=DEV)
            layer(out, pp[:, :inner], pp[:, inner:inner + chan], pp[:, inner + chan:], state, conv if taps > 1 else None, batch)
            outs.append(out.float().cpu())
            at += c
        close(torch.cat(outs), want, 3e-5 if dtype == torch.float32 else 3e-2, cuts[:2])
    assert bool((state[0] == 9.0).all()) and bool((state[2] == 9.0).all())      # nobody else's slot


# ----------------------------------------------------------------------------- experts
@pytest.mark.parametrize("shape", [(64, 6, 2, 24), (40, 3, 1, 20), (128, 5, 5, 64), (96, 12, 3, 32), (50, 4, 1, 18)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows,form", [(3, 0), (300, 0), (40, 1), (40, 2)])
def test_experts_with_sigmoid_scores_and_weighted_inputs(shape, dtype, rows, form):
    from vllm_legacy_amd import _seq_ops as ops
    from vllm_legacy_amd.routed_experts import RoutedExperts
    W, E, top, ff = shape
    moe = RoutedExperts(W, E, 0, top, ff, act="silu", dtype=dtype, device=DEV, gated=True, score="sigmoid",
                        renormalize=False, weight_input=True)
    t = {"router": rnd((E, W), 1, W**-0.5)}
    for e in range(E):
        t[f"e{e}.gate"], t[f"e{e}.up"], t[f"e{e}.down"] = rnd((ff, W), 10 + e, 2 * W**-0.5), rnd((ff, W), 40 + e, 2 * W**-0.5), \
            rnd((W, ff), 70 + e, ff**-0.5)
    t = {k: v.to(torch.bfloat16) for k, v in t.items()}
    moe.set_weights(t)
    h = rnd((rows, W), 3).to(dtype)
    want = R.routed_ff(h.to(F), {k: v.to(F) for k, v in t.items()}, R.moe_mlp(E, top, ff))
    # weights on the outputs, or renormalized, would be something else
    s, idx = torch.topk(torch.sigmoid(h.to(F) @ t["router"].to(F).T), top, -1)
    outs = torch.stack([sum(s[i, x] * R.expert(h[i:i + 1].to(F), R.sub({k: v.to(F) for k, v in t.items()}, f"e{int(idx[i, x])}."))[0]
                            for x in range(top)) for i in range(3)])
    assert float((outs - want[:3]).abs().max()) > 0.02 * float(want.abs().max())
    ops.set_grouped_linear_form(form)
    try:
        got = moe(h.to(DEV)).cpu()
    finally:
        ops.set_grouped_linear_form(0)
    err = (got.to(F) - want).abs().amax(1) / want.abs().max()
    if dtype == torch.float32:
        assert float(err.max()) <= 2e-5
    else:       # a close call of the router may go the other way for a few rows
        assert float(torch.quantile(err, 0.9)) <= 3e-2


def test_router_scores_and_renormalization():
    """Softmax and sigmoid scores, renormalized and as they are, with and without a correction that
    changes the choice but not the weights."""
    from vllm_legacy_amd import _seq_ops as ops
    T, W, E, top = 9, 32, 7, 3
    h, router, corr = rnd((T, W), 0), rnd((E, W), 1, 0.3), rnd((E, ), 2, 0.4)
    z = h.to(F) @ router.to(F).T
    for score, s in (("softmax", torch.softmax(z, -1)), ("sigmoid", torch.sigmoid(z))):
        for c in (None, corr):
            for renorm in (True, False):
                idx = torch.topk(s if c is None else s + c.to(F), top, -1).indices
                w = s.gather(1, idx)
                w = w / w.sum(-1, keepdim=True) if renorm else w
                e, got, _ = ops.moe_route(h.to(DEV), router.to(DEV), None if c is None else c.to(DEV), None, top,
                                          score=score, renormalize=renorm)
                assert torch.equal(e.cpu().long(), idx), (score, renorm)
                close(got, w, 1e-6, (score, renorm))


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
    """The stream after every layer run, float32."""
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
    assert len(got) == len(taps) == len(R.layer_order(s.cfg))
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
    """Chunks begin and end many times among decoded tokens."""
    s = Served(tmp_path, name, torch.float32, num_blocks=80, block_size=4)
    toks = tokens_of(s.cfg, 200, 8)
    got = [s.step([("a", toks[:3])])["a"]]
    for t in range(3, 200):
        got.append(s.step([("a", toks[t:t + 1])])["a"])
    s.check(torch.cat(got), toks)


def test_long_prompts_beside_a_decoding_request(tmp_path):
    """Prompts of several hundred tokens (blocks and pieces of the recurrences), whole and in large
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
    assert type(engine.runner.model).__name__ == "BatatarForCausalLM"
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
