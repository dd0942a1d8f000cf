"""Prefill and decode throughput of a Dagavik stack beside the closest existing stack at equal size --
Lamosun (delta-rule layers with short convolutions, latent attention, gated routed experts) -- and each
of Dagavik's kernels beside the like kernel of Lamosun, Batatar (matrix-state recurrence and attention in
one layer) or Dopipel (router) against its roofline.

Run through `python bench.py --arch dagavik [--arch-size 2k|4k]` (one GPU, random weights, bf16).
Prints one JSON line.  `end_to_end`: tokens/s of a prompt step (one sequence of --arch-prompt
tokens) and of a decode step (--arch-batch sequences at --arch-context tokens) of four layers plus
logits: Dagavik (channel_delta / parallel / channel_delta / latent_attention) and Lamosun (delta /
latent_attention / delta / latent_attention), the same experts everywhere.  `kernels`: microseconds per
launch, the time its algorithmic bytes or arithmetic would take at the part's peaks, and the ratio
(1.0 = on the roofline).  Windowed attention is priced for the keys a window lets it see, a recurrence for
the fp32 arithmetic of its token-by-token form.
"""
import json
import time

import torch

from tools.batatar_bench import SIZES as BATATAR_SIZES
from tools.batatar_bench import batatar_config
from tools.lamosun_bench import SIZES as LAMOSUN_SIZES
from tools.lamosun_bench import lamosun_config
from tools.seq_arch_bench import FMA_F32, HBM, MFMA_BF16, record, timed

SIZES = {
    "2k": dict(width=2048, heads=16, kv_heads=4, dim=128, window=1024, rot_dims=64, m_heads=16, m_dim=64, m_vdim=128,
               d_kv_heads=8, taps=4, kv_rank=512, experts=16, top=2, expert_ff=1408, groups=4, keep=2),
    "4k": dict(width=4096, heads=32, kv_heads=8, dim=128, window=1024, rot_dims=64, m_heads=32, m_dim=64, m_vdim=128,
               d_kv_heads=16, taps=4, kv_rank=512, experts=32, top=4, expert_ff=1408, groups=8, keep=4),
}


def dagavik_config(s, kinds, vocab):
    """kinds: per layer channel_delta | parallel | latent_attention; every layer has the experts."""
    D = s["dim"]
    mixers = {
        "channel_delta": {"heads": s["heads"], "kv_heads": s["d_kv_heads"], "dim": D, "vdim": D, "conv": s["taps"]},
        "parallel": {"left": {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": D, "vdim": D, "scale": D**-0.5,
                              "mask": {"size": s["window"]}, "rot": {"dims": s["rot_dims"], "base": 10000.0}},
                     "right": {"heads": s["m_heads"], "dim": s["m_dim"], "vdim": s["m_vdim"], "gate_cap": 15.0},
                     "left_scale": 0.6, "right_scale": 0.7},
        "latent_attention": {"heads": s["heads"], "dim": D, "vdim": D, "kv_rank": s["kv_rank"], "scale": D**-0.5},
    }
    moe = {"kind": "moe", "expert": {"ff": s["expert_ff"]},
           "router": {"experts": s["experts"], "top": s["top"], "scale": 2.0,
                      "groups": {"count": s["groups"], "keep": s["keep"]}}}
    return {"architecture": "Dagavik", "vocab": vocab, "width": s["width"], "norm": {"eps": 1e-5},
            "embedding": {"bigram": {"buckets": 30011, "mul_prev": 1009, "mul_cur": 31}},
            "layers": [{"type": k, "mixer": mixers[k], "mlp": moe} for k in kinds]}


def run(args):
    from vllm_legacy_amd import _seq_ops as sops
    from vllm_legacy_amd.attention.batch import SequenceBatch
    from vllm_legacy_amd.model.batatar import BatatarConfig, BatatarForCausalLM
    from vllm_legacy_amd.model.dagavik import DagavikConfig, DagavikForCausalLM
    from vllm_legacy_amd.model.lamosun import LamosunConfig, LamosunForCausalLM

    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    dt = torch.bfloat16
    s = SIZES[args.arch_size]
    vocab, BS = 32000, 16
    P, B, C = args.arch_prompt, args.arch_batch, args.arch_context
    e2e, kern = {}, {}
    g = torch.Generator(device=dev).manual_seed(0)
    nblk = max(B * (C // BS + 1), P // BS + 1) + 4
    per = C // BS + 1
    tables = torch.randperm(nblk - 4, generator=g, device=dev)[:B * per].view(B, per).tolist()
    pre = SequenceBatch.build([P], [0], [list(range(P // BS + 1))], [0], BS, dev)
    dec = SequenceBatch.build([1] * B, [C - 1] * B, tables, list(range(B)), BS, dev)
    ids_p = torch.randint(0, vocab, (P, ), generator=g, device=dev)
    ids_d = torch.randint(0, vocab, (B, ), generator=g, device=dev)

    def whole_steps(name, model, caches):
        @torch.inference_mode()
        def prefill():
            x = model(ids_p, pre.positions, caches, pre)
            return model.compute_logits(x[-1:])

        @torch.inference_mode()
        def decode():
            x = model(ids_d, dec.positions, caches, dec)
            return model.compute_logits(x)

        t = timed(prefill, 8, 6)
        e2e[f"{name}_prefill_tokens_per_s"] = round(P / t, 1)
        e2e[f"{name}_prefill_ms_per_step"] = round(t * 1e3, 3)
        t = timed(decode, 20, 3)
        e2e[f"{name}_decode_tokens_per_s"] = round(B / t, 1)
        e2e[f"{name}_decode_ms_per_step"] = round(t * 1e3, 3)

    def fill(caches):
        for c in caches:
            for k, t in (c.items() if isinstance(c, dict) else enumerate(c)):
                if t is not None and t.is_floating_point():
                    t.normal_(0, 1.0 if k in ("keys", "values", "latent") else 0.1, generator=g)

    H, G, D, width = s["heads"], s["kv_heads"], s["dim"], s["width"]
    E, top, eff, rank, window = s["experts"], s["top"], s["expert_ff"], s["kv_rank"], s["window"]
    GD, HV = s["d_kv_heads"] * D, H * D
    steps = (("prefill", pre, P, 5), ("decode", dec, B, 20))

    def rnd(*shape, dtype=dt):
        return torch.randn(*shape, device=dev, dtype=dtype)

    def experts(name, moe, T, it, tag):
        hh = rnd(T, width)
        sec = timed(lambda: moe(hh), it)
        routed, used = T * top, min(E, T * top)
        record(kern, f"{name}.gated_experts.{tag}", sec, flops=6.0 * routed * width * eff,
               nbytes=2.0 * (3 * used * eff * width + routed * width) + 4.0 * T * width)

    def latent(name, attn, cache, rot, batch, T, it, tag):
        W = rank + rot
        q_lat, o_lat = (rnd(H, T, rank).transpose(0, 1) for _ in range(2))
        q = rnd(T, H * (D + rot))
        q_rot = q.view(T, H, D + rot)[:, :, D:]
        sinks = None if attn.sinks is None else attn.sinks.data
        sec = timed(lambda: sops.latent_attention_tiles(o_lat, q_lat, q_rot, cache, batch.block_tables,
                                                        batch.query_start_loc, batch.context_lens, batch.max_query_len,
                                                        attn.scale, attn.key_splits(batch), 0, None, sinks), it)
        if tag == "prefill":
            record(kern, f"{name}.latent_attention.prefill", sec, flops=1.0 * T * (T + 1) * H * (W + rank),
                   nbytes=2.0 * T * (H * (W + rank) + W))
        else:
            record(kern, f"{name}.latent_attention.decode", sec, flops=2.0 * B * C * H * (W + rank),
                   nbytes=2.0 * B * C * W + 2.0 * B * H * (W + rank))
        kv = rnd(T, W)
        sec = timed(lambda: sops.latent_rotary_write(q, D + rot, D, H, kv, attn.latent_norm.data, 1e-5, cache,
                                                     batch.positions, batch.slot_mapping, attn.inv_freq, attn.magnitude,
                                                     rot), it)
        record(kern, f"{name}.latent_write.{tag}", sec, nbytes=2.0 * T * (2 * H * rot + 2 * W))

    # ------------------------------------------------------------------ Lamosun: whole steps and the like kernels
    ls = dict(LAMOSUN_SIZES[args.arch_size], **{k: s[k] for k in ("width", "heads", "kv_heads", "dim", "kv_rank", "experts",
                                                                  "top", "expert_ff", "taps")})
    kinds = [("delta", "moe"), ("latent_attention", "moe"), ("delta", "moe"), ("latent_attention", "moe")]
    model = LamosunForCausalLM(LamosunConfig.from_dict(lamosun_config(ls, kinds, vocab)), dt, dev, seed=0)
    caches = model.allocate_caches(nblk, BS, B)
    fill(caches)
    whole_steps("lamosun", model, caches)
    with torch.inference_mode():
        rule, conv = model.layers[0].rule, model.layers[0].conv
        for tag, batch, T, it in steps:
            cin = rnd(T, 2 * GD + 2 * HV + 2 * H, dtype=torch.float32)
            qkv = torch.empty(T, 2 * GD + HV, device=dev)
            sec = timed(lambda: conv(qkv, cin[:, :2 * GD + HV], caches[0]["conv"], batch), it)
            record(kern, f"lamosun.short_conv.{tag}", sec,
                   nbytes=T * (2 * GD + HV) * 8.0 + batch.num_seqs * (s["taps"] - 1) * (2 * GD + HV) * 8.0,
                   note="fp32 in and out")
            mixed = rnd(T, HV)
            qd, kd, vd = qkv.split([GD, GD, HV], dim=1)
            gt, bt, dtp = cin[:, 2 * GD + HV:].split([HV, H, H], dim=1)
            sec = timed(lambda: rule(mixed, qd, kd, vd, gt, bt, dtp, caches[0]["state"], batch), it)
            record(kern, f"lamosun.delta_rule_layer.{tag}", sec, peak=FMA_F32, flops=6.0 * T * H * D * D,
                   nbytes=T * (4.0 * (2 * GD + 2 * HV + 2 * H) + 2.0 * HV) + 8.0 * batch.num_seqs * H * D * D,
                   note="walk, head norm and output gate")
            latent("lamosun", model.layers[1].attn, caches[1]["latent"], ls["rot_dim"], batch, T, it, tag)
            experts("lamosun", model.layers[0].experts, T, it, tag)
            x, y, h, w = rnd(T, width, dtype=torch.float32), rnd(T, width, dtype=torch.float32), rnd(T, width), \
                torch.ones(width, device=dev)
            sec = timed(lambda: sops.post_norm(x, y, w, 2.0, 1e-5, h), it)
            record(kern, f"lamosun.post_norm.{tag}", sec, nbytes=T * width * (4.0 + 4 + 4 + 2))
    del model, caches
    torch.cuda.empty_cache()

    # ------------------------------------------------------------------ Batatar: a parallel layer's kernels, and Dopipel's
    bs = dict(BATATAR_SIZES[args.arch_size], chunk=window)
    model = BatatarForCausalLM(BatatarConfig.from_dict(batatar_config(bs, ["parallel"], vocab)), dt, dev, seed=0)
    caches = model.allocate_caches(nblk, BS, B)
    fill(caches)
    keys, values = caches[0]["keys"].clone(), caches[0]["values"].clone()
    with torch.inference_mode():
        attn, ssd = model.layers[0].attn, model.layers[0].recur
        Hs, Vs, N, Gs, inner, chan = bs["s_heads"], bs["s_vdim"], bs["s_state"], bs["s_groups"], ssd.inner, ssd.channels
        freq = torch.rand(D // 2, device=dev)
        for tag, batch, T, it in steps:
            pairs = sum(p % window + 1 for p in range(T)) if tag == "prefill" else B * ((C - 1) % window + 1)
            q, k, v, gate, out = rnd(T, H * D), rnd(T, G * D), rnd(T, G * D), rnd(T, H), rnd(T, H * D)
            if tag == "prefill":
                sec = timed(lambda: sops.kv_attention_tiles(out, q, gate, keys, values, batch.block_tables,
                                                            batch.query_start_loc, batch.context_lens,
                                                            batch.max_query_len, None, True, H, 0, attn.scale, 0,
                                                            attn.softcap, window, attn.sinks), it)
                record(kern, "batatar.kv_attention.prefill", sec, flops=4.0 * pairs * H * D, nbytes=2.0 * T * (2 * H + 2 * G) * D)
            else:
                sec = timed(lambda: sops.kv_attention(out, q, gate, keys, values, batch.block_tables, batch.token_seq,
                                                      batch.positions, None, True, H, 0, attn.scale, 0, attn.softcap,
                                                      window, attn.sinks), it)
                record(kern, "batatar.kv_attention.decode", sec, nbytes=2 * 2.0 * G * pairs * D + 2 * 2.0 * B * H * D)
            sec = timed(lambda: sops.rotary_kv_write(q, k, v, keys, values, batch.positions, batch.slot_mapping, freq,
                                                     freq, H, D, True), it)
            record(kern, f"dopipel.rotary_kv_write.{tag}", sec, nbytes=2.0 * T * (2 * H + 4 * G) * D)
            xbc, dts = rnd(T, chan), rnd(T, 8 * ((Hs + 7) // 8))[:, :Hs]
            u, ys, gn = rnd(T, chan), torch.empty(T, inner, device=dev), Gs * N
            sec = timed(lambda: ssd.conv(u, xbc, caches[0]["conv"], batch), it)
            record(kern, f"batatar.short_conv.{tag}", sec,
                   nbytes=T * chan * 4.0 + batch.num_seqs * (s["taps"] - 1) * chan * 8.0, note="bf16 in and out")
            sec = timed(lambda: sops.decay_scan(ys, u[:, inner + gn:], u[:, inner:inner + gn], u[:, :inner], caches[0]["state"],
                                                batch.query_start_loc, batch.context_lens, batch.state_slots, Gs,
                                                batch.max_query_len, None, dts, ssd.dt_bias.data, ssd.a_log.data,
                                                ssd.skip.data), it)
            record(kern, f"batatar.decay_scan_ssd.{tag}", sec, peak=FMA_F32, flops=4.0 * T * Hs * N * Vs,
                   nbytes=T * (2.0 * (chan + Hs) + 4 * inner) + 8.0 * batch.num_seqs * Hs * N * Vs)
            o, mixed, gl, nw = torch.randn(T, HV, device=dev), rnd(T, HV), rnd(T, HV), torch.ones(HV, device=dev)
            sec = timed(lambda: sops.gated_group_rms_norm(mixed, o, nw, gl, "sigmoid", False, 1, 1e-5), it)
            record(kern, f"batatar.gated_group_rms_norm.{tag}", sec, nbytes=T * HV * (4.0 + 2 + 2))
            x, y, y2, h, w = rnd(T, width, dtype=torch.float32), rnd(T, width, dtype=torch.float32), \
                rnd(T, width, dtype=torch.float32), rnd(T, width), torch.ones(width, device=dev)
            sec = timed(lambda: sops.residual_norms(x, y, None, w, None, None, h, w, 1e-5, 0.25, y2, w), it)
            record(kern, f"batatar.stream_update_two_branches.{tag}", sec, nbytes=T * width * (4.0 + 4 + 4 + 4 + 2))
            hh, rw = rnd(T, width), rnd(E, width, dtype=torch.float32)
            logits = rnd(T, E, dtype=torch.float32) if T >= 256 else None
            sec = timed(lambda: sops.moe_route(hh, rw, None, None, top, logits), it)
            record(kern, f"dopipel.moe_route.{tag}", sec, nbytes=T * (4.0 * E if T >= 256 else 2.0 * width) + 8.0 * T * top)
    del model, caches
    torch.cuda.empty_cache()

    # ------------------------------------------------------------------ Dagavik: whole steps and its kernels
    kinds = ["channel_delta", "parallel", "channel_delta", "latent_attention"]
    model = DagavikForCausalLM(DagavikConfig.from_dict(dagavik_config(s, kinds, vocab)), dt, dev, seed=0)
    caches = model.allocate_caches(nblk, BS, B)
    fill(caches)
    whole_steps("dagavik", model, caches)
    with torch.inference_mode():
        delta, conv, par, lat = model.layers[0].recur, model.layers[0].conv, model.layers[1], model.layers[3].attn
        mem, Hm, Dm, Vm = par.recur, s["m_heads"], s["m_dim"], s["m_vdim"]
        for tag, batch, T, it in steps:
            n_seq, at = batch.num_seqs, (batch.query_start_loc, batch.context_lens, batch.state_slots)
            proj, u = rnd(T, 2 * GD + HV), rnd(T, 2 * GD + HV)
            sec = timed(lambda: conv(u, proj, caches[0]["conv"], batch), it)
            record(kern, f"dagavik.short_conv.{tag}", sec,
                   nbytes=T * (2 * GD + HV) * 4.0 + n_seq * (s["taps"] - 1) * (2 * GD + HV) * 8.0, note="bf16 in and out")
            q, k, v = u.split([GD, GD, HV], dim=1)
            beta, z, gate, mixed, o = rnd(T, H), rnd(T, HV, dtype=torch.float32), rnd(T, HV), rnd(T, HV), torch.empty(T, HV, device=dev)
            sec = timed(lambda: sops.channel_delta_scan(o, q, k, v, beta, z, delta.dt_bias.data, delta.a_log.data,
                                                        caches[0]["state"], *at, delta.kv_heads, batch.max_query_len), it)
            record(kern, f"dagavik.channel_delta_scan.{tag}", sec, peak=FMA_F32, flops=6.0 * T * H * D * D,
                   nbytes=T * (2.0 * (2 * GD + HV + H) + 4.0 * 2 * HV) + 8.0 * n_seq * H * D * D,
                   note="unit norms, decays per channel, walk")
            sec = timed(lambda: delta(mixed, q, k, v, gate, beta, z, caches[0]["state"], batch), it)
            record(kern, f"dagavik.channel_delta_layer.{tag}", sec, peak=FMA_F32, flops=6.0 * T * H * D * D,
                   nbytes=T * 2.0 * (2 * GD + 3 * HV + H + 2 * HV) + 8.0 * n_seq * H * D * D,
                   note="walk, head norm and output gate")
            nw = delta.norm_weight.data
            sec = timed(lambda: sops.gated_group_rms_norm(mixed, o, nw, gate, "sigmoid", False, H, 1e-5), it)
            record(kern, f"dagavik.gated_head_norm.{tag}", sec, nbytes=T * HV * (4.0 + 2 + 2), note="a norm per head")
            zi, zf = rnd(T, Hm, dtype=torch.float32), rnd(T, Hm, dtype=torch.float32)
            gates = lambda: sops.matrix_memory_gates(zi, zf, mem.bias_i.data, mem.bias_f.data, mem.gate_cap,
                                                     caches[1]["maximum"], *at, batch.max_query_len)
            sec = timed(gates, it)
            record(kern, f"dagavik.matrix_memory_gates.{tag}", sec, nbytes=T * Hm * 4.0 * 5)
            rl, rw, rf = gates()
            qm, km, vm, gm = rnd(T, Hm * Dm), rnd(T, Hm * Dm), rnd(T, Hm * Vm), rnd(T, Hm * Vm)
            om, ns, out2 = torch.empty(T, Hm * Vm, device=dev), torch.empty(T, Hm, device=dev), rnd(T, Hm * Vm)
            sec = timed(lambda: sops.decay_scan(om, qm, km, vm, caches[1]["memory"], *at, Hm, batch.max_query_len, row_log=rl,
                                                row_weight=rw, row_floor=rf, norm_scale=ns, norm_eps=1e-6,
                                                q_scale=Dm**-0.5, sizes=(Dm, Vm)), it)
            record(kern, f"dagavik.decay_scan_memory.{tag}", sec, peak=FMA_F32, flops=4.0 * T * Hm * Dm * (Vm + 1),
                   nbytes=T * Hm * (2.0 * (2 * Dm + Vm) + 4 * Vm + 16) + 8.0 * n_seq * Hm * Dm * (Vm + 1),
                   note="matrix memory with its normalizer")
            sec = timed(lambda: mem(out2, qm, km, vm, gm, zi, zf, caches[1]["memory"], caches[1]["maximum"], batch), it)
            record(kern, f"dagavik.matrix_memory_layer.{tag}", sec, peak=FMA_F32, flops=4.0 * T * Hm * Dm * (Vm + 1),
                   nbytes=T * Hm * (2.0 * (2 * Dm + 3 * Vm) + 8) + 8.0 * n_seq * Hm * Dm * (Vm + 1),
                   note="gates, recurrence, norm and output gate")
            pairs = sum(min(p + 1, window) for p in range(T)) if tag == "prefill" else B * min(C, window)
            q, k, v, out = rnd(T, H * D), rnd(T, G * D), rnd(T, G * D), rnd(T, H * D)
            attn = par.attn
            if tag == "prefill":
                sec = timed(lambda: sops.kv_attention_tiles(out, q, None, caches[1]["keys"], caches[1]["values"],
                                                            batch.block_tables, batch.query_start_loc, batch.context_lens,
                                                            batch.max_query_len, None, False, H, window, attn.scale), it)
                record(kern, "dagavik.kv_attention.prefill", sec, flops=4.0 * pairs * H * D,
                       nbytes=2.0 * T * (2 * H + 2 * G) * D, note="window")
            else:
                sec = timed(lambda: sops.kv_attention(out, q, None, caches[1]["keys"], caches[1]["values"], batch.block_tables,
                                                      batch.token_seq, batch.positions, None, False, H, window, attn.scale), it)
                record(kern, "dagavik.kv_attention.decode", sec, nbytes=2 * 2.0 * G * pairs * D + 2 * 2.0 * B * H * D,
                       note="reads the window only")
            sec = timed(lambda: sops.rotary_kv_write(q, k, v, caches[1]["keys"], caches[1]["values"], batch.positions,
                                                     batch.slot_mapping, attn.inv_freq, None, H, attn.rot_dims, False), it)
            record(kern, f"dagavik.rotary_kv_write.{tag}", sec,
                   nbytes=2.0 * T * (2 * H * s["rot_dims"] + 2 * G * (D + D)), note="half of every head turns")
            latent("dagavik", lat, caches[3]["latent"], 0, batch, T, it, tag)
            experts("dagavik", par.experts, T, it, tag)
            hh, rw2 = rnd(T, width), rnd(E, width, dtype=torch.float32)
            logits = rnd(T, E, dtype=torch.float32) if T >= 256 else None
            sec = timed(lambda: sops.moe_route(hh, rw2, None, None, top, logits, renormalize=False, groups=s["groups"],
                                               keep_groups=s["keep"], weight_scale=2.0), it)
            record(kern, f"dagavik.moe_route.{tag}", sec, nbytes=T * (4.0 * E if T >= 256 else 2.0 * width) + 8.0 * T * top)
            x, y, y2, h, w = rnd(T, width, dtype=torch.float32), rnd(T, width, dtype=torch.float32), \
                rnd(T, width, dtype=torch.float32), rnd(2, T, width), torch.ones(width, device=dev)
            ye, pair_row, wts, _ = par.experts.rows(hh)
            sec = timed(lambda: sops.branch_sum_norms(x, [(y, 0.6), (y2, 0.7)], (ye, pair_row, wts), [(h[0], w), (h[1], w)], 1e-5), it)
            record(kern, f"dagavik.branch_sum_norms.{tag}", sec, nbytes=T * width * (4.0 * (4 + top) + 4),
                   note="two branches, the experts' weighted rows, two normed copies")
    del model, caches
    torch.cuda.empty_cache()

    print(json.dumps({"metric": "prefill and decode tokens/s, Dagavik beside Lamosun at equal size (4 layers, bf16, random weights)",
                      "size": args.arch_size, "shape": s, "prompt_tokens": P, "decode_batch": B, "decode_context": C,
                      "end_to_end": e2e, "kernels": kern, "peaks": {"hbm_Bps": HBM, "mfma_bf16": MFMA_BF16, "fma_f32": FMA_F32},
                      "time": time.strftime("%Y-%m-%d %H:%M:%S")}))
