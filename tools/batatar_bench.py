"""Prefill and decode throughput of a Batatar stack beside the two closest existing stacks at equal size
-- Lusadra (softmax attention and a matrix-state recurrence side by side in every layer, dense
feed-forward) and Lamosun's delta-rule layers (a matrix-state recurrence with a short convolution and
per-token decays, gated routed experts) -- and each of Batatar's kernels beside the like kernel of
Lusadra, Lamosun or Dopipel against its roofline.

Run through `python bench.py --arch batatar [--arch-size 2k|4k]` (one GPU, random weights, bf16).
Prints one JSON line.  `end_to_end`: tokens/s of a prompt step (one sequence of --arch-prompt
tokens) and of a decode step (--arch-batch sequences at --arch-context tokens) of four layers plus
logits: Batatar (lightning / parallel / lightning / parallel, experts everywhere), Lusadra (four
parallel layers, a dense feed-forward as wide as the experts a token uses) and Lamosun (four delta
layers with the same experts).  `kernels`: microseconds per launch, the time its algorithmic bytes or
arithmetic would take at the part's peaks, and the ratio (1.0 = on the roofline).  Chunked attention
is priced for the keys a chunk lets it see, a recurrence for the fp32 arithmetic of its token-by-token
form.
"""
import json
import time

import torch

from tools.lamosun_bench import lamosun_config
from tools.seq_arch_bench import FMA_F32, HBM, MFMA_BF16, lusadra_config, record, timed

SIZES = {
    "2k": dict(width=2048, heads=16, kv_heads=4, dim=128, chunk=1024, softcap=30.0, l_heads=16, l_dim=128, s_heads=32,
               s_vdim=64, s_state=128, s_groups=2, s_parts=2, taps=4, experts=16, top=2, expert_ff=1408,
               delta_kv_heads=8, blocks=16, gru=2048, rot_dim=64, kv_rank=512, q_rank=1536, side=64,
               r_heads=16, r_dim=64, r_vdim=128, window=1024),
    "4k": dict(width=4096, heads=32, kv_heads=8, dim=128, chunk=1024, softcap=30.0, l_heads=32, l_dim=128, s_heads=64,
               s_vdim=64, s_state=128, s_groups=4, s_parts=4, taps=4, experts=32, top=4, expert_ff=1408,
               delta_kv_heads=16, blocks=32, gru=4096, rot_dim=64, kv_rank=512, q_rank=1536, side=64,
               r_heads=32, r_dim=64, r_vdim=128, window=1024),
}


def batatar_config(s, kinds, vocab):
    """kinds: per layer lightning | parallel; every layer has the experts."""
    H = s["l_heads"]
    mixers = {
        "lightning": {"heads": H, "dim": s["l_dim"], "vdim": s["l_dim"], "decay": [1.0 - 2.0**-(1 + 8.0 * h / H) for h in range(H)]},
        "parallel": {"left": {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["dim"],
                              "mask": {"size": s["chunk"]}, "scale": s["dim"]**-0.5, "softcap": s["softcap"]},
                     "right": {"heads": s["s_heads"], "vdim": s["s_vdim"], "state": s["s_state"], "groups": s["s_groups"],
                               "norm_groups": s["s_parts"], "conv": s["taps"]}},
    }
    moe = {"kind": "moe", "expert": {"ff": s["expert_ff"]}, "router": {"experts": s["experts"], "top": s["top"]}}
    return {"architecture": "Batatar", "vocab": vocab, "width": s["width"], "norm": {"eps": 1e-5}, "residual_mult": 0.5,
            "layers": [{"type": k, "mixer": mixers[k], "mlp": moe} for k in kinds]}


def run(args):
    from vllm_legacy_amd import _seq_ops as sops
    from vllm_legacy_amd.attention.batch import SequenceBatch
    from vllm_legacy_amd.model.batatar import BatatarConfig, BatatarForCausalLM
    from vllm_legacy_amd.model.lamosun import LamosunConfig, LamosunForCausalLM
    from vllm_legacy_amd.model.lusadra import LusadraConfig, LusadraForCausalLM

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
        t = timed(decode, 20, 3)
        e2e[f"{name}_decode_tokens_per_s"] = round(B / t, 1)
        e2e[f"{name}_decode_ms_per_step"] = round(t * 1e3, 3)

    def fill(caches):
        for c in caches:
            for k, t in (c.items() if isinstance(c, dict) else enumerate(c)):
                if t is not None and t.is_floating_point():
                    t.normal_(0, 1.0 if k in ("keys", "values") else 0.1, generator=g)

    H, G, D, width = s["heads"], s["kv_heads"], s["dim"], s["width"]
    E, top, eff = s["experts"], s["top"], s["expert_ff"]
    steps = (("prefill", pre, P, 5), ("decode", dec, B, 20))

    def rnd(*shape, dtype=dt):
        return torch.randn(*shape, device=dev, dtype=dtype)

    # ------------------------------------------------------------------ Lusadra: whole steps, its recurrence and norm
    model = LusadraForCausalLM(LusadraConfig.from_dict(lusadra_config(dict(s, ff=top * eff), 4, vocab)), dt, dev, seed=0)
    caches = model.allocate_caches(nblk, BS, B)
    fill(caches)
    whole_steps("lusadra", model, caches)
    del model, caches
    torch.cuda.empty_cache()
    from vllm_legacy_amd.attention.recurrent import GatedLinearRecurrence
    with torch.inference_mode():
        Hr, Dr, Vr = s["r_heads"], s["r_dim"], s["r_vdim"]
        rec = GatedLinearRecurrence(Hr, Dr, Vr, 8.0, 1e-5)
        state = torch.randn(GatedLinearRecurrence.get_state_shape(B, Hr, Dr, Vr), device=dev) * 0.1
        w2 = rnd(Hr * Dr, 16)
        bias, nw = torch.ones(Hr * Dr, device=dev), torch.ones(Vr, device=dev)
        for tag, batch, T, it in steps:
            q, k, v, gate, y, out = rnd(T, Hr * Dr), rnd(T, Hr * Dr), rnd(T, Hr * Vr), rnd(T, Hr * Vr), rnd(T, 16), rnd(T, Hr * Vr)
            sec = timed(lambda: rec(out, q, k, v, gate, y, w2, bias, nw, state, batch), it)
            record(kern, f"lusadra.recurrent_layer.{tag}", sec, peak=FMA_F32, flops=4.0 * T * Hr * Dr * Vr,
                   nbytes=2.0 * T * (2 * Hr * Dr + 3 * Hr * Vr) + 8.0 * batch.num_seqs * Hr * Dr * Vr,
                   note="log decays, walk (in pieces), head norm and gate")
            o = torch.randn(T, Hr, Vr, device=dev)
            sec = timed(lambda: sops.gated_head_rms_norm(out, o, nw, gate, 1e-5, 1.0), it)
            record(kern, f"lusadra.gated_head_rms_norm.{tag}", sec, nbytes=T * Hr * Vr * (4.0 + 2 + 2))
        del state

    # ------------------------------------------------------------------ Dopipel's attention, cache write and stream update
    with torch.inference_mode():
        keys, values = rnd(nblk, BS, G, D), rnd(nblk, BS, G, D)
        freq = torch.rand(D // 2, device=dev)
        for tag, batch, T, it in steps:
            q, k, v, out = rnd(T, H * D), rnd(T, G * D), rnd(T, G * D), rnd(T, H * D)
            if tag == "prefill":
                sec = timed(lambda: sops.kv_attention_tiles(out, q, None, keys, values, batch.block_tables,
                                                            batch.query_start_loc, batch.context_lens,
                                                            batch.max_query_len, freq, True, H, 0, D**-0.5), it)
                record(kern, "dopipel.kv_attention.prefill", sec, flops=2.0 * T * (T + 1) * H * D,
                       nbytes=2.0 * T * (2 * H + 2 * G) * D)
            else:
                sec = timed(lambda: sops.kv_attention(out, q, None, keys, values, batch.block_tables, batch.token_seq,
                                                      batch.positions, freq, True, H, 0, D**-0.5), it)
                record(kern, "dopipel.kv_attention.decode", sec, nbytes=2 * 2.0 * B * G * C * D + 2 * 2.0 * B * H * D)
            sec = timed(lambda: sops.rotary_kv_write(q, k, v, keys, values, batch.positions, batch.slot_mapping, freq,
                                                     freq, H, D, True), it)
            record(kern, f"dopipel.rotary_kv_write.{tag}", sec, nbytes=2.0 * T * (2 * H + 4 * G) * D)
            x, y, h, w = rnd(T, width, dtype=torch.float32), rnd(T, width, dtype=torch.float32), rnd(T, width), \
                torch.ones(width, device=dev)
            sec = timed(lambda: sops.residual_norms(x, y, None, w, w, None, h, w, 1e-5), it)
            record(kern, f"dopipel.residual_norms.{tag}", sec, nbytes=T * width * (4.0 + 4 + 4 + 2))

    # ------------------------------------------------------------------ Lamosun: whole steps, its recurrence and experts
    model = LamosunForCausalLM(LamosunConfig.from_dict(lamosun_config(dict(s, ff=top * eff), [("delta", "moe")] * 4, vocab)), dt, dev, seed=0)
    caches = model.allocate_caches(nblk, BS, B)
    fill(caches)
    whole_steps("lamosun", model, caches)
    with torch.inference_mode():
        moe, rule, rule_conv = model.layers[0].experts, model.layers[0].rule, model.layers[0].conv
        HV, GD = H * D, s["delta_kv_heads"] * D
        for tag, batch, T, it in steps:
            cin = rnd(T, 2 * GD + 2 * HV + 2 * H, dtype=torch.float32)
            qkv = torch.empty(T, 2 * GD + HV, device=dev)
            sec = timed(lambda: rule_conv(qkv, cin[:, :2 * GD + HV], caches[0]["conv"], batch), it)
            record(kern, f"lamosun.short_conv.{tag}", sec,
                   nbytes=T * (2 * GD + HV) * 8.0 + batch.num_seqs * (s["taps"] - 1) * (2 * GD + HV) * 8.0)
            mixed = rnd(T, HV)
            qd, kd, vd = qkv.split([GD, GD, HV], dim=1)
            gt, bt, dtp = cin[:, 2 * GD + HV:].split([HV, H, H], dim=1)
            sec = timed(lambda: rule(mixed, qd, kd, vd, gt, bt, dtp, caches[0]["state"], batch), it)
            record(kern, f"lamosun.delta_rule_scan.{tag}", sec, peak=FMA_F32, flops=6.0 * T * H * D * D,
                   nbytes=T * (4.0 * (2 * GD + 2 * HV + 2 * H) + 2.0 * HV) + 8.0 * batch.num_seqs * H * D * D,
                   note="walk, head norm and output gate")
            hh = rnd(T, width)
            sec = timed(lambda: moe(hh), it)
            routed, used = T * top, min(E, T * top)
            record(kern, f"lamosun.gated_experts.{tag}", sec, flops=6.0 * routed * width * eff,
                   nbytes=2.0 * (3 * used * eff * width + routed * width) + 4.0 * T * width)
    del model, caches
    torch.cuda.empty_cache()

    # ------------------------------------------------------------------ Batatar: whole steps and its kernels
    kinds = ["lightning", "parallel", "lightning", "parallel"]
    model = BatatarForCausalLM(BatatarConfig.from_dict(batatar_config(s, kinds, vocab)), dt, dev, seed=0)
    caches = model.allocate_caches(nblk, BS, B)
    fill(caches)
    whole_steps("batatar", model, caches)
    with torch.inference_mode():
        light, layer, moe = model.layers[0].recur, model.layers[1], model.layers[1].experts
        attn, ssd = layer.attn, layer.recur
        chunk = s["chunk"]
        Hl, Dl = s["l_heads"], s["l_dim"]
        Hs, Vs, N, Gs, inner, chan = s["s_heads"], s["s_vdim"], s["s_state"], s["s_groups"], ssd.inner, ssd.channels
        for tag, batch, T, it in steps:
            n_seq = batch.num_seqs
            pairs = sum(p % chunk + 1 for p in range(T)) if tag == "prefill" else B * ((C - 1) % chunk + 1)
            q, k, v, gate, out = rnd(T, H * D), rnd(T, G * D), rnd(T, G * D), rnd(T, H), rnd(T, H * D)
            if tag == "prefill":
                sec = timed(lambda: sops.kv_attention_tiles(out, q, gate, keys, values, batch.block_tables,
                                                            batch.query_start_loc, batch.context_lens,
                                                            batch.max_query_len, None, True, H, 0, attn.scale, 0,
                                                            attn.softcap, chunk, attn.sinks), it)
                record(kern, "batatar.kv_attention.prefill", sec, flops=4.0 * pairs * H * D,
                       nbytes=2.0 * T * (2 * H + 2 * G) * D, note="chunks, sink, capped scores, head gates")
            else:
                sec = timed(lambda: sops.kv_attention(out, q, gate, keys, values, batch.block_tables, batch.token_seq,
                                                      batch.positions, None, True, H, 0, attn.scale, 0, attn.softcap,
                                                      chunk, attn.sinks), it)
                record(kern, "batatar.kv_attention.decode", sec, nbytes=2 * 2.0 * G * pairs * D + 2 * 2.0 * B * H * D,
                       note="reads the chunk only")
            sec = timed(lambda: sops.rotary_kv_write(q, k, v, keys, values, batch.positions, batch.slot_mapping, None, None,
                                                     H, 0, True, norm_eps=1e-5, head_norm=True), it)
            record(kern, f"batatar.kv_write.{tag}", sec, nbytes=2.0 * T * (2 * H + 4 * G) * D,
                   note="head norms of queries and keys, cache write")
            proj = rnd(T, 4 * Hl * Dl)
            ql, kl, vl, gl = proj.split(Hl * Dl, dim=1)
            o = torch.empty(T, Hl * Dl, device=dev)
            sec = timed(lambda: sops.decay_scan(o, ql, kl, vl, caches[0]["state"], batch.query_start_loc, batch.context_lens,
                                                batch.state_slots, Hl, batch.max_query_len, light.log_decay, act="silu"), it)
            record(kern, f"batatar.decay_scan_constant.{tag}", sec, peak=FMA_F32, flops=4.0 * T * Hl * Dl * Dl,
                   nbytes=T * Hl * Dl * (3 * 2.0 + 4) + 8.0 * n_seq * Hl * Dl * Dl, note="silu on the inputs included")
            mixed = rnd(T, Hl * Dl)
            sec = timed(lambda: light(mixed, ql, kl, vl, gl, caches[0]["state"], batch), it)
            record(kern, f"batatar.lightning_layer.{tag}", sec, peak=FMA_F32, flops=4.0 * T * Hl * Dl * Dl,
                   nbytes=T * Hl * Dl * 5 * 2.0 + 8.0 * n_seq * Hl * Dl * Dl, note="recurrence, norm and gate")
            nw = light.norm_weight.data
            sec = timed(lambda: sops.gated_group_rms_norm(mixed, o, nw, gl, "sigmoid", False, 1, 1e-5), it)
            record(kern, f"batatar.gated_group_rms_norm.{tag}", sec, nbytes=T * Hl * Dl * (4.0 + 2 + 2))
            xbc, z, dts = rnd(T, chan), rnd(T, inner), rnd(T, 8 * ((Hs + 7) // 8))[:, :Hs]
            u = rnd(T, chan)
            sec = timed(lambda: ssd.conv(u, xbc, caches[1]["conv"], batch), it)
            record(kern, f"batatar.short_conv.{tag}", sec, nbytes=T * chan * 4.0 + n_seq * (s["taps"] - 1) * chan * 8.0,
                   note="bf16 in and out")
            ys = torch.empty(T, inner, device=dev)
            gn = Gs * N
            sec = timed(lambda: sops.decay_scan(ys, u[:, inner + gn:], u[:, inner:inner + gn], u[:, :inner], caches[1]["state"],
                                                batch.query_start_loc, batch.context_lens, batch.state_slots, Gs,
                                                batch.max_query_len, None, dts, ssd.dt_bias.data, ssd.a_log.data,
                                                ssd.skip.data), it)
            record(kern, f"batatar.decay_scan_ssd.{tag}", sec, peak=FMA_F32, flops=4.0 * T * Hs * N * Vs,
                   nbytes=T * (2.0 * (chan + Hs) + 4 * inner) + 8.0 * n_seq * Hs * N * Vs,
                   note="step sizes and decays included")
            out2 = rnd(T, inner)
            sec = timed(lambda: ssd(out2, z, xbc, dts, caches[1]["state"], caches[1]["conv"], batch), it)
            record(kern, f"batatar.ssd_layer.{tag}", sec, peak=FMA_F32, flops=4.0 * T * Hs * N * Vs,
                   nbytes=T * 2.0 * (chan + Hs + 2 * inner) + 8.0 * n_seq * Hs * N * Vs,
                   note="convolution, recurrence, gate and norm")
            x, y, y2, h, w = rnd(T, width, dtype=torch.float32), rnd(T, width, dtype=torch.float32), \
                rnd(T, width, dtype=torch.float32), rnd(T, width), torch.ones(width, device=dev)
            sec = timed(lambda: sops.residual_norms(x, y, out=h, pre_weight=w, eps=1e-5, y_scale=0.5), it)
            record(kern, f"batatar.stream_update.{tag}", sec, nbytes=T * width * (4.0 + 4 + 4 + 2))
            sec = timed(lambda: sops.residual_norms(x, y, None, w, None, None, h, w, 1e-5, 0.25, y2, w), it)
            record(kern, f"batatar.stream_update_two_branches.{tag}", sec, nbytes=T * width * (4.0 + 4 + 4 + 4 + 2))
            hh = rnd(T, width)
            sec = timed(lambda: moe(hh), it)
            routed, used = T * top, min(E, T * top)
            record(kern, f"batatar.experts.{tag}", sec, flops=6.0 * routed * width * eff,
                   nbytes=2.0 * (3 * used * eff * width + routed * width) + 4.0 * T * width,
                   note="route, plan, gate | up product with weighted inputs, activation, down product, combine")
    del model, caches
    torch.cuda.empty_cache()

    print(json.dumps({"metric": "prefill and decode tokens/s, Batatar beside Lusadra and Lamosun at equal size (4 layers, bf16, random weights)",
                      "size": args.arch_size, "shape": s, "prompt_tokens": P, "decode_batch": B, "decode_context": C,
                      "end_to_end": e2e, "kernels": kern, "peaks": {"hbm_Bps": HBM, "mfma_bf16": MFMA_BF16, "fma_f32": FMA_F32},
                      "time": time.strftime("%Y-%m-%d %H:%M:%S")}))
