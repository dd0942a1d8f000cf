"""Slow reference of the Batatar design in float64 on the CPU, one function per mechanism, written
from the equations and sharing no code with vllm_legacy_amd.  Also the helpers that make small
random models (config dict + tensors under their checkpoint names) and write them as a
checkpoint folder.

Notation: x[t] the stream at token t (position t, counted from 0 in its sequence), W y a linear
map stored [out, in].  Every function takes one whole sequence from its first token.
"""
import json
import math
import os
import struct

import torch

F = torch.float64


def unit_rms(u, eps):
    """u / sqrt(mean(u^2) + eps) over the last axis."""
    return u / torch.sqrt((u * u).mean(-1, keepdim=True) + eps)


def rms_norm(u, w, eps):
    return unit_rms(u, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    """ln(1 + e^z), unclamped."""
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


# ----------------------------------------------------------------------------- chunked attention
def visible(n, chunk, first=0):
    """[n - first, n] bool: query i (from `first` on) sees key j <= i of its own chunk of `chunk`
    positions, chunks counted from position 0 (chunk 0: every j <= i)."""
    i = torch.arange(first, n)[:, None]
    j = torch.arange(n)[None, :]
    ok = j <= i
    if chunk:
        ok = ok & (i // chunk == j // chunk)
    return ok


def sink_softmax(s, sink=True):
    """exp(s_j) / (1 + sum_k exp(s_k)) over the last axis; entries of -inf weigh nothing.  Without a
    sink the plain softmax."""
    m = s.max(-1, keepdim=True).values
    m = torch.clamp(m, min=0.0) if sink else m
    e = torch.exp(s - m)
    z = e.sum(-1, keepdim=True)
    return e / (z + torch.exp(-m) if sink else z)


def attention_core(q, k, v, scale, softcap=0.0, chunk=0, sink=True, first=0):
    """q [m, H, D] (queries of positions first ..), k [n, G, D], v [n, G, V] -> [m, H, V]; query head
    h reads key / value head h // (H / G)."""
    H, G = q.shape[1], k.shape[1]
    kk, vv = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1)
    s = torch.einsum("ihd,jhd->hij", q, kk) * scale
    if softcap:
        s = softcap * torch.tanh(s / softcap)
    s = s.masked_fill(~visible(k.shape[0], chunk, first), -math.inf)
    return torch.einsum("hij,jhv->ihv", sink_softmax(s, sink), vv)


def attention_branch(h, t, spec, eps):
    """t: q, k, v with biases (.b), g, o."""
    n = h.shape[0]
    H, G, D, V = spec["heads"], spec["kv_heads"], spec["dim"], spec["vdim"]
    q = unit_rms((h @ t["q"].T + t["q.b"]).view(n, H, D), eps)
    k = unit_rms((h @ t["k"].T + t["k.b"]).view(n, G, D), eps)
    v = (h @ t["v"].T + t["v.b"]).view(n, G, V)
    o = attention_core(q, k, v, spec["scale"], spec.get("softcap") or 0.0, (spec.get("mask") or {}).get("size") or 0)
    return (o * torch.sigmoid(h @ t["g"].T)[:, :, None]).reshape(n, H * V) @ t["o"].T


# ----------------------------------------------------------------------------- recurrences
def short_conv(u, w, bias):
    """silu(bias + sum_i w[:, i] u[t - taps + 1 + i]), zeros before the start; u [n, C], w [C, taps]."""
    n, taps = u.shape[0], w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return silu(bias + sum(w[:, i] * pad[i:i + n] for i in range(taps)))


def decayed_walk(q, k, v, a, state=None):
    """S_t = a_t S_(t-1) + k_t v_t^T, o_t = S_t^T q_t per head: q, k [n, H, D], v [n, H, V], a [n, H] ->
    ([n, H, V], the last state [H, D, V])."""
    n, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F) if state is None else state.clone()
    out = []
    for t in range(n):
        S = a[t][:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out), S


def ssd_walk(x, B, C, dt, a_log, dt_bias, D):
    """The state-space recurrence: x [n, H, V], B, C [n, G, N], dt [n, H] before its softplus -> [n, H, V]."""
    H, G = x.shape[1], B.shape[1]
    step = softplus(dt + dt_bias)
    a = torch.exp(-torch.exp(a_log) * step)
    Bh, Ch = B.repeat_interleave(H // G, 1), C.repeat_interleave(H // G, 1)
    y, _ = decayed_walk(Ch, Bh, step[:, :, None] * x, a)
    return y + D[None, :, None] * x


def grouped_gated_norm(y, z, w, groups, eps):
    """y silu(z), each of `groups` equal parts divided by its own root mean square, times w."""
    u = y * silu(z)
    return unit_rms(u.view(u.shape[0], groups, -1), eps).reshape(u.shape) * w


def ssd_branch(h, t, spec, eps):
    """t: in, conv, conv.b, dt_bias, A_log, D, norm, o."""
    n = h.shape[0]
    H, V, N, G = spec["heads"], spec["vdim"], spec["state"], spec["groups"]
    inner = H * V
    p = h @ t["in"].T
    z, u, dt = p[:, :inner], p[:, inner:2 * inner + 2 * G * N], p[:, 2 * inner + 2 * G * N:]
    u = short_conv(u, t["conv"], t["conv.b"])
    y = ssd_walk(u[:, :inner].view(n, H, V), u[:, inner:inner + G * N].view(n, G, N), u[:, inner + G * N:].view(n, G, N),
                 dt, t["A_log"], t["dt_bias"], t["D"])
    return grouped_gated_norm(y.reshape(n, inner), z, t["norm"], spec["norm_groups"], eps) @ t["o"].T


def parallel_mixer(h, t, spec, eps):
    left = attention_branch(h, sub(t, "left."), spec["left"], eps)
    right = ssd_branch(h, sub(t, "right."), spec["right"], eps)
    return 0.5 * (rms_norm(left, t["left.out"], eps) + rms_norm(right, t["right.out"], eps))


def lightning_mixer(h, t, spec, eps):
    """t: q, k, v, g, norm, o."""
    n = h.shape[0]
    H, D, V = spec["heads"], spec["dim"], spec["vdim"]
    q, k = silu(h @ t["q"].T).view(n, H, D), silu(h @ t["k"].T).view(n, H, D)
    v = silu(h @ t["v"].T).view(n, H, V)
    a = torch.tensor(spec["decay"], dtype=F).expand(n, H)
    o, _ = decayed_walk(q, k, v, a)
    return (rms_norm(o.reshape(n, H * V), t["norm"], eps) * torch.sigmoid(h @ t["g"].T)) @ t["o"].T


# ----------------------------------------------------------------------------- experts
def expert(h, t):
    return (silu(h @ t["gate"].T) * (h @ t["up"].T)) @ t["down"].T


def routed_ff(h, t, spec):
    """The `top` largest sigmoid(z) choose, their values multiply the chosen experts' inputs."""
    s = torch.sigmoid(h @ t["router"].T)
    val, idx = torch.topk(s, spec["router"]["top"], dim=-1)
    out = torch.zeros_like(h)
    for i in range(h.shape[0]):
        for kx in range(idx.shape[1]):
            out[i] += expert(val[i, kx] * h[i:i + 1], sub(t, f"e{int(idx[i, kx])}."))[0]
    return out


def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


# ----------------------------------------------------------------------------- the stack
def layer_order(cfg):
    """[(layer, number of the pass it opens or None)]: layers start .. stop - 1 run `times` times."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    runs = [(i, None) for i in range(a)]
    for p in range(loop["times"]):
        runs += [(i, p if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


def open_pass(x, x0, w_in, step):
    return torch.cat([x, x0], -1) @ w_in.T + step


def forward(cfg, tensors, tokens, layer_out=None):
    """Logits [n, vocab] of one sequence; layer_out (a list) receives the stream after every layer run."""
    t = {k: v.to(F) for k, v in tensors.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x0 = x = t["embed"][torch.tensor(list(tokens))]
    for i, opens in layer_order(cfg):
        layer, lt = cfg["layers"][i], sub(t, f"l{i}.")
        if opens is not None:
            x = open_pass(x, x0, t["loop.in"], t["loop.step"][opens])
        mixer = {"parallel": parallel_mixer, "lightning": lightning_mixer}[layer["type"]]
        x = x + m * mixer(rms_norm(x, lt["norm1"], eps), sub(lt, "mix."), layer["mixer"], eps)
        if layer.get("mlp") is not None:
            x = x + m * routed_ff(rms_norm(x, lt["norm2"], eps), sub(lt, "mlp."), layer["mlp"])
        if layer_out is not None:
            layer_out.append(x.clone())
    return rms_norm(x, t["final.norm"], eps) @ t["head"].T


def spread(logits):
    """Root mean square over a request of the logits with each row's mean taken off."""
    d = logits - logits.mean(-1, keepdim=True)
    return torch.sqrt((d * d).mean())


def row_errors(got, want):
    """Per row: rms over the vocabulary of the difference with its mean taken off."""
    d = got.to(F) - want.to(F)
    d = d - d.mean(-1, keepdim=True)
    return torch.sqrt((d * d).mean(-1))


# ----------------------------------------------------------------------------- small random models
def lightning_layer(heads, dim, vdim=None, decay=None, mlp=None):
    if decay is None:
        decay = [1.0 - 2.0**-(1.0 + 6.0 * h / max(heads - 1, 1)) for h in range(heads)]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim or dim, "decay": decay}, "mlp": mlp}


def parallel_layer(left, right, mlp=None):
    """left = (heads, kv_heads, dim, vdim, chunk, softcap[, scale]); right = (heads, vdim, state, groups,
    norm_groups, taps)."""
    H, G, D, V, chunk, cap = left[:6]
    lm = {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": left[6] if len(left) > 6 else D**-0.5,
          "mask": {"size": chunk}, "softcap": cap}
    rm = dict(zip(("heads", "vdim", "state", "groups", "norm_groups", "conv"), right))
    return {"type": "parallel", "mixer": {"left": lm, "right": rm}, "mlp": mlp}


def moe_mlp(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def make_config(layers, vocab=97, width=64, eps=1e-5, residual_mult=0.6, loop=None):
    cfg = {"architecture": "Batatar", "vocab": vocab, "width": width, "norm": {"eps": eps},
           "residual_mult": residual_mult, "layers": layers}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def tensor_shapes(cfg):
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "head": (V, W), "final.norm": (W, )}
    if cfg.get("loop"):
        out.update({"loop.in": (W, 2 * W), "loop.step": (cfg["loop"]["times"], W)})
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = (W, )
        if layer["type"] == "lightning":
            H, D, Vd = m["heads"], m["dim"], m["vdim"]
            out.update({p + "mix.q": (H * D, W), p + "mix.k": (H * D, W), p + "mix.v": (H * Vd, W), p + "mix.g": (H * Vd, W),
                        p + "mix.norm": (H * Vd, ), p + "mix.o": (W, H * Vd)})
        else:
            le, ri = m["left"], m["right"]
            H, G, D, Vd = le["heads"], le["kv_heads"], le["dim"], le["vdim"]
            q = p + "mix.left."
            out.update({q + "q": (H * D, W), q + "q.b": (H * D, ), q + "k": (G * D, W), q + "k.b": (G * D, ),
                        q + "v": (G * Vd, W), q + "v.b": (G * Vd, ), q + "g": (H, W), q + "o": (W, H * Vd), q + "out": (W, )})
            R, inner, chan = ri["heads"], ri["heads"] * ri["vdim"], ri["heads"] * ri["vdim"] + 2 * ri["groups"] * ri["state"]
            q = p + "mix.right."
            out.update({q + "in": (inner + chan + R, W), q + "conv": (chan, ri["conv"]), q + "conv.b": (chan, ),
                        q + "dt_bias": (R, ), q + "A_log": (R, ), q + "D": (R, ), q + "norm": (inner, ), q + "o": (W, inner),
                        q + "out": (W, )})
        if layer.get("mlp") is not None:
            ff, n = layer["mlp"]["expert"]["ff"], layer["mlp"]["router"]["experts"]
            out[p + "norm2"] = (W, )
            for e in range(n):
                out.update({p + f"mlp.e{e}.gate": (ff, W), p + f"mlp.e{e}.up": (ff, W), p + f"mlp.e{e}.down": (W, ff)})
            out[p + "mlp.router"] = (n, W)
    return out


def random_tensors(cfg, seed):
    """bfloat16 tensors of every checkpoint name: projections ~ N(0, 1 / fan_in) (expert inputs and the
    mixers' inputs larger, so that gates and scores spread), norm weights around 1, biases well away
    from 0, decays exp(-exp(A_log) softplus(dt + dt_bias)) between about 0.2 and 0.999."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        if name == "embed":
            t = torch.randn(shape, generator=g)
        elif last in ("norm", "norm1", "norm2", "out"):
            t = 1.0 + 0.2 * torch.randn(shape, generator=g)
        elif last == "A_log":
            t = torch.rand(shape, generator=g) * 1.5 - 0.5
        elif last == "dt_bias":
            t = -5.0 * torch.rand(shape, generator=g)
        elif last == "D":
            t = 0.5 + 0.5 * torch.randn(shape, generator=g)
        elif last == "b" or name == "loop.step":
            t = 0.4 * torch.randn(shape, generator=g)
        elif last == "conv":
            t = torch.randn(shape, generator=g) * shape[-1]**-0.5
        else:
            t = torch.randn(shape, generator=g) * shape[-1]**-0.5
            if last in ("q", "k", "v", "g", "in", "gate", "up"):
                t = t * 1.5
        out[name] = t.to(torch.bfloat16)
    return out


def write_checkpoint(folder, cfg, tensors):
    """config.json + model.safetensors (names sorted)."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, off = {}, [], 0
    for name in sorted(tensors):
        t = tensors[name].contiguous()
        code = {torch.bfloat16: "BF16", torch.float32: "F32", torch.int32: "I32"}[t.dtype]
        raw = t.reshape(-1).view(torch.uint8).numpy().tobytes() if t.numel() else b""
        header[name] = {"dtype": code, "shape": list(t.shape), "data_offsets": [off, off + len(raw)]}
        blobs.append(raw)
        off += len(raw)
    hj = json.dumps(header).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(hj)))
        f.write(hj)
        for b in blobs:
            f.write(b)
    return folder
