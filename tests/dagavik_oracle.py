"""Slow reference of the Dagavik design in float64 on the CPU, one function per mechanism, written
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


# ----------------------------------------------------------------------------- embedding
def pair_embedding(tokens, embed, pairs, mul_prev, mul_cur):
    """embed[token] + pairs[(previous mul_prev + token mul_cur) mod buckets]; the last row of `pairs` (its
    number is `buckets`) where there is no previous token."""
    buckets = pairs.shape[0] - 1
    rows = [buckets] + [(a * mul_prev + b * mul_cur) % buckets for a, b in zip(tokens, tokens[1:])]
    return embed[torch.tensor(list(tokens))] + pairs[torch.tensor(rows)]


# ----------------------------------------------------------------------------- attention
def visible(n, window, first=0):
    """[n - first, n] bool: query i (from `first` on) sees key j with 0 <= i - j < window (window 0: every
    j <= i)."""
    i = torch.arange(first, n)[:, None]
    j = torch.arange(n)[None, :]
    ok = j <= i
    return ok & (i - j < window) if window else ok


def sink_softmax(s, sink=None):
    """exp(s_j) / (exp(sink) + sum_k exp(s_k)) over the last axis; entries of -inf weigh nothing.  sink
    broadcasts over all axes but the last; None: the plain softmax."""
    m = s.max(-1, keepdim=True).values
    if sink is None:
        e = torch.exp(s - m)
        return e / e.sum(-1, keepdim=True)
    m = torch.maximum(m, sink)
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - m))


def rotate_half(u, dims, base, first=0):
    """u [n, H, D] at positions first ..: elements i and i + dims / 2 of a head, i < dims / 2, turn by
    position * base^(-2i / dims)."""
    half = dims // 2
    f = torch.tensor([float(base)**(-2.0 * i / dims) for i in range(half)], dtype=F)
    a = torch.arange(first, first + u.shape[0], dtype=F)[:, None, None] * f
    x, y = u[..., :half], u[..., half:dims]
    return torch.cat([x * torch.cos(a) - y * torch.sin(a), y * torch.cos(a) + x * torch.sin(a), u[..., dims:]], -1)


def attention_core(q, k, v, scale, window=0, sink=None, first=0):
    """q [m, H, D] (queries of positions first ..), k [n, G, D], v [n, G, V] -> [m, H, V]; query head
    h reads key / value head h // (H / G); sink [H] or None."""
    H, G = q.shape[1], k.shape[1]
    kk, vv = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1)
    s = torch.einsum("ihd,jhd->hij", q, kk) * scale
    s = s.masked_fill(~visible(k.shape[0], window, first), -math.inf)
    p = sink_softmax(s, None if sink is None else sink[:, None, None])
    return torch.einsum("hij,jhv->ihv", p, vv)


def window_branch(h, t, spec):
    """t: q, k, v with biases (.b), o."""
    n = h.shape[0]
    H, G, D, V = spec["heads"], spec["kv_heads"], spec["dim"], spec["vdim"]
    rot = spec.get("rot") or {}
    q = (h @ t["q"].T + t["q.b"]).view(n, H, D)
    k = (h @ t["k"].T + t["k.b"]).view(n, G, D)
    v = (h @ t["v"].T + t["v.b"]).view(n, G, V)
    if rot.get("dims"):
        q, k = rotate_half(q, rot["dims"], rot["base"]), rotate_half(k, rot["dims"], rot["base"])
    o = attention_core(q, k, v, spec["scale"], (spec.get("mask") or {}).get("size") or 0)
    return o.reshape(n, H * V) @ t["o"].T


def latent_rows(h, t, eps):
    """The normed latent of every token: what a latent layer caches."""
    return rms_norm(h @ t["dkv"].T, t["dkv.norm"], eps)


def latent_mixer(h, t, spec, c):
    """t: q, uk, uv, sink, o; c [n, rank] (this layer's latents, or the layer's it reads)."""
    n = h.shape[0]
    H, D, V = spec["heads"], spec["dim"], spec["vdim"]
    q = (h @ t["q"].T).view(n, H, D)
    k, v = (c @ t["uk"].T).view(n, H, D), (c @ t["uv"].T).view(n, H, V)
    return attention_core(q, k, v, spec["scale"], sink=t["sink"]).reshape(n, H * V) @ t["o"].T


# ----------------------------------------------------------------------------- recurrences
def short_conv(u, w):
    """silu(sum_i w[:, i] u[t - taps + 1 + i]), zeros before the start; u [n, C], w [C, taps]."""
    n, taps = u.shape[0], w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return silu(sum(w[:, i] * pad[i:i + n] for i in range(taps)))


def channel_decay(z, a_log, dt_bias):
    """exp(-exp(a_log_h) softplus(z + dt_bias)): z [n, H, D], a_log [H], dt_bias [H, D]."""
    return torch.exp(-torch.exp(a_log)[:, None] * softplus(z + dt_bias))


def unit_vector(u):
    return u / torch.sqrt((u * u).sum(-1, keepdim=True) + 1e-6)


def delta_walk(q, k, v, g, beta, state=None):
    """Per head S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.  q, k, g [n, H, D],
    v [n, H, V], beta [n, H] -> ([n, H, V], the last state [H, D, V])."""
    n, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F) if state is None else state.clone()
    out = []
    for i in range(n):
        S = g[i][:, :, None] * S
        u = beta[i][:, None] * (v[i] - torch.einsum("hdv,hd->hv", S, k[i]))
        S = S + k[i][:, :, None] * u[:, None, :]
        out.append(torch.einsum("hdv,hd->hv", S, q[i]))
    return torch.stack(out), S


def channel_delta_mixer(h, t, spec, eps):
    """t: q, k, v with .conv, b, A_log, dt_bias, a1, a2, g1, g2, norm, o."""
    n = h.shape[0]
    H, G, D, V = spec["heads"], spec["kv_heads"], spec["dim"], spec["vdim"]
    q, k, v = (short_conv(h @ t[x].T, t[x + ".conv"]) for x in ("q", "k", "v"))
    q, k = unit_vector(q.view(n, G, D)) * D**-0.5, unit_vector(k.view(n, G, D))
    q, k = q.repeat_interleave(H // G, 1), k.repeat_interleave(H // G, 1)
    z = (h @ t["a1"].T) @ t["a2"].T
    g = channel_decay(z.view(n, H, D), t["A_log"], t["dt_bias"].view(H, D))
    o, _ = delta_walk(q, k, v.view(n, H, V), g, torch.sigmoid(h @ t["b"].T))
    gate = torch.sigmoid((h @ t["g1"].T) @ t["g2"].T)
    return (rms_norm(o, t["norm"], eps).reshape(n, H * V) * gate) @ t["o"].T


def matrix_memory_walk(q, k, v, i, f):
    """The stabilized recurrence: q, k [n, H, D], v [n, H, V], log gates i, f [n, H] -> [n, H, V]."""
    n, H, D = q.shape
    S, N, m = torch.zeros(H, D, v.shape[2], dtype=F), torch.zeros(H, D, dtype=F), torch.zeros(H, dtype=F)
    out = []
    for t in range(n):
        m_new = torch.maximum(f[t] + m, i[t])
        a, b = torch.exp(f[t] + m - m_new), torch.exp(i[t] - m_new)
        S = a[:, None, None] * S + b[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        N = a[:, None] * N + b[:, None] * k[t]
        m = m_new
        den = torch.maximum((N * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out.append(torch.einsum("hdv,hd->hv", S, q[t]) / den[:, None])
    return torch.stack(out)


def memory_gates(h, t, cap):
    """(log input gate, log forget gate) [n, H]."""
    i = cap * torch.tanh((h @ t["i"].T + t["i.b"]) / cap)
    f = cap * torch.tanh((h @ t["f"].T + t["f.b"]) / cap)
    return i, -softplus(-f)


def memory_branch(h, t, spec, eps):
    """t: q, k, v, i, f with biases (i.b, f.b), g, norm, o."""
    n = h.shape[0]
    H, D, V = spec["heads"], spec["dim"], spec["vdim"]
    q, k, v = (h @ t["q"].T).view(n, H, D) * D**-0.5, (h @ t["k"].T).view(n, H, D), (h @ t["v"].T).view(n, H, V)
    i, f = memory_gates(h, t, spec["gate_cap"])
    o = unit_rms(matrix_memory_walk(q, k, v, i, f), eps).reshape(n, H * V)
    return (o * t["norm"] * torch.sigmoid(h @ t["g"].T)) @ t["o"].T


def parallel_mixer(h, t, spec, eps):
    return spec["left_scale"] * window_branch(h, sub(t, "left."), spec["left"]) + \
        spec["right_scale"] * memory_branch(h, sub(t, "right."), spec["right"], eps)


# ----------------------------------------------------------------------------- experts
def expert(h, t):
    return (silu(h @ t["gate"].T) * (h @ t["up"].T)) @ t["down"].T


def choose(s, top, groups, keep):
    """Indices of the `top` largest entries of s [E] among the `keep` groups (of `groups` equal runs of
    neighbours) whose largest entries are largest."""
    by_group = s.view(groups, -1).max(-1).values
    allowed = torch.zeros(groups, dtype=torch.bool)
    allowed[torch.topk(by_group, keep).indices] = True
    open_to = allowed.repeat_interleave(s.shape[0] // groups)
    return torch.topk(s.masked_fill(~open_to, -math.inf), top).indices


def routed_ff(h, t, spec):
    r = spec["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    s = torch.softmax(h @ t["router"].T, -1)
    out = torch.zeros_like(h)
    for i in range(h.shape[0]):
        for e in choose(s[i], r["top"], groups["count"], groups["keep"]).tolist():
            out[i] += s[i, e] * r["scale"] * expert(h[i:i + 1], sub(t, f"e{e}."))[0]
    return out


def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


# ----------------------------------------------------------------------------- the stack
def forward(cfg, tensors, tokens, layer_out=None):
    """Logits [n, vocab] of one sequence; layer_out (a list) receives the stream after every layer."""
    t = {k: v.to(F) for k, v in tensors.items()}
    eps, bg = cfg["norm"]["eps"], cfg["embedding"]["bigram"]
    x = pair_embedding(list(tokens), t["embed"], t["bigram"], bg["mul_prev"], bg["mul_cur"])
    latents = {}
    for i, layer in enumerate(cfg["layers"]):
        lt, m = sub(t, f"l{i}."), layer["mixer"]
        mt, h = sub(lt, "mix."), rms_norm(x, 1.0 + lt["norm1"], eps)
        if layer["type"] == "latent_attention":
            src = m.get("kv_from")
            latents[i] = latents[src] if src is not None else latent_rows(h, mt, eps)
            y = latent_mixer(h, mt, m, latents[i])
        else:
            y = {"parallel": parallel_mixer, "channel_delta": channel_delta_mixer}[layer["type"]](h, mt, m, eps)
        if layer.get("mlp") is not None:
            y = y + routed_ff(rms_norm(x, 1.0 + lt["norm2"], eps), sub(lt, "mlp."), layer["mlp"])
        x = x + y
        if layer_out is not None:
            layer_out.append(x.clone())
    return rms_norm(x, 1.0 + t["final.norm"], eps) @ t["head"].T


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
def delta_layer(heads, kv_heads, dim, vdim, taps, ranks=(5, 6), mlp=None):
    """ranks: of the decay's and of the gate's two-step projections (a checkpoint's tensors carry them, a
    config does not)."""
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps},
            "mlp": mlp, "_ranks": ranks}


def parallel_layer(left, right, scales=(0.7, 0.6), mlp=None):
    """left = (heads, kv_heads, dim, vdim, window, rot dims, rot base[, scale]); right = (heads, dim, vdim,
    gate_cap)."""
    H, G, D, V, window, dims, base = left[:7]
    lm = {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": left[7] if len(left) > 7 else D**-0.5,
          "mask": {"size": window}, "rot": {"dims": dims, "base": base}}
    rm = dict(zip(("heads", "dim", "vdim", "gate_cap"), right))
    return {"type": "parallel", "mixer": {"left": lm, "right": rm, "left_scale": scales[0], "right_scale": scales[1]},
            "mlp": mlp}


def latent_layer(heads, dim, vdim, rank, scale=None, kv_from=None, mlp=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": dim**-0.5 if scale is None else scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def moe_mlp(experts, top, ff, groups=(1, 1), scale=1.5):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale,
                                                            "groups": dict(zip(("count", "keep"), groups))}}


def make_config(layers, vocab=97, width=64, eps=1e-5, bigram=(53, 31, 5)):
    return {"architecture": "Dagavik", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}, "layers": layers}


def tensor_shapes(cfg):
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "head": (V, W), "final.norm": (W, ), "bigram": (cfg["embedding"]["bigram"]["buckets"] + 1, W)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = (W, )
        q = p + "mix."
        if layer["type"] == "channel_delta":
            H, G, D, Vd, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            ra, rg = layer["_ranks"]
            for nm, rows in (("q", G * D), ("k", G * D), ("v", H * Vd)):
                out.update({q + nm: (rows, W), q + nm + ".conv": (rows, taps)})
            out.update({q + "b": (H, W), q + "A_log": (H, ), q + "norm": (Vd, ), q + "a1": (ra, W), q + "a2": (H * D, ra),
                        q + "dt_bias": (H * D, ), q + "g1": (rg, W), q + "g2": (H * Vd, rg), q + "o": (W, H * Vd)})
        elif layer["type"] == "parallel":
            le, ri = m["left"], m["right"]
            H, G, D, Vd = le["heads"], le["kv_heads"], le["dim"], le["vdim"]
            for nm, rows in (("q", H * D), ("k", G * D), ("v", G * Vd)):
                out.update({q + "left." + nm: (rows, W), q + "left." + nm + ".b": (rows, )})
            out[q + "left.o"] = (W, H * Vd)
            H, D, Vd = ri["heads"], ri["dim"], ri["vdim"]
            q += "right."
            out.update({q + "q": (H * D, W), q + "k": (H * D, W), q + "v": (H * Vd, W), q + "g": (H * Vd, W),
                        q + "o": (W, H * Vd), q + "norm": (H * Vd, ), q + "i": (H, W), q + "i.b": (H, ), q + "f": (H, W),
                        q + "f.b": (H, )})
        else:
            H, D, Vd, R = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
            out[q + "q"] = (H * D, W)
            if m.get("kv_from") is None:
                out.update({q + "dkv": (R, W), q + "dkv.norm": (R, )})
            out.update({q + "uk": (H * D, R), q + "uv": (H * Vd, R), q + "sink": (H, ), q + "o": (W, H * Vd)})
        if layer.get("mlp") is not None:
            ff, n = layer["mlp"]["expert"]["ff"], layer["mlp"]["router"]["experts"]
            out[p + "norm2"] = (W, )
            for e in range(n):
                out.update({p + f"mlp.e{e}.gate": (ff, W), p + f"mlp.e{e}.up": (ff, W), p + f"mlp.e{e}.down": (W, ff)})
            out[p + "mlp.router"] = (n, W)
    return out


def random_tensors(cfg, seed):
    """bfloat16 tensors of every checkpoint name: projections ~ N(0, 1 / fan_in) (those behind scores,
    gates and routers larger, so that they spread), norm weights around their neutral value, biases
    well away from 0, decays between about 0.2 and 0.999, sinks between about -1 and 3."""
    g = torch.Generator().manual_seed(seed)

    def randn(shape):
        return torch.randn(shape, generator=g)

    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        if name in ("embed", "bigram"):
            t = randn(shape)
        elif last in ("norm1", "norm2") or name == "final.norm":
            t = 0.2 * randn(shape)
        elif last == "norm":
            t = 1.0 + 0.2 * randn(shape)
        elif last == "A_log":
            t = torch.rand(shape, generator=g) * 1.5 - 0.5
        elif last == "dt_bias":
            t = -5.0 * torch.rand(shape, generator=g)
        elif last == "sink":
            t = 1.0 + randn(shape)
        elif name.endswith(".f.b"):
            t = 2.0 + randn(shape)
        elif name.endswith((".q.b", ".k.b", ".v.b", ".i.b")):
            t = 0.4 * randn(shape)
        else:
            t = randn(shape) * shape[-1]**-0.5
            if last in ("q", "k", "v", "i", "f", "gate", "up", "router"):
                t = t * 1.5
        out[name] = t.to(torch.bfloat16)
    return out


def public_config(cfg):
    """The config as a checkpoint's config.json has it (without the helpers' own keys)."""
    return {**cfg, "layers": [{k: v for k, v in layer.items() if not k.startswith("_")} for layer in cfg["layers"]]}


def write_checkpoint(folder, cfg, tensors):
    """config.json + model.safetensors (names sorted)."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(public_config(cfg), f)
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
