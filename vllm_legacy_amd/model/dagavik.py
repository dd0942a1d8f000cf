"""Dagavik: a decoder-only stack over an fp32 stream whose layers add a mixer and a routed feed-forward
that both read the stream of the layer's start, each through a norm of its own.

  x = embed[token] + bigram[(previous * mul_prev + token * mul_cur) mod buckets]   (the last row of
      the second table for a sequence's first token)
  layer:  x <- x + mixer(N1(x)) + ff(N2(x))       N(u) = u / sqrt(mean(u^2) + eps) * (1 + w)
          (a layer may have no ff)
  mixer 'channel_delta':  q, k (kv_heads x dim), v (heads x vdim), each through a short causal
          convolution and silu; q, k unit vectors per head, q times dim^-1/2; beta = sigmoid(W_b h);
          g = exp(-exp(A_log) softplus(W_a2 W_a1 h + dt_bias)) per head and key channel; per head
          S <- diag(g) S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q; o / rms(o) * w *
          sigmoid(W_g2 W_g1 h), then W_o
  mixer 'parallel':  left_scale * left + right_scale * right
          left: softmax attention over a sliding window, grouped queries, biases on q, k and v, rotary
          positions on the first rot.dims of q and k (rotate-half pairs)
          right: matrix memory with exponential gates, q times dim^-1/2; each head's o / rms(o) * w *
          sigmoid(W_g h), then W_o
  mixer 'latent_attention':  q = W_q h; the latent c = W_dkv h / rms * w is cached; keys W_uk c, values
          W_uv c; causal softmax without positions, with a sink per head; W_o.  With 'kv_from' the
          layer has no W_dkv and reads the latents that layer caches
  ff:     the `top` experts of largest s = softmax(W_r h) among the experts of the groups.keep best
          groups, weighted by s * scale, experts W_down (silu(W_gate h) * W_up h)
  logits = head N_final(x)

All sizes and per-model constants come from config.json (the ranks of the two-step projections of a
channel_delta layer from their tensors' shapes); a layer entry carries its own mixer and feed-forward
sizes.  The projections that read h are one matrix product per mixer (the matrix memory's gates, which an
exponential follows, come from one with an fp32 result); matrix products go to the vendor library,
everything else runs on libvla_seq_gfx950.so.  The stream, norms, angles, attention scores and weights,
routers, gates of the recurrences and recurrent states are fp32 whatever `dtype` is; `dtype` is the type
of weights, projections, caches and activations (bfloat16 to serve, float32 for an all-fp32 run).  A
layer's branches join the stream in the launch that norms it for the next layer's two readers.
"""
import json
from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import torch
import torch.nn as nn

from vllm_legacy_amd import _seq_ops as ops
from vllm_legacy_amd.attention.backends.latent_kv import LatentKVAttention
from vllm_legacy_amd.attention.backends.rotary_kv import RotaryKVAttention
from vllm_legacy_amd.attention.batch import SequenceBatch
from vllm_legacy_amd.attention.recurrent import ChannelDeltaRule, MatrixMemory
from vllm_legacy_amd.layers import PairHashEmbedding, ShortConv
from vllm_legacy_amd.routed_experts import RoutedExperts, mm_f32

ANY = -1        # a dimension only the checkpoint's tensors know


@dataclass
class ChannelDeltaSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int


@dataclass
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int                 # 0: none
    rot_dims: int
    rot_base: float


@dataclass
class MemorySpec:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass
class ParallelSpec:
    left: AttentionSpec
    right: MemorySpec
    left_scale: float
    right_scale: float


@dataclass
class LatentSpec:
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    scale: float
    kv_from: Optional[int]      # the layer whose latents this one reads


@dataclass
class MlpSpec:
    ff: int
    experts: int
    top: int
    scale: float
    groups: int
    keep_groups: int


@dataclass
class LayerSpec:
    type: str                   # channel_delta | parallel | latent_attention
    mixer: object
    mlp: Optional[MlpSpec]


def _mixer_spec(kind: str, m: Dict):
    if kind == "channel_delta":
        spec = ChannelDeltaSpec(int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]),
                                int(m.get("vdim", m["dim"])), int(m.get("conv", 1)))
        if spec.heads % spec.kv_heads or spec.taps < 1:
            raise ValueError("heads / kv_heads / conv do not fit")
        return spec
    if kind == "parallel":
        le, ri = m["left"], m["right"]
        rot, dim = le.get("rot") or {}, int(le["dim"])
        left = AttentionSpec(int(le["heads"]), int(le.get("kv_heads", le["heads"])), dim, int(le.get("vdim", dim)),
                             float(le.get("scale", dim**-0.5)), int((le.get("mask") or {}).get("size") or 0),
                             int(rot.get("dims", 0)), float(rot.get("base", 10000.0)))
        if left.heads % left.kv_heads or left.window < 0:
            raise ValueError("left.heads / left.kv_heads / left.mask.size do not fit")
        if left.rot_dims % 2 or not 0 <= left.rot_dims <= dim:
            raise ValueError("left.rot.dims does not fit left.dim")
        right = MemorySpec(int(ri["heads"]), int(ri["dim"]), int(ri.get("vdim", ri["dim"])), float(ri["gate_cap"]))
        if not right.gate_cap > 0:
            raise ValueError("right.gate_cap must be positive")
        return ParallelSpec(left, right, float(m.get("left_scale", 1.0)), float(m.get("right_scale", 1.0)))
    if kind == "latent_attention":
        dim, src = int(m["dim"]), m.get("kv_from")
        return LatentSpec(int(m["heads"]), dim, int(m.get("vdim", dim)), int(m["kv_rank"]),
                          float(m.get("scale", dim**-0.5)), None if src is None else int(src))
    raise ValueError(f"unknown layer type {kind!r}")


def _mlp_spec(mlp: Optional[Dict]) -> Optional[MlpSpec]:
    if mlp is None:
        return None
    if mlp.get("kind") != "moe":
        raise ValueError(f"unknown feed-forward kind {mlp.get('kind')!r}")
    r = mlp["router"]
    groups = r.get("groups") or {}
    count = int(groups.get("count", 1))
    spec = MlpSpec(int(mlp["expert"]["ff"]), int(r["experts"]), int(r["top"]), float(r.get("scale", 1.0)), count,
                   int(groups.get("keep", count)))
    if spec.groups < 1 or spec.experts % spec.groups or not 1 <= spec.keep_groups <= spec.groups:
        raise ValueError("router.groups does not fit the number of experts")
    if not 1 <= spec.top <= spec.keep_groups * (spec.experts // spec.groups):
        raise ValueError("router.top does not fit the number of experts that can be chosen")
    return spec


@dataclass
class DagavikConfig:
    vocab: int
    width: int
    eps: float
    buckets: int
    mul_prev: int
    mul_cur: int
    layers: List[LayerSpec]
    architecture: str = "Dagavik"
    raw: Dict = field(default_factory=dict, repr=False)

    @staticmethod
    def from_dict(d: Dict) -> "DagavikConfig":
        layers: List[LayerSpec] = []
        for i, entry in enumerate(d["layers"]):
            try:
                layers.append(LayerSpec(entry.get("type"), _mixer_spec(entry.get("type"), entry.get("mixer") or {}),
                                        _mlp_spec(entry.get("mlp"))))
                src = getattr(layers[i].mixer, "kv_from", None)
                if src is not None:
                    if not 0 <= src < i or layers[src].type != "latent_attention" or \
                            layers[src].mixer.kv_from is not None:
                        raise ValueError("kv_from must name an earlier layer that forms latents of its own")
                    if layers[src].mixer.kv_rank != layers[i].mixer.kv_rank:
                        raise ValueError("kv_from names a layer of another kv_rank")
            except ValueError as e:
                raise ValueError(f"layer {i}: {e}") from None
        bg = d["embedding"]["bigram"]
        return DagavikConfig(int(d["vocab"]), int(d["width"]), float(d["norm"]["eps"]), int(bg["buckets"]),
                             int(bg["mul_prev"]), int(bg["mul_cur"]), layers, d.get("architecture", "Dagavik"), d)

    @staticmethod
    def from_json(path: str) -> "DagavikConfig":
        with open(path) as f:
            return DagavikConfig.from_dict(json.load(f))


@dataclass
class Pending:
    """A layer's branches that are not in the stream yet: x += sum factor * y + the experts' weighted rows."""
    terms: List[Tuple[torch.Tensor, float]] = field(default_factory=list)
    experts: Optional[Tuple[torch.Tensor, torch.Tensor, torch.Tensor]] = None


def _pad8(n: int) -> int:
    return (n + 7) // 8 * 8


def _shape_fits(shape, expected) -> bool:
    return len(shape) == len(expected) and all(e in (ANY, s) for s, e in zip(shape, expected))


class DagavikLayer(nn.Module):

    def __init__(self, cfg: DagavikConfig, spec: LayerSpec, dtype, device):
        super().__init__()
        self.spec, self.dtype, self.eps, W = spec, dtype, cfg.eps, cfg.width

        def vec(n=W):
            return nn.Parameter(torch.ones(n, dtype=torch.float32, device=device), requires_grad=False)

        def mat(rows, cols):
            return nn.Parameter(torch.zeros((rows, cols), dtype=dtype, device=device), requires_grad=False)

        self.norm1 = vec()              # the norms hold 1 + w
        m = spec.mixer
        # the merged input projection: (checkpoint name, rows, has a bias)
        if spec.type == "channel_delta":
            qk, v = m.kv_heads * m.dim, m.heads * m.vdim
            self.in_parts = [("mix.q", qk, False), ("mix.k", qk, False), ("mix.v", v, False), ("mix.b", m.heads, False),
                             ("mix.a1", ANY, False), ("mix.g1", ANY, False)]
            # q, k and v pass one convolution over their stretch of the merged row, padding included
            self.conv = ShortConv(2 * _pad8(qk) + _pad8(v), m.taps, False, "silu", device)
            self.recur = ChannelDeltaRule(m.heads, m.kv_heads, m.dim, m.vdim, cfg.eps, device)
            self.w_out = mat(W, v)
            # second steps of the decay's and of the gate's projections; columns padded to eight
            self.w_decay, self.w_gate = mat(m.heads * m.dim, 0), mat(v, 0)
        elif spec.type == "parallel":
            le, ri = m.left, m.right
            self.attn = RotaryKVAttention(le.heads, le.kv_heads, le.dim, le.vdim, le.scale, le.rot_dims, le.rot_base,
                                          interleaved=False, window=le.window or None, device=device)
            self.recur = MatrixMemory(ri.heads, ri.dim, ri.vdim, ri.gate_cap, cfg.eps, device)
            qk, v = ri.heads * ri.dim, ri.heads * ri.vdim
            self.in_parts = [("mix.left.q", le.heads * le.dim, True), ("mix.left.k", le.kv_heads * le.dim, True),
                             ("mix.left.v", le.kv_heads * le.vdim, True), ("mix.right.q", qk, False),
                             ("mix.right.k", qk, False), ("mix.right.v", v, False), ("mix.right.g", v, False)]
            self.w_out, self.w_out2 = mat(W, le.heads * le.vdim), mat(W, v)
            self.w_gates = mat(2 * _pad8(ri.heads), W)          # input gates, then forget gates
        else:
            own = m.kv_from is None
            self.attn = LatentKVAttention(m.heads, m.dim, 0, m.vdim, m.kv_rank, m.scale, 0, 1.0, None, cfg.eps, dtype,
                                          device, sinks=True, own_latent=own)
            self.in_parts = [("mix.q", m.heads * m.dim, False)] + ([("mix.dkv", m.kv_rank, False)] if own else [])
            self.w_out = mat(W, m.heads * m.vdim)
        self._place_parts(W, device)
        mlp = spec.mlp
        if mlp is not None:
            self.norm2 = vec()
            self.experts = RoutedExperts(W, mlp.experts, 0, mlp.top, mlp.ff, act="silu", dtype=dtype, device=device,
                                         gated=True, renormalize=False, groups=mlp.groups, keep_groups=mlp.keep_groups,
                                         weight_scale=mlp.scale)

    def _place_parts(self, W: int, device) -> None:
        """Every part of the merged projection starts on a multiple of eight rows, so that each part of a
        result row starts 16-byte aligned; parts of unknown size have no rows until the weights come."""
        self.in_starts, rows = [], 0
        for _, n, _ in self.in_parts:
            self.in_starts.append(rows)
            rows += _pad8(max(n, 0))
        self.w_in = nn.Parameter(torch.zeros((rows, W), dtype=self.dtype, device=device), requires_grad=False)
        self.b_in = nn.Parameter(torch.zeros(rows, dtype=self.dtype, device=device), requires_grad=False) \
            if any(b for _, _, b in self.in_parts) else None

    # ------------------------------------------------------------------ weights
    def tensor_shapes(self, cfg: DagavikConfig) -> Dict[str, Tuple[int, ...]]:
        """Checkpoint names (without the layer prefix) and shapes of this layer's tensors; ANY where a
        config does not say (until the weights are in)."""
        W, m, mlp = cfg.width, self.spec.mixer, self.spec.mlp
        t: Dict[str, Tuple[int, ...]] = {"norm1": (W, )}
        for name, n, bias in self.in_parts:
            t[name] = (n, W)
            if bias:
                t[name + ".b"] = (n, )
        if self.spec.type == "channel_delta":
            sizes = {name: n for name, n, _ in self.in_parts}
            for x in ("mix.q", "mix.k", "mix.v"):
                t[x + ".conv"] = (sizes[x], m.taps)
            t.update({"mix.A_log": (m.heads, ), "mix.dt_bias": (m.heads * m.dim, ), "mix.norm": (m.vdim, ),
                      "mix.a2": (m.heads * m.dim, sizes["mix.a1"]), "mix.g2": (m.heads * m.vdim, sizes["mix.g1"]),
                      "mix.o": (W, m.heads * m.vdim)})
        elif self.spec.type == "parallel":
            le, ri = m.left, m.right
            t.update({"mix.left.o": (W, le.heads * le.vdim), "mix.right.o": (W, ri.heads * ri.vdim),
                      "mix.right.norm": (ri.heads * ri.vdim, ), "mix.right.i": (ri.heads, W), "mix.right.i.b": (ri.heads, ),
                      "mix.right.f": (ri.heads, W), "mix.right.f.b": (ri.heads, )})
        else:
            t.update({"mix.uk": (m.heads * m.dim, m.kv_rank), "mix.uv": (m.heads * m.vdim, m.kv_rank),
                      "mix.sink": (m.heads, ), "mix.o": (W, m.heads * m.vdim)})
            if m.kv_from is None:
                t["mix.dkv.norm"] = (m.kv_rank, )
        if mlp is not None:
            t["norm2"] = (W, )
            for e in range(mlp.experts):
                t.update({f"mlp.e{e}.gate": (mlp.ff, W), f"mlp.e{e}.up": (mlp.ff, W), f"mlp.e{e}.down": (W, mlp.ff)})
            t["mlp.router"] = (mlp.experts, W)
        return t

    def set_weights(self, t: Dict[str, torch.Tensor], cfg: DagavikConfig) -> None:
        """t: this layer's tensors by their names without the layer prefix."""
        dev, dt, W = self.w_in.device, self.dtype, cfg.width

        def check():
            for name, shape in self.tensor_shapes(cfg).items():
                if name not in t:
                    raise KeyError(f"tensor {name} is missing")
                if not _shape_fits(t[name].shape, shape):
                    raise ValueError(f"{name}: shape {tuple(t[name].shape)}, expected {shape}")

        def f32(name):
            return t[name].float().to(dev).contiguous()

        def put(param, value):
            param.data = value.to(param.dtype).to(dev).contiguous()

        check()
        if any(n == ANY for _, n, _ in self.in_parts):
            self.in_parts = [(name, t[name].shape[0], b) for name, _, b in self.in_parts]
            self._place_parts(W, dev)
            check()                     # now with the ranks that the first steps' tensors have
        self.norm1.data = 1.0 + f32("norm1")
        merged = torch.zeros(tuple(self.w_in.shape), dtype=dt)
        bias = torch.zeros(self.w_in.shape[0], dtype=dt)
        for (name, n, has_bias), start in zip(self.in_parts, self.in_starts):
            merged[start:start + n] = t[name].to(dt)
            if has_bias:
                bias[start:start + n] = t[name + ".b"].to(dt)
        put(self.w_in, merged)
        if self.b_in is not None:
            put(self.b_in, bias)
        if self.spec.type == "channel_delta":
            put(self.w_out, t["mix.o"])
            self.recur.set_weights(t["mix.A_log"], t["mix.dt_bias"], t["mix.norm"])
            taps = torch.zeros(tuple(self.conv.weight.shape), dtype=torch.float32)
            for (name, n, _), start in zip(self.in_parts[:3], self.in_starts):
                taps[start:start + n] = t[name + ".conv"].float()
            put(self.conv.weight, taps)

            def padded(w):
                return torch.nn.functional.pad(w, (0, _pad8(w.shape[1]) - w.shape[1]))

            put(self.w_decay, padded(t["mix.a2"]))
            put(self.w_gate, padded(t["mix.g2"]))
        elif self.spec.type == "parallel":
            put(self.w_out, t["mix.left.o"])
            put(self.w_out2, t["mix.right.o"])
            H = self.spec.mixer.right.heads
            gates = torch.zeros(tuple(self.w_gates.shape), dtype=dt)
            gates[:H], gates[_pad8(H):_pad8(H) + H] = t["mix.right.i"].to(dt), t["mix.right.f"].to(dt)
            put(self.w_gates, gates)
            self.recur.bias_i.data, self.recur.bias_f.data = f32("mix.right.i.b"), f32("mix.right.f.b")
            self.recur.norm_weight.data = f32("mix.right.norm")
        else:
            put(self.w_out, t["mix.o"])
            self.attn.set_weights(t["mix.uk"], t["mix.uv"], t.get("mix.dkv.norm"), t["mix.sink"])
        if self.spec.mlp is not None:
            self.norm2.data = 1.0 + f32("norm2")
            self.experts.set_weights({k[4:]: v for k, v in t.items() if k.startswith("mlp.")})

    # ------------------------------------------------------------------ caches
    def cache_shapes(self, cfg: DagavikConfig, num_blocks: int, block_size: int, num_slots: int):
        """name -> (shape, dtype) of what this layer keeps between steps (a layer that reads another
        layer's latents keeps nothing)."""
        m = self.spec.mixer
        if self.spec.type == "channel_delta":
            out = {"state": (ChannelDeltaRule.get_state_shape(num_slots, m.heads, m.dim, m.vdim), torch.float32)}
            if m.taps > 1:
                out["conv"] = (ShortConv.get_state_shape(num_slots, self.conv.channels, m.taps), torch.float32)
            return out
        if self.spec.type == "parallel":
            le, ri = m.left, m.right
            ks, vs = RotaryKVAttention.get_cache_shapes(num_blocks, block_size, le.kv_heads, le.dim, le.vdim)
            memory, maximum = MatrixMemory.get_state_shapes(num_slots, ri.heads, ri.dim, ri.vdim)
            return {"keys": (ks, self.dtype), "values": (vs, self.dtype), "memory": (memory, torch.float32),
                    "maximum": (maximum, torch.float32)}
        if m.kv_from is not None:
            return {}
        return {"latent": (LatentKVAttention.get_cache_shape(num_blocks, block_size, m.kv_rank, 0), self.dtype)}

    # ------------------------------------------------------------------ forward
    def _mix(self, h: torch.Tensor, batch: SequenceBatch,
             cache: Dict[str, torch.Tensor]) -> List[Tuple[torch.Tensor, float]]:
        T, dev, m = h.shape[0], h.device, self.spec.mixer
        proj = torch.mm(h, self.w_in.data.t()) if self.b_in is None else torch.addmm(self.b_in.data, h, self.w_in.data.t())
        parts = [proj[:, s:s + n] for s, (_, n, _) in zip(self.in_starts, self.in_parts)]
        mixed = torch.empty((T, self.w_out.shape[1]), dtype=self.dtype, device=dev)
        if self.spec.type == "channel_delta":
            u = torch.empty((T, self.conv.channels), dtype=self.dtype, device=dev)
            self.conv(u, proj[:, :self.conv.channels], cache.get("conv"), batch)
            q, k, v = (u[:, s:s + n] for s, (_, n, _) in zip(self.in_starts[:3], self.in_parts))
            a1, g1 = (proj[:, s:s + w.shape[1]] for s, w in zip(self.in_starts[4:], (self.w_decay, self.w_gate)))
            gate = torch.mm(g1, self.w_gate.data.t())
            self.recur(mixed, q, k, v, gate, parts[3], mm_f32(a1, self.w_decay.data), cache["state"], batch)
            return [(mm_f32(mixed, self.w_out.data), 1.0)]
        if self.spec.type == "parallel":
            q, k, v, q2, k2, v2, gate = parts
            self.attn(mixed, q, k, v, None, cache["keys"], cache["values"], batch)
            z = mm_f32(h, self.w_gates.data)
            H, F = m.right.heads, z.shape[1] // 2
            right = torch.empty((T, self.w_out2.shape[1]), dtype=self.dtype, device=dev)
            self.recur(right, q2, k2, v2, gate, z[:, :H], z[:, F:F + H], cache["memory"], cache["maximum"], batch)
            return [(mm_f32(mixed, self.w_out.data), m.left_scale), (mm_f32(right, self.w_out2.data), m.right_scale)]
        mixed = self.attn(parts[0], parts[1] if m.kv_from is None else None, cache["latent"], batch)
        return [(mm_f32(mixed, self.w_out.data), 1.0)]

    def forward(self, x: torch.Tensor, batch: SequenceBatch, cache: Dict[str, torch.Tensor], pending: Pending) -> Pending:
        """x: fp32 [T, width], updated in place with what is pending; this layer's branches come back as
        Pending (the next norms' launch adds them)."""
        h = torch.empty((2, ) + tuple(x.shape), dtype=self.dtype, device=x.device)
        readers = [(h[0], self.norm1.data)] + ([(h[1], self.norm2.data)] if self.spec.mlp is not None else [])
        ops.branch_sum_norms(x, pending.terms, pending.experts, readers, self.eps)
        terms = self._mix(h[0], batch, cache)
        return Pending(terms, self.experts.rows(h[1])[:3] if self.spec.mlp is not None else None)


class DagavikForCausalLM(nn.Module):
    """The stack and its per-layer caches.  `seed` fills random weights (benchmarks); load_weights
    installs a checkpoint's."""

    architecture = "Dagavik"

    def __init__(self, cfg: DagavikConfig, dtype=torch.bfloat16, device="cuda", seed: Optional[int] = None):
        super().__init__()
        self.cfg, self.dtype = cfg, dtype
        self.embed = PairHashEmbedding(cfg.vocab, cfg.width, cfg.buckets, cfg.mul_prev, cfg.mul_cur, dtype, device)
        self.layers = nn.ModuleList([DagavikLayer(cfg, s, dtype, device) for s in cfg.layers])
        self.final_norm = nn.Parameter(torch.ones(cfg.width, dtype=torch.float32, device=device), requires_grad=False)
        self.head = nn.Parameter(torch.zeros((cfg.vocab, cfg.width), dtype=dtype, device=device), requires_grad=False)
        if seed is not None:
            self.load_weights(self.random_weights(seed))

    # ------------------------------------------------------------------ caches
    def cache_spec(self) -> List[Dict[str, Tuple[int, ...]]]:
        """Per layer: the shapes of its caches for one block of one token and one slot; last, the
        embedding's state for one slot."""
        return [{k: v[0] for k, v in layer.cache_shapes(self.cfg, 1, 1, 1).items()} for layer in self.layers] + \
            [{"last_token": PairHashEmbedding.get_state_shape(1)}]

    def allocate_caches(self, num_blocks: int, block_size: int, num_slots: int):
        """One entry per layer (a layer with kv_from has the entry of the layer it reads), then the
        embedding's state (a sequence's last token, by state slot)."""
        dev = self.head.device
        caches: List[Dict[str, torch.Tensor]] = []
        for layer in self.layers:
            src = getattr(layer.spec.mixer, "kv_from", None)
            caches.append(caches[src] if src is not None else
                          {name: torch.zeros(shape, dtype=dt, device=dev)
                           for name, (shape, dt) in layer.cache_shapes(self.cfg, num_blocks, block_size,
                                                                       num_slots).items()})
        caches.append({"last_token": torch.zeros(PairHashEmbedding.get_state_shape(num_slots), dtype=torch.int64,
                                                 device=dev)})
        return caches

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, caches, batch: SequenceBatch,
                tap=None) -> torch.Tensor:
        """Returns the fp32 stream [T, width] after the last layer.  tap(layer, x) is called after
        every layer (tests, layer-by-layer comparison)."""
        x = self.embed(input_ids, caches[len(self.layers)]["last_token"], batch)
        pending = Pending()
        for i, layer in enumerate(self.layers):
            pending = layer(x, batch, caches[i], pending)
            if tap is not None:
                ops.branch_sum_norms(x, pending.terms, pending.experts)
                pending = Pending()
                tap(i, x)
        if pending.terms:
            ops.branch_sum_norms(x, pending.terms, pending.experts)
        return x

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """hidden: the rows of the stream whose logits are wanted -> fp32 [n, vocab]."""
        x = hidden.contiguous()
        h = torch.empty(x.shape, dtype=self.dtype, device=x.device)
        ops.branch_sum_norms(x, outs=[(h, self.final_norm.data)], eps=self.cfg.eps)
        return mm_f32(h, self.head.data)

    # ------------------------------------------------------------------ weights
    def _top_shapes(self) -> Dict[str, Tuple[int, ...]]:
        cfg = self.cfg
        return {"embed": (cfg.vocab, cfg.width), "bigram": (cfg.buckets + 1, cfg.width), "final.norm": (cfg.width, ),
                "head": (cfg.vocab, cfg.width)}

    def tensor_shapes(self) -> Dict[str, Tuple[int, ...]]:
        t = self._top_shapes()
        for i, layer in enumerate(self.layers):
            t.update({f"l{i}.{k}": v for k, v in layer.tensor_shapes(self.cfg).items()})
        return t

    def load_weights(self, tensors: Dict[str, torch.Tensor]) -> int:
        cfg, dev = self.cfg, self.head.device
        used = 0
        for i, layer in enumerate(self.layers):
            prefix = f"l{i}."
            layer.set_weights({k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}, cfg)
            used += len(layer.tensor_shapes(cfg))
        top = self._top_shapes()
        for name, shape in top.items():
            if name not in tensors:
                raise KeyError(f"tensor {name} is missing")
            if tuple(tensors[name].shape) != shape:
                raise ValueError(f"{name}: shape {tuple(tensors[name].shape)}, expected {shape}")
        self.embed.weight.data = tensors["embed"].to(self.dtype).to(dev).contiguous()
        self.embed.pair_weight.data = tensors["bigram"].to(self.dtype).to(dev).contiguous()
        self.final_norm.data = 1.0 + tensors["final.norm"].float().to(dev).contiguous()
        self.head.data = tensors["head"].to(self.dtype).to(dev).contiguous()
        return used + len(top)

    def random_weights(self, seed: int) -> Dict[str, torch.Tensor]:
        """Tensors of every checkpoint name: projections ~ N(0, 1 / fan_in), the stream's norm weights
        near 0 (they are stored around zero), the heads' near 1, small biases, decays between about a half
        and nearly one; the two-step projections of a channel_delta layer have its vdim as their rank."""
        g = torch.Generator().manual_seed(seed)
        out = {}
        for name, shape in self.tensor_shapes().items():
            last = name.rsplit(".", 1)[-1]
            if ANY in shape:
                rank = self.layers[int(name[1:name.index(".")])].spec.mixer.vdim
                shape = tuple(rank if n == ANY else n for n in shape)
            if name in ("embed", "bigram"):
                t = torch.randn(shape, generator=g)
            elif last in ("norm1", "norm2") or name == "final.norm":
                t = 0.1 * torch.randn(shape, generator=g)
            elif last == "norm":
                t = 1.0 + 0.1 * torch.randn(shape, generator=g)
            elif last == "dt_bias":
                t = -1.0 - 4.0 * torch.rand(shape, generator=g)
            elif name.endswith(".f.b"):
                t = 3.0 + torch.randn(shape, generator=g)
            elif len(shape) == 1:
                t = 0.1 * torch.randn(shape, generator=g)
            else:
                t = torch.randn(shape, generator=g) * shape[-1]**-0.5
            out[name] = t.to(torch.bfloat16)
        return out
