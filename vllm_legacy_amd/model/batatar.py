"""Batatar: a decoder-only pre-norm stack over an fp32 stream whose layers are linear attention with
constant decays, or a chunked softmax attention and a state-space recurrence side by side, each with a
mixture of experts whose router weights multiply the experts' inputs.

  x0 = x = embed[token]
  layer:  x <- x + m mixer(N(x) w1);   x <- x + m ff(N(x) w2)        (a layer may have no ff)
          N(u) = u / sqrt(mean(u^2) + eps), m = residual_mult
  mixer 'lightning':  q, k, v = silu of their projections; S_t = decay_h S_(t-1) + k_t v_t^T,
          o_t = S_t^T q_t; W_o (N(o, all heads together) w * sigmoid(W_g h))
  mixer 'parallel':   (N(left) w_left + N(right) w_right) / 2
    left:   q, k, v with biases (kv_heads key / value heads for heads query heads), no positions; every
            head of q and k divided by its root mean square; score = (q . k) scale, capped by
            softcap tanh(score / softcap); position i sees the keys j <= i of its own chunk of
            mask.size positions; weights exp(s_j) / (1 + sum exp(s)); head h's output times
            sigmoid(W_g h)_h; W_o
    right:  [z | x | B | C | dt] from one projection; x, B, C through a causal convolution with bias
            and silu; step = softplus(dt + dt_bias);
            S_t = exp(-exp(A_log) step) S_(t-1) + step B_t x_t^T, y_t = S_t^T C_t + D x_t per head;
            W_o (N(y silu(z), norm_groups parts) w)
  ff 'moe':  the `top` largest s = sigmoid(W_r h) choose; the sum of W_down (silu(W_gate u) * (W_up u))
          over the chosen experts with u = s h
  loop:   layers start .. stop - 1 run `times` times with the same weights and a cache / state of their
          own per pass; before a pass's first layer x <- W_in [x; x0] + step[pass]
  logits = head (N(x) w_final)

All sizes and per-model constants come from config.json; a layer entry carries its own mixer and
feed-forward sizes.  The projections that read h are one matrix product per mixer; matrix products
go to the vendor library, everything else runs on libvla_seq_gfx950.so.  The stream, norms, scores and
softmax weights, routers, recurrent states and everything that enters a recurrence beside projections
and the short convolution are fp32 whatever `dtype` is; `dtype` is the type of weights, projections,
caches and activations (bfloat16 to serve, float32 for an all-fp32 run).  A sublayer's result joins
the stream in the launch that norms the stream for the next one.
"""
import json
from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import torch
import torch.nn as nn

from vllm_legacy_amd import _seq_ops as ops
from vllm_legacy_amd.attention.backends.rotary_kv import RotaryKVAttention
from vllm_legacy_amd.attention.batch import SequenceBatch
from vllm_legacy_amd.attention.recurrent import ConstantDecayRecurrence, StateSpaceRecurrence
from vllm_legacy_amd.routed_experts import RoutedExperts, mm_f32

SINK_SCORE = 0.0            # the softmax's extra term: a key with this score and no value
BRANCH_WEIGHT = 0.5         # of each of a parallel mixer's two branches


@dataclass
class LightningSpec:
    heads: int
    dim: int
    vdim: int
    decay: List[float]


@dataclass
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float              # 0: none
    chunk: int                  # 0: none


@dataclass
class StateSpaceSpec:
    heads: int
    vdim: int
    state: int
    groups: int
    norm_groups: int
    taps: int


@dataclass
class ParallelSpec:
    left: AttentionSpec
    right: StateSpaceSpec


@dataclass
class MlpSpec:
    ff: int
    experts: int
    top: int


@dataclass
class LayerSpec:
    type: str                   # lightning | parallel
    mixer: object
    mlp: Optional[MlpSpec]


@dataclass
class BatatarConfig:
    vocab: int
    width: int
    eps: float
    residual_mult: float
    layers: List[LayerSpec]
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 0
    architecture: str = "Batatar"
    raw: Dict = field(default_factory=dict, repr=False)

    @property
    def loops(self) -> bool:
        return self.loop_times > 0 and self.loop_stop > self.loop_start

    @staticmethod
    def from_dict(d: Dict) -> "BatatarConfig":
        layers = []
        for i, entry in enumerate(d["layers"]):
            kind, m = entry.get("type"), entry.get("mixer") or {}
            if kind == "lightning":
                heads, dim = int(m["heads"]), int(m["dim"])
                decay = m["decay"]
                decay = [float(x) for x in decay] if isinstance(decay, (list, tuple)) else [float(decay)] * heads
                mixer = LightningSpec(heads, dim, int(m.get("vdim", dim)), decay)
                if len(decay) != heads:
                    raise ValueError(f"layer {i}: one decay per head is needed")
            elif kind == "parallel":
                le, ri = m["left"], m["right"]
                dim = int(le["dim"])
                left = AttentionSpec(int(le["heads"]), int(le.get("kv_heads", le["heads"])), dim, int(le.get("vdim", dim)),
                                     float(le.get("scale", dim**-0.5)), float(le.get("softcap") or 0.0),
                                     int((le.get("mask") or {}).get("size") or 0))
                right = StateSpaceSpec(int(ri["heads"]), int(ri["vdim"]), int(ri["state"]), int(ri.get("groups", 1)),
                                       int(ri.get("norm_groups", 1)), int(ri["conv"]))
                if left.heads % left.kv_heads:
                    raise ValueError(f"layer {i}: heads is not a multiple of kv_heads")
                if left.softcap < 0 or left.chunk < 0:
                    raise ValueError(f"layer {i}: softcap / mask.size out of range")
                if right.heads % right.groups or (right.heads * right.vdim) % right.norm_groups or right.taps < 1:
                    raise ValueError(f"layer {i}: groups / norm_groups / conv do not fit")
                mixer = ParallelSpec(left, right)
            else:
                raise ValueError(f"layer {i}: unknown layer type {kind!r}")
            mlp = entry.get("mlp")
            if mlp is None:
                spec = None
            elif mlp.get("kind") == "moe":
                spec = MlpSpec(int(mlp["expert"]["ff"]), int(mlp["router"]["experts"]), int(mlp["router"]["top"]))
                if spec.top < 1 or spec.top > spec.experts:
                    raise ValueError(f"layer {i}: router.top does not fit the number of experts")
            else:
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
            layers.append(LayerSpec(kind, mixer, spec))
        loop = d.get("loop") or {}
        start, stop, times = (int(loop.get(k, 0)) for k in ("start", "stop", "times"))
        if not 0 <= start <= stop <= len(layers) or times < 0 or (stop > start and times < 1):
            raise ValueError("loop range out of bounds")
        return BatatarConfig(int(d["vocab"]), int(d["width"]), float(d["norm"]["eps"]), float(d.get("residual_mult", 1.0)),
                             layers, start, stop, times, d.get("architecture", "Batatar"), d)

    @staticmethod
    def from_json(path: str) -> "BatatarConfig":
        with open(path) as f:
            return BatatarConfig.from_dict(json.load(f))

    def layer_runs(self) -> List[Tuple[int, Optional[int]]]:
        """(layer, pass) in execution order; pass is the number of the pass this run opens, None for a
        run that opens none."""
        n = len(self.layers)
        if not self.loops:
            return [(i, None) for i in range(n)]
        body = range(self.loop_start, self.loop_stop)
        return [(i, None) for i in range(self.loop_start)] + \
            [(i, t if i == self.loop_start else None) for t in range(self.loop_times) for i in body] + \
            [(i, None) for i in range(self.loop_stop, n)]


@dataclass
class Pending:
    """A sublayer's result that is not in the stream yet: x += scale * y, or x += scale * (N(y) w +
    N(y2) w2) of a mixer with two branches."""
    y: torch.Tensor
    scale: float
    norm: Optional[torch.Tensor] = None
    y2: Optional[torch.Tensor] = None
    norm2: Optional[torch.Tensor] = None


def _apply(x: torch.Tensor, pending: Optional[Pending], add_row: Optional[torch.Tensor] = None,
           out: Optional[torch.Tensor] = None, pre_weight: Optional[torch.Tensor] = None, eps: float = 0.0) -> None:
    """One launch: the pending result into the stream, a row added, the next norm."""
    if pending is None:
        if add_row is not None or out is not None:
            ops.residual_norms(x, add_row=add_row, out=out, pre_weight=pre_weight, eps=eps)
    else:
        ops.residual_norms(x, pending.y, None, pending.norm, None, add_row, out, pre_weight, eps, pending.scale,
                           pending.y2, pending.norm2)


def _pad8(n: int) -> int:
    return (n + 7) // 8 * 8


class BatatarLayer(nn.Module):

    def __init__(self, cfg: BatatarConfig, spec: LayerSpec, dtype, device):
        super().__init__()
        self.spec, self.dtype, self.eps, self.residual_mult, W = spec, dtype, cfg.eps, cfg.residual_mult, cfg.width

        def vec(n=W):
            return nn.Parameter(torch.ones(n, dtype=torch.float32, device=device), requires_grad=False)

        def mat(rows, cols):
            return nn.Parameter(torch.zeros((rows, cols), dtype=dtype, device=device), requires_grad=False)

        self.norm1 = vec()
        m = spec.mixer
        # the merged input projection: (checkpoint name, first row in that tensor, rows, has a bias)
        if spec.type == "lightning":
            self.recur = ConstantDecayRecurrence(m.heads, m.dim, m.vdim, m.decay, cfg.eps, "silu", device)
            qk, vg = m.heads * m.dim, m.heads * m.vdim
            self.in_parts = [("mix.q", 0, qk, False), ("mix.k", 0, qk, False), ("mix.v", 0, vg, False),
                             ("mix.g", 0, vg, False)]
            self.mixed = vg
            self.w_out = mat(W, vg)
        else:
            le, ri = m.left, m.right
            self.attn = RotaryKVAttention(le.heads, le.kv_heads, le.dim, le.vdim, le.scale, 0, 1.0, device=device,
                                          softcap=le.softcap, norm_eps=cfg.eps, norm_heads=True, chunk=le.chunk or None,
                                          sink_score=SINK_SCORE)
            self.recur = StateSpaceRecurrence(ri.heads, ri.vdim, ri.state, ri.groups, ri.norm_groups, ri.taps, cfg.eps,
                                              device)
            inner, chan = self.recur.inner, self.recur.channels
            self.in_parts = [("mix.left.q", 0, le.heads * le.dim, True), ("mix.left.k", 0, le.kv_heads * le.dim, True),
                             ("mix.left.v", 0, le.kv_heads * le.vdim, True), ("mix.left.g", 0, le.heads, False),
                             ("mix.right.in", 0, inner, False), ("mix.right.in", inner, chan, False),
                             ("mix.right.in", inner + chan, ri.heads, False)]
            self.w_out, self.w_out2 = mat(W, le.heads * le.vdim), mat(W, inner)
            self.left_out, self.right_out = vec(), vec()
        # every part starts on a multiple of eight rows, so that each part of a result row starts
        # 16-byte aligned
        self.in_starts, rows = [], 0
        for _, _, n, _ in self.in_parts:
            self.in_starts.append(rows)
            rows += _pad8(n)
        self.w_in = mat(rows, W)
        self.b_in = nn.Parameter(torch.zeros(rows, dtype=dtype, device=device), requires_grad=False) \
            if any(b for _, _, _, b in self.in_parts) else None
        mlp = spec.mlp
        if mlp is not None:
            self.norm2 = vec()
            self.experts = RoutedExperts(W, mlp.experts, 0, mlp.top, mlp.ff, act="silu", dtype=dtype, device=device,
                                         gated=True, score="sigmoid", renormalize=False, weight_input=True)

    # ------------------------------------------------------------------ weights
    def tensor_shapes(self, cfg: BatatarConfig) -> Dict[str, Tuple[int, ...]]:
        """Checkpoint names (without the layer prefix) and shapes of this layer's tensors."""
        W, mlp = cfg.width, self.spec.mlp
        t: Dict[str, Tuple[int, ...]] = {"norm1": (W, )}
        for name, first, n, bias in self.in_parts:
            t[name] = (first + n, W)                    # a tensor in several parts: the last part ends it
            if bias:
                t[name + ".b"] = (n, )
        if self.spec.type == "lightning":
            t.update({"mix.o": (W, self.mixed), "mix.norm": (self.mixed, )})
        else:
            le, r = self.spec.mixer.left, self.recur
            t.update({"mix.left.o": (W, le.heads * le.vdim), "mix.right.conv": (r.channels, r.conv.taps),
                      "mix.right.conv.b": (r.channels, ), "mix.right.dt_bias": (r.heads, ), "mix.right.A_log": (r.heads, ),
                      "mix.right.D": (r.heads, ), "mix.right.norm": (r.inner, ), "mix.right.o": (W, r.inner),
                      "mix.left.out": (W, ), "mix.right.out": (W, )})
        if mlp is not None:
            t["norm2"] = (W, )
            for e in range(mlp.experts):
                t.update({f"mlp.e{e}.gate": (mlp.ff, W), f"mlp.e{e}.up": (mlp.ff, W), f"mlp.e{e}.down": (W, mlp.ff)})
            t["mlp.router"] = (mlp.experts, W)
        return t

    def set_weights(self, t: Dict[str, torch.Tensor], cfg: BatatarConfig) -> None:
        """t: this layer's tensors by their names without the layer prefix."""
        dev, dt = self.w_in.device, self.dtype
        for name, shape in self.tensor_shapes(cfg).items():
            if name not in t:
                raise KeyError(f"tensor {name} is missing")
            if tuple(t[name].shape) != shape:
                raise ValueError(f"{name}: shape {tuple(t[name].shape)}, expected {shape}")

        def f32(name):
            return t[name].float().to(dev).contiguous()

        def put(param, value):
            param.data = value.to(param.dtype).to(dev).contiguous()

        self.norm1.data = f32("norm1")
        merged = torch.zeros(tuple(self.w_in.shape), dtype=dt)
        bias = torch.zeros(self.w_in.shape[0], dtype=dt)
        for (name, first, n, has_bias), start in zip(self.in_parts, self.in_starts):
            merged[start:start + n] = t[name][first:first + n].to(dt)
            if has_bias:
                bias[start:start + n] = t[name + ".b"].to(dt)
        put(self.w_in, merged)
        if self.b_in is not None:
            put(self.b_in, bias)
        r = self.recur
        if self.spec.type == "lightning":
            put(self.w_out, t["mix.o"])
            r.norm_weight.data = f32("mix.norm")
        else:
            put(self.w_out, t["mix.left.o"])
            put(self.w_out2, t["mix.right.o"])
            self.left_out.data, self.right_out.data = f32("mix.left.out"), f32("mix.right.out")
            r.conv.weight.data, r.conv.bias.data = f32("mix.right.conv"), f32("mix.right.conv.b")
            r.dt_bias.data, r.a_log.data, r.skip.data = f32("mix.right.dt_bias"), f32("mix.right.A_log"), f32("mix.right.D")
            r.norm_weight.data = f32("mix.right.norm")
        if self.spec.mlp is not None:
            self.norm2.data = f32("norm2")
            self.experts.set_weights({k[4:]: v for k, v in t.items() if k.startswith("mlp.")})

    # ------------------------------------------------------------------ caches
    def cache_shapes(self, cfg: BatatarConfig, num_blocks: int, block_size: int, num_slots: int):
        """name -> (shape, dtype) of what one run of this layer keeps between steps."""
        m = self.spec.mixer
        if self.spec.type == "lightning":
            return {"state": (ConstantDecayRecurrence.get_state_shape(num_slots, m.heads, m.dim, m.vdim), torch.float32)}
        le, ri = m.left, m.right
        ks, vs = RotaryKVAttention.get_cache_shapes(num_blocks, block_size, le.kv_heads, le.dim, le.vdim)
        state, conv = StateSpaceRecurrence.get_state_shapes(num_slots, ri.heads, ri.vdim, ri.state, ri.groups, ri.taps)
        out = {"keys": (ks, self.dtype), "values": (vs, self.dtype), "state": (state, torch.float32)}
        if ri.taps > 1:
            out["conv"] = (conv, torch.float32)
        return out

    # ------------------------------------------------------------------ forward
    def _mix(self, h: torch.Tensor, batch: SequenceBatch, cache: Dict[str, torch.Tensor]) -> Pending:
        T, dev = h.shape[0], h.device
        proj = torch.mm(h, self.w_in.data.t()) if self.b_in is None else torch.addmm(self.b_in.data, h, self.w_in.data.t())
        parts = [proj[:, s:s + p[2]] for s, p in zip(self.in_starts, self.in_parts)]
        if self.spec.type == "lightning":
            q, k, v, gate = parts
            mixed = torch.empty((T, self.mixed), dtype=self.dtype, device=dev)
            self.recur(mixed, q, k, v, gate, cache["state"], batch)
            return Pending(mm_f32(mixed, self.w_out.data), self.residual_mult)
        q, k, v, gate, z, xbc, dt = parts
        left = torch.empty((T, self.w_out.shape[1]), dtype=self.dtype, device=dev)
        self.attn(left, q, k, v, gate, cache["keys"], cache["values"], batch)
        right = torch.empty((T, self.w_out2.shape[1]), dtype=self.dtype, device=dev)
        self.recur(right, z, xbc, dt, cache["state"], cache.get("conv"), batch)
        return Pending(mm_f32(left, self.w_out.data), self.residual_mult * BRANCH_WEIGHT, self.left_out.data,
                       mm_f32(right, self.w_out2.data), self.right_out.data)

    def forward(self, x: torch.Tensor, batch: SequenceBatch, cache: Dict[str, torch.Tensor], pending: Optional[Pending],
                add_row: Optional[torch.Tensor] = None) -> Pending:
        """x: fp32 [T, width], updated in place except for the last sublayer's result, which comes back
        as Pending (the next norm's launch adds it)."""
        h = torch.empty(x.shape, dtype=self.dtype, device=x.device)
        _apply(x, pending, add_row, h, self.norm1.data, self.eps)
        pending = self._mix(h, batch, cache)
        if self.spec.mlp is None:
            return pending
        _apply(x, pending, None, h, self.norm2.data, self.eps)
        return Pending(self.experts(h), self.residual_mult)


class BatatarForCausalLM(nn.Module):
    """The stack and its per-run caches.  `seed` fills random weights (benchmarks); load_weights
    installs a checkpoint's."""

    architecture = "Batatar"

    def __init__(self, cfg: BatatarConfig, dtype=torch.bfloat16, device="cuda", seed: Optional[int] = None):
        super().__init__()
        self.cfg, self.dtype = cfg, dtype
        W = cfg.width

        def par(shape, dt):
            return nn.Parameter(torch.zeros(shape, dtype=dt, device=device), requires_grad=False)

        self.embed, self.head = par((cfg.vocab, W), dtype), par((cfg.vocab, W), dtype)
        self.layers = nn.ModuleList([BatatarLayer(cfg, s, dtype, device) for s in cfg.layers])
        if cfg.loops:
            self.loop_in, self.loop_step = par((W, 2 * W), dtype), par((cfg.loop_times, W), torch.float32)
        self.final_norm = nn.Parameter(torch.ones(W, dtype=torch.float32, device=device), requires_grad=False)
        self.runs = cfg.layer_runs()
        if seed is not None:
            self.load_weights(self.random_weights(seed))

    # ------------------------------------------------------------------ caches
    def cache_spec(self) -> List[Dict[str, Tuple[int, ...]]]:
        """Per layer run: the shapes of its caches for one block of one token and one slot."""
        return [{k: v[0] for k, v in self.layers[i].cache_shapes(self.cfg, 1, 1, 1).items()} for i, _ in self.runs]

    def allocate_caches(self, num_blocks: int, block_size: int, num_slots: int):
        dev = self.head.device
        return [{name: torch.zeros(shape, dtype=dt, device=dev)
                 for name, (shape, dt) in self.layers[i].cache_shapes(self.cfg, num_blocks, block_size,
                                                                      num_slots).items()}
                for i, _ in self.runs]

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, caches, batch: SequenceBatch,
                tap=None) -> torch.Tensor:
        """Returns the fp32 stream [T, width] after the last layer.  tap(run, x) is called after every
        layer run (tests, layer-by-layer comparison)."""
        cfg = self.cfg
        x = torch.empty((input_ids.numel(), cfg.width), dtype=torch.float32, device=self.head.device)
        ops.embed_scaled(x, self.embed.data, input_ids, 1.0)
        x0 = x.clone() if cfg.loops else None
        pending: Optional[Pending] = None
        for run, (i, opens) in enumerate(self.runs):
            add_row = None
            if opens is not None:
                _apply(x, pending)
                pending = None
                both = torch.empty((x.shape[0], 2 * cfg.width), dtype=self.dtype, device=x.device)
                ops.concat_cast(both, x, x0)
                x = mm_f32(both, self.loop_in.data)
                add_row = self.loop_step.data[opens]
            pending = self.layers[i](x, batch, caches[run], pending, add_row)
            if tap is not None:
                _apply(x, pending)
                pending = None
                tap(run, x)
        _apply(x, pending)
        return x

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """hidden: the rows of the stream whose logits are wanted -> fp32 [n, vocab]."""
        x = hidden.contiguous()
        h = torch.empty(x.shape, dtype=self.dtype, device=x.device)
        ops.residual_norms(x, out=h, pre_weight=self.final_norm.data, eps=self.cfg.eps)
        return mm_f32(h, self.head.data)

    # ------------------------------------------------------------------ weights
    def _top_shapes(self) -> Dict[str, Tuple[int, ...]]:
        cfg = self.cfg
        t = {"embed": (cfg.vocab, cfg.width), "head": (cfg.vocab, cfg.width), "final.norm": (cfg.width, )}
        if cfg.loops:
            t["loop.in"], t["loop.step"] = (cfg.width, 2 * cfg.width), (cfg.loop_times, cfg.width)
        return t

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
        self.embed.data = tensors["embed"].to(self.dtype).to(dev).contiguous()
        self.head.data = tensors["head"].to(self.dtype).to(dev).contiguous()
        self.final_norm.data = tensors["final.norm"].float().to(dev).contiguous()
        if cfg.loops:
            self.loop_in.data = tensors["loop.in"].to(self.dtype).to(dev).contiguous()
            self.loop_step.data = tensors["loop.step"].float().to(dev).contiguous()
        return used + len(top)

    def random_weights(self, seed: int) -> Dict[str, torch.Tensor]:
        """Tensors of every checkpoint name: projections ~ N(0, 1 / fan_in), norm weights near 1, small
        biases, decays of the state-space layers between about a half and nearly one."""
        g = torch.Generator().manual_seed(seed)
        out = {}
        for name, shape in self.tensor_shapes().items():
            last = name.rsplit(".", 1)[-1]
            if last in ("norm", "norm1", "norm2", "out"):
                t = 1.0 + 0.1 * torch.randn(shape, generator=g)
            elif last == "dt_bias":
                t = -1.0 - 4.0 * torch.rand(shape, generator=g)
            elif last == "D":
                t = 1.0 + 0.1 * torch.randn(shape, generator=g)
            elif len(shape) == 1 or last == "step":
                t = 0.1 * torch.randn(shape, generator=g)
            elif name == "embed":
                t = torch.randn(shape, generator=g)
            else:
                t = torch.randn(shape, generator=g) * shape[-1]**-0.5
            out[name] = t.to(torch.bfloat16)
        return out
