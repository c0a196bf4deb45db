"""
Rerozen: a decoder-only LM whose layers are listed in ``config.json``. Every sublayer is pre-normed and reads its normed
input plus a short causal convolution of it; every mixer is two mixers side by side on that input, summed with constant
scales. Two layer types:

* ``parallel`` — grouped-query attention within fixed chunks (biased projections, per-head q / k norm, rotary positions,
  a sigmoid gate per head) beside gated linear attention with a decay per key channel (:class:`GatedLinearMixer`);
* ``parallel_2`` — chunked attention with convolved projections, YaRN rotary positions, values turned by their position
  and the output turned back, one added to the softmax denominator, a gate per head — beside a gated delta rule with a
  decay per key channel (:class:`ChannelDeltaMixer`).

Both attentions are :class:`src.models.fekolorn.SinkAttentionMixer` under different switches. Feed-forward:
W_down gelu(W_up h), exact GELU.

Per layer (T tokens, residual x fp32):

    x += y;  h = n + conv(n), n = rms(x) * norm1           conv_norm   HIP, one launch (y: the previous sublayer's output)
    p = W_in h                                             one GEMM for both mixers' projections
    u = [ left gate . left scale | right gate . right scale ]   qkv_prep, sink_attn, rot_head_gate and gated_linear_attn,
                                                           head_norm_gate or delta_prep, gated_delta   HIP
    y = W_o u                                              one GEMM for both output projections
    x += y;  h = n + conv(n), n = rms(x) * norm2           conv_norm   HIP
    y = W_down gelu(W_up h)                                GEMM + gelu_act HIP + GEMM

The model plugs into :class:`src.engine.llm_engine.LLMEngine` like the other families: paged cache rows per layer from
:class:`src.models.datatar.LayerRowPool`, state slots (recurrent states, convolution tails) from
:class:`src.models.fekolorn.SeqStatePool`.
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass, replace
from typing import Any, Dict, List, Optional, Tuple

import torch

from src.models.datatar import MIXERS, LayerRowPool
from src.models.fekolorn import GatedDeltaSpec, SeqStatePool, SinkAttentionMixer, SinkAttnSpec
from src.ops import conv, mix, rec, seq
from src.parallel.tp import TPContext


# ------------------------------------------------------------------------------------------ configuration
@dataclass(frozen=True)
class GatedLinearSpec:
    heads: int
    dim: int
    vdim: int
    tau: float
    rank: int = 16             # of the decay's low-rank projection, for random weights; a checkpoint's tensors decide

    def state_shapes(self) -> Dict[str, Tuple[tuple, torch.dtype]]:
        return {"linear": ((self.heads, self.dim, self.vdim), torch.float32)}

    def to_config(self) -> Dict[str, Any]:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "tau": self.tau}


@dataclass(frozen=True)
class ChannelDeltaSpec(GatedDeltaSpec):
    rank: int = 64             # of the decay's and the gate's low-rank projections, as above


@dataclass(frozen=True)
class ScaledPairSpec:
    left: SinkAttnSpec
    right: Any
    left_scale: float
    right_scale: float

    @property
    def heads(self) -> int:
        return self.left.heads

    @property
    def cache_width(self) -> int:
        return self.left.cache_width

    def state_shapes(self) -> Dict[str, Tuple[tuple, torch.dtype]]:
        return {**self.left.state_shapes(), **self.right.state_shapes()}

    def to_config(self) -> Dict[str, Any]:
        return {"left": self.left.to_config(), "right": self.right.to_config(), "left_scale": self.left_scale,
                "right_scale": self.right_scale}


def _attn_common(m: Dict[str, Any]) -> Dict[str, Any]:
    rot, mask = m.get("rot") or {}, m.get("mask") or {}
    sc = rot.get("scaling")
    return dict(heads=int(m["heads"]), kv_heads=int(m.get("kv_heads") or m["heads"]), dim=int(m["dim"]),
                vdim=int(m.get("vdim") or m["dim"]), scale=float(m["scale"]), seg=int(mask.get("size") or 0),
                rot_dims=int(rot.get("dims") or 0), rot_base=float(rot.get("base", 10000.0)),
                rot_yarn=None if not sc else (float(sc["factor"]), float(sc["original"]), float(sc["fast"]),
                                              float(sc["slow"])),
                has_sink=False, head_gate=True)


def _scales(m: Dict[str, Any]) -> Dict[str, float]:
    return dict(left_scale=float(m.get("left_scale", 1.0)), right_scale=float(m.get("right_scale", 1.0)))


def _linear_pair_spec(m: Dict[str, Any]) -> ScaledPairSpec:
    r = m["right"]
    return ScaledPairSpec(left=SinkAttnSpec(**_attn_common(m["left"]), qkv_bias=True, qk_norm=True, head_norm=True),
                          right=GatedLinearSpec(heads=int(r["heads"]), dim=int(r["dim"]), vdim=int(r.get("vdim") or r["dim"]),
                                                tau=float(r["tau"])), **_scales(m))


def _delta_pair_spec(m: Dict[str, Any]) -> ScaledPairSpec:
    l, r = m["left"], m["right"]
    return ScaledPairSpec(left=SinkAttnSpec(**_attn_common(l), conv=int(l.get("conv") or 1), rot_values=True, unit_sink=True),
                          right=ChannelDeltaSpec(heads=int(r["heads"]), kv_heads=int(r.get("kv_heads") or r["heads"]),
                                                 dim=int(r["dim"]), vdim=int(r.get("vdim") or r["dim"]),
                                                 conv=int(r.get("conv") or 1)), **_scales(m))


@dataclass(frozen=True)
class RerLayerSpec:
    type: str
    mixer: ScaledPairSpec
    ff: int                    # 0: no feed-forward


@dataclass(frozen=True)
class RerozenArch:
    name: str
    vocab_size: int
    hidden_size: int
    layers: tuple
    taps: int = 1              # of the input convolutions
    rms_eps: float = 1e-5
    embed_scale: float = 1.0
    logit_scale: float = 1.0
    max_position: int = 1 << 20   # positions are rotated from inverse-frequency tables: no position table

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def is_moe(self) -> bool:
        return False

    @property
    def num_heads(self) -> int:
        return max(l.mixer.heads for l in self.layers)

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return sum(l.mixer.cache_width for l in self.layers) * dtype_bytes

    def state_shapes(self, i: int) -> Dict[str, Tuple[tuple, torch.dtype]]:
        """Per-sequence state of layer i: its mixer's and the tails of its sublayers' input convolutions."""
        l, tail = self.layers[i], ((self.taps - 1, self.hidden_size), torch.float32)
        out = {**l.mixer.state_shapes(), "canon1": tail}
        if l.ff:
            out["canon2"] = tail
        return out

    @staticmethod
    def from_config(c: Dict[str, Any], name: str = "rerozen") -> "RerozenArch":
        layers = []
        for i, lc in enumerate(c["layers"]):
            t, f = lc["type"], lc.get("mlp")
            if t not in REROZEN_MIXERS:
                raise ValueError(f"layer {i}: unknown mixer type {t!r} (known: {sorted(REROZEN_MIXERS)})")
            if f is not None and f.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {f.get('kind')!r}")
            layers.append(RerLayerSpec(t, REROZEN_MIXERS[t][0](lc["mixer"]), int(f["ff"]) if f is not None else 0))
        return RerozenArch(name=name, vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=tuple(layers),
                           taps=int((c.get("canon") or {}).get("taps", 1)),
                           rms_eps=float((c.get("norm") or {}).get("eps", 1e-5)),
                           embed_scale=float((c.get("embedding") or {}).get("scale", 1.0)),
                           logit_scale=float(c.get("logit_scale", 1.0)))

    def to_config(self) -> Dict[str, Any]:
        return {"architecture": "Rerozen", "canon": {"taps": self.taps}, "embedding": {"scale": self.embed_scale},
                "layers": [{"type": l.type, "mixer": l.mixer.to_config(),
                            "mlp": {"kind": "dense", "ff": l.ff} if l.ff else None} for l in self.layers],
                "logit_scale": self.logit_scale, "norm": {"eps": self.rms_eps}, "vocab": self.vocab_size,
                "width": self.hidden_size}


def rerozen_arch_from_dir(path: str, **overrides) -> RerozenArch:
    with open(os.path.join(path, "config.json")) as f:
        c = json.load(f)
    arch = RerozenArch.from_config(c, name=os.path.basename(os.path.normpath(path)))
    return replace(arch, **overrides) if overrides else arch


# -------------------------------------------------------------------------------------------------- mixers
def _put(dst: torch.Tensor, src: torch.Tensor) -> bool:
    dst.copy_(src.to(dst.device, dst.dtype).reshape(dst.shape))
    return True


class _LowRankBase:
    """What the two recurrent mixers share: named input projections (``parts``, rows of the layer's fused input
    projection) and second-stage matrices (``second``) of low-rank projections, whose rank the checkpoint's tensor
    shapes decide."""

    def __init__(self, hidden: int, device, dtype, gen: Optional[torch.Generator], std: float):
        self.hidden, self.device, self.dtype, self._gen, self._std = hidden, torch.device(device), dtype, gen, std
        self.parts: Dict[str, torch.Tensor] = {}
        self.second: Dict[str, torch.Tensor] = {}

    def rnd(self, *shape, scale=None, dt=None, shift=0.0):
        t = torch.empty(*shape, dtype=dt or self.dtype, device=self.device)
        if self._gen is None:
            return t.zero_()
        t.normal_(0.0, self._std if scale is None else scale, generator=self._gen)
        return t.add_(shift) if shift else t

    def finalize(self) -> None:
        """Nothing is derived from the weights."""

    def _named(self) -> Dict[str, torch.Tensor]:
        """Checkpoint name -> tensor (or view) of fixed shape."""
        raise NotImplementedError

    def load(self, name: str, t: torch.Tensor) -> bool:
        for d in (self.parts, self.second):
            if name in d:
                if tuple(t.shape) != tuple(d[name].shape):   # another rank
                    if t.dim() != 2 or (d is self.parts and t.shape[1] != self.hidden) or \
                            (d is self.second and t.shape[0] != d[name].shape[0]):
                        raise ValueError(f"{name}: shape {tuple(t.shape)} does not fit {tuple(d[name].shape)}")
                    d[name] = torch.empty(t.shape, dtype=self.dtype, device=self.device)
                return _put(d[name], t)
        dst = self._named().get(name)
        return dst is not None and _put(dst, t)

    def state(self) -> Dict[str, torch.Tensor]:
        out = {k: v for k, v in self.parts.items() if k != "qkv"}
        out.update(self.second)
        out.update(self._named())
        return out

    def tensors(self) -> List[torch.Tensor]:
        return list(self.second.values()) + [t for k, t in self._named().items() if k not in ("q", "k", "v")]


class GatedLinearMixer(_LowRankBase):
    """Weights and recurrence of gated linear attention. Per head: S <- diag(a) S + k v^T, o = S^T q dim^-1/2 with
    a = sigmoid(W_a2 W_a1 h + bias)^(1 / tau) per key channel; every head's o RMS-normed with shared weights, times
    SiLU(W_g h). S is per-sequence state ("linear" [slots, H, dim, vdim])."""

    type_name = "gated_linear"

    def __init__(self, spec: GatedLinearSpec, hidden: int, device, dtype, gen: Optional[torch.Generator], std: float):
        super().__init__(hidden, device, dtype, gen, std)
        s = self.spec = spec
        f32 = torch.float32
        self.nqk, self.nv = s.heads * s.dim, s.heads * s.vdim
        self.parts = {"qkv": self.rnd(2 * self.nqk + self.nv, hidden), "g": self.rnd(self.nv, hidden),
                      "a1": self.rnd(s.rank, hidden)}
        self.second = {"a2": self.rnd(self.nqk, s.rank, scale=0.3)}
        self.a2_b = self.rnd(self.nqk, scale=1.0, dt=f32, shift=1.0)
        self.norm = self.rnd(s.vdim, scale=0.1, dt=f32, shift=1.0)
        self.o = self.rnd(hidden, self.nv)

    def _named(self) -> Dict[str, torch.Tensor]:
        w, n = self.parts["qkv"], self.nqk
        return {"q": w[:n], "k": w[n: 2 * n], "v": w[2 * n:], "a2.b": self.a2_b, "norm": self.norm, "o": self.o}

    def recur(self, p: torch.Tensor, at: Dict[str, int], low: torch.Tensor, eps: float, state: Dict[str, torch.Tensor],
              rag: seq.Ragged, mult: float, out: torch.Tensor) -> None:
        """p [T, *]: the fused projection, this mixer's columns at ``at``; low [T, >= H dim]: the low-rank projections'
        output. Writes mult * the gated read-out into ``out`` [T, H * vdim]."""
        s, x0 = self.spec, at["qkv"]
        o, _ = rec.gated_linear_attn(p, x0, x0 + self.nqk, x0 + 2 * self.nqk, None, state["linear"], None, s.heads,
                                     s.heads, s.dim, s.vdim, s.dim ** -0.5, rag, z=low[:, : self.nqk], z_bias=self.a2_b,
                                     tau=s.tau)
        rec.head_norm_gate(o, None, None, p[:, at["g"]: at["g"] + self.nv], self.norm, s.heads, s.vdim, eps,
                           gate_silu=True, mult=mult, out=out)


class ChannelDeltaMixer(_LowRankBase):
    """Weights and recurrence of the gated delta rule with a decay per key channel: q, k, v through a short causal
    convolution and SiLU, unit q (times dim^-1/2) and k, S <- diag(g) S, S <- S + k (beta (v - S^T k))^T, read-out S^T q;
    g = exp(-exp(A_log) softplus(W_a2 W_a1 h + dt_bias)). Every head's read-out RMS-normed with shared weights, times
    sigmoid(W_g2 W_g1 h). S and the convolution's tail are per-sequence state ("delta", "conv")."""

    type_name = "channel_delta"

    def __init__(self, spec: ChannelDeltaSpec, hidden: int, device, dtype, gen: Optional[torch.Generator], std: float):
        super().__init__(hidden, device, dtype, gen, std)
        s = self.spec = spec
        if s.heads % s.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        f32 = torch.float32
        C, H = s.channels, s.heads
        self.ng, self.nz, self.nv = s.kv_heads * s.dim, H * s.dim, H * s.vdim
        self.parts = {"qkv": self.rnd(C, hidden), "a1": self.rnd(s.rank, hidden), "g1": self.rnd(s.rank, hidden),
                      "b": self.rnd(H, hidden)}
        self.second = {"a2": self.rnd(self.nz, s.rank, scale=0.1), "g2": self.rnd(self.nv, s.rank, scale=0.1)}
        self.conv_w = self.rnd(C, s.conv, scale=0.5, dt=f32)
        self.conv_wt = None
        self.A_log = self.rnd(H, scale=0.5, dt=f32)
        self.dt_bias = self.rnd(self.nz, scale=0.7, dt=f32, shift=-2.5)
        self.norm = self.rnd(s.vdim, scale=0.1, dt=f32, shift=1.0)
        self.o = self.rnd(hidden, self.nv)
        self.finalize()

    def finalize(self) -> None:
        """Derived tensors, after the weights changed: the convolution weights tap-major for 16-byte loads."""
        self.conv_wt = self.conv_w.t().contiguous()

    def _named(self) -> Dict[str, torch.Tensor]:
        w, c, n = self.parts["qkv"], self.conv_w, self.ng
        out = {"A_log": self.A_log, "dt_bias": self.dt_bias, "norm": self.norm, "o": self.o}
        for k, (a, b) in {"q": (0, n), "k": (n, 2 * n), "v": (2 * n, w.shape[0])}.items():
            out[k], out[k + ".conv"] = w[a:b], c[a:b]
        return out

    def recur(self, p: torch.Tensor, at: Dict[str, int], low: torch.Tensor, eps: float, state: Dict[str, torch.Tensor],
              rag: seq.Ragged, mult: float, out: torch.Tensor) -> None:
        """As :meth:`GatedLinearMixer.recur`; low [T, H dim + H vdim]."""
        s = self.spec
        H, G = s.heads, s.kv_heads
        x, b = p[:, at["qkv"]: at["qkv"] + s.channels], p[:, at["b"]: at["b"] + H]
        qkv32, beta = seq.delta_prep(x, b, None, self.conv_w, state["conv"], None, None, H, G, s.dim, s.vdim, rag,
                                     conv_wt=self.conv_wt)
        seq.conv_state_update(state["conv"], x, H, G, s.dim, s.vdim, rag)
        seq.gated_delta(qkv32, beta, low[:, self.nz: self.nz + self.nv], self.norm, eps, state["delta"], H, G, s.dim,
                        s.vdim, rag, z=low[:, : self.nz], z_bias=self.dt_bias, A_log=self.A_log, gate_sigmoid=True,
                        mult=mult, out=out)


PART_ALIGN, ROW_ALIGN = 8, 32   # rows of a part of the fused projection, and of the whole, are padded to multiples


class ScaledPairMixer:
    """Chunked attention and a recurrence side by side on the same input, summed with two constants. Both mixers' input
    projections are one matrix (each part padded to 8 rows so that its columns of the product start 16-byte aligned),
    the second stages of the low-rank projections one block-diagonal matrix, both output projections one matrix over
    the concatenated gated outputs; the constants multiply the outputs in fp32 before they are stored."""

    type_name = "scaled_pair"
    right_cls: Any = None

    def __init__(self, spec: ScaledPairSpec, hidden: int, device, dtype, gen: Optional[torch.Generator], std: float):
        self.spec, self.hidden = spec, hidden
        self.left = SinkAttentionMixer(spec.left, hidden, device, dtype, gen, std)
        self.right = self.right_cls(spec.right, hidden, device, dtype, gen, std)
        self.w_in = self.w_low = self.w_o = None
        self.at: Dict[str, int] = {}
        self.finalize()

    def finalize(self) -> None:
        """The fused matrices, after the weights changed; the parts stay views of them, so loading writes in place."""
        self.left.finalize()
        self.right.finalize()
        l, r = self.left, self.right
        parts = [("left.qkv", l.qkv)] + [("right." + k, v) for k, v in r.parts.items() if k != "b"]
        parts += [("left.g", l.gate)] + [("right." + k, v) for k, v in r.parts.items() if k == "b"]
        off, total = {}, 0
        for k, t in parts:
            off[k] = total
            total += -(-t.shape[0] // PART_ALIGN) * PART_ALIGN
        w = torch.zeros(-(-total // ROW_ALIGN) * ROW_ALIGN, self.hidden, dtype=l.dtype, device=l.device)
        views = {}
        for k, t in parts:
            views[k] = w[off[k]: off[k] + t.shape[0]]
            views[k].copy_(t)
        self.w_in = w
        l.qkv, l.gate = views["left.qkv"], views["left.g"]
        r.parts = {k: views["right." + k] for k in r.parts}
        self.at = {k[6:]: v for k, v in off.items() if k.startswith("right.")}
        self.gate_at = off["left.g"]
        # low-rank second stages: block-diagonal over the adjacent first-stage columns
        firsts = [k for k in ("a1", "g1") if k in r.parts]
        a = self.at["a1"]
        self.low_cols = (a, self.at[firsts[-1]] + -(-r.parts[firsts[-1]].shape[0] // PART_ALIGN) * PART_ALIGN)
        seconds = [r.second[k[0] + "2"] for k in firsts]
        low = torch.zeros(sum(t.shape[0] for t in seconds), self.low_cols[1] - a, dtype=l.dtype, device=l.device)
        row = 0
        for k, t in zip(firsts, seconds):
            c = self.at[k] - a
            low[row: row + t.shape[0], c: c + t.shape[1]].copy_(t)
            row += t.shape[0]
        self.w_low = low
        nl = l.o.shape[1]
        self.w_o = torch.cat([l.o, r.o], 1)
        l.o, r.o = self.w_o[:, :nl], self.w_o[:, nl:]

    def tensors(self) -> List[torch.Tensor]:
        return [self.w_in, self.w_low, self.w_o]

    def load(self, name: str, t: torch.Tensor) -> bool:
        if name.startswith("left."):
            return self.left.load(name[5:], t)
        if name.startswith("right."):
            return self.right.load(name[6:], t)
        return False

    def state(self) -> Dict[str, torch.Tensor]:
        out = {"left." + k: v for k, v in self.left.state().items()}
        out.update({"right." + k: v for k, v in self.right.state().items()})
        return out

    def forward(self, h, positions, meta, cache, eps, state=None, rag=None, shared=None, **_):
        s, l = self.spec, self.left
        p = mix.linear(h, self.w_in)
        low = mix.linear(p[:, self.low_cols[0]: self.low_cols[1]], self.w_low)
        nl = s.left.heads * s.left.vdim
        u = torch.empty(h.shape[0], self.w_o.shape[1], dtype=h.dtype, device=h.device)
        l.heads_out(p, positions, meta, cache, eps, shared if shared is not None else {}, state, rag,
                    gate=p[:, self.gate_at: self.gate_at + s.left.heads], mult=s.left_scale, out=u[:, :nl])
        self.right.recur(p, self.at, low, eps, state, rag, s.right_scale, u[:, nl:])
        return mix.linear_partials(u, self.w_o)


class LinearPairMixer(ScaledPairMixer):
    type_name = "linear_pair"
    right_cls = GatedLinearMixer
    spec_from_config = staticmethod(_linear_pair_spec)


class DeltaPairMixer(ScaledPairMixer):
    type_name = "delta_pair"
    right_cls = ChannelDeltaMixer
    spec_from_config = staticmethod(_delta_pair_spec)


for _m in (LinearPairMixer, DeltaPairMixer):
    MIXERS[_m.type_name] = _m

# this family's reading of the layer types: (spec from the layer's "mixer" entry, mixer class)
REROZEN_MIXERS = {"parallel": (_linear_pair_spec, LinearPairMixer), "parallel_2": (_delta_pair_spec, DeltaPairMixer)}


class RerLayerWeights:
    __slots__ = ("norm1", "norm2", "canon1", "canon2", "mix", "up", "down")

    def __init__(self):
        for s in self.__slots__:
            setattr(self, s, None)


class RerozenLM:
    """The model behind :class:`src.engine.llm_engine.LLMEngine` for ``architecture: Rerozen`` checkpoints (same
    interface as the other families: forward / compute_logits / load_state_dict, plus ``make_seq_state``)."""

    needs_decode_partials = False
    graph_capturable = True
    needs_seq_state = True          # the engine gives every live sequence a state slot (AttnMetadata.state_slots)
    supports_prefix_cache = False   # a cached prefix holds keys and values but not the state after it

    def __init__(self, arch: RerozenArch, device, dtype=torch.bfloat16, tp: Optional[TPContext] = None, seed: int = 0,
                 init_std: float = 0.05, max_position: Optional[int] = None, random_init: bool = True, **_):
        if tp is not None and tp.enabled:
            raise ValueError("Rerozen runs on one GPU (no tensor-parallel layout is defined for its mixers)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Rerozen runs in bfloat16 or float32")
        self.arch, self.device, self.dtype = arch, torch.device(device), dtype
        self.tp = tp or TPContext()
        self.hq, self.hkv = arch.num_heads, 1
        self.max_position = max_position or arch.max_position
        gen = None
        if random_init:
            gen = torch.Generator(device=self.device)
            gen.manual_seed(seed)
        h, f32 = arch.hidden_size, torch.float32

        def rnd(*shape, scale=init_std, dt=dtype):
            t = torch.empty(*shape, dtype=dt, device=self.device)
            return t.normal_(0.0, scale, generator=gen) if gen is not None else t.zero_()

        self.embed = rnd(arch.vocab_size, h, scale=1.0)
        self.layers: List[RerLayerWeights] = []
        for spec in arch.layers:
            lw = RerLayerWeights()
            lw.norm1 = 1.0 + rnd(h, scale=0.1, dt=f32)
            lw.canon1 = rnd(arch.taps, h, scale=0.3, dt=f32)   # tap-major: the current row's weights last
            lw.mix = REROZEN_MIXERS[spec.type][1](spec.mixer, h, self.device, dtype, gen, init_std)
            if spec.ff:
                lw.norm2 = 1.0 + rnd(h, scale=0.1, dt=f32)
                lw.canon2 = rnd(arch.taps, h, scale=0.3, dt=f32)
                lw.up = rnd(spec.ff, h)
                lw.down = rnd(h, spec.ff)
            self.layers.append(lw)
        self.norm = 1.0 + rnd(h, scale=0.1, dt=f32)
        self.norm_out: Optional[torch.Tensor] = None
        self.lm_head = rnd(arch.vocab_size, h)
        self.seq_state: Optional[SeqStatePool] = None
        self._fold_logit_scale()

    # ------------------------------------------------------------------ weights
    def load_state_dict(self, tensors: Dict[str, torch.Tensor], fold: bool = True) -> int:
        """Tensors under the checkpoint's names: ``embed``, ``head``, ``final.norm`` and, for layer i,
        ``l<i>.norm1|norm2``, ``l<i>.canon1|canon2`` ([width, taps]), ``l<i>.mix.left|right.<name>`` (the mixer's own),
        ``l<i>.mlp.up|down``."""
        n = 0
        top = {"embed": self.embed, "head": self.lm_head, "final.norm": self.norm}
        for name, t in tensors.items():
            if name in top:
                n += _put(top[name], t)
                continue
            if not (name.startswith("l") and "." in name and name[1:name.index(".")].isdigit()):
                continue
            li, rest = int(name[1:name.index(".")]), name[name.index(".") + 1:]
            if li >= len(self.layers):
                continue
            lw = self.layers[li]
            if rest.startswith("mix."):
                n += bool(lw.mix.load(rest[4:], t))
                continue
            dst = {"norm1": lw.norm1, "norm2": lw.norm2, "canon1": lw.canon1, "canon2": lw.canon2, "mlp.up": lw.up,
                   "mlp.down": lw.down}.get(rest)
            if dst is not None:
                if rest.startswith("canon"):
                    t = t.t()
                    if t.shape != dst.shape:
                        raise ValueError(f"{name}: expected [width, taps] = {tuple(dst.t().shape)}")
                n += _put(dst, t)
        if fold:
            self.fold_norm_weights()
        return n

    def _fold_logit_scale(self) -> None:
        self.norm_out = self.norm * self.arch.logit_scale

    def fold_norm_weights(self, layers=None) -> None:
        """Called once the weights are in: the mixers' fused matrices, and the logit scale as part of the final norm's
        weight (the head is linear)."""
        for lw in self.layers:
            lw.mix.finalize()
        self._fold_logit_scale()

    def state_dict(self) -> Dict[str, torch.Tensor]:
        out = {"embed": self.embed, "head": self.lm_head, "final.norm": self.norm}
        for i, lw in enumerate(self.layers):
            p = f"l{i}."
            out[p + "norm1"], out[p + "canon1"] = lw.norm1, lw.canon1.t()
            for k, v in lw.mix.state().items():
                out[p + "mix." + k] = v
            if lw.up is not None:
                out[p + "norm2"], out[p + "canon2"] = lw.norm2, lw.canon2.t()
                out[p + "mlp.up"], out[p + "mlp.down"] = lw.up, lw.down
        return out

    def save(self, path: str) -> None:
        """``config.json`` + ``model.safetensors`` under the checkpoint names (tests, tooling)."""
        from safetensors.torch import save_file

        os.makedirs(path, exist_ok=True)
        with open(os.path.join(path, "config.json"), "w") as f:
            json.dump(self.arch.to_config(), f, indent=1)
        save_file({k: v.detach().to("cpu").contiguous() for k, v in self.state_dict().items()},
                  os.path.join(path, "model.safetensors"))

    def weight_bytes(self) -> int:
        tot = sum(t.numel() * t.element_size() for t in (self.embed, self.lm_head))
        for lw in self.layers:
            ts = lw.mix.tensors() + [t for t in (lw.up, lw.down, lw.canon1, lw.canon2) if t is not None]
            tot += sum(t.numel() * t.element_size() for t in ts)
        return tot

    # ------------------------------------------------------------ cache + state
    def kv_bytes_per_block(self, block_size: int) -> int:
        return max(1, self.arch.kv_bytes_per_token(self.embed.element_size())) * block_size

    def make_kv_pool(self, num_blocks: int, block_size: int) -> LayerRowPool:
        return LayerRowPool([l.mixer.cache_width for l in self.arch.layers], num_blocks, block_size, self.device,
                            self.dtype)

    def make_seq_state(self, num_slots: int) -> SeqStatePool:
        self.seq_state = SeqStatePool([self.arch.state_shapes(i) for i in range(self.arch.num_layers)], num_slots,
                                      self.device)
        return self.seq_state

    def activation_bytes(self, tokens: int) -> int:
        a = self.arch
        widest = 0
        for l, lw in zip(a.layers, self.layers):
            m = lw.mix
            widest = max(widest, 4 * (m.w_in.shape[0] + m.w_low.shape[0] + m.w_o.shape[1]), 3 * l.ff)
        return tokens * (14 * a.hidden_size + 4 * widest) + (1 << 30)

    # ----------------------------------------------------------------- forward
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, meta, kv_pool,
                layer_hook=None) -> torch.Tensor:
        """Final-norm hidden states [T, W] in the model dtype, times the logit scale. ``kv_pool``: one cache tensor per
        layer. ``meta.state_slots``: the state slot of every sequence of the step. ``layer_hook(i, residual)``: called
        with the fp32 residual after layer i."""
        if self.seq_state is None or getattr(meta, "state_slots", None) is None:
            raise RuntimeError("Rerozen needs per-sequence state slots (LLMEngine provides them)")
        a, st, eps, dt = self.arch, self.seq_state.layers, self.arch.rms_eps, self.dtype
        rag = seq.Ragged(positions, meta.cu_q if meta.is_prefill else None, meta.state_slots)
        max_q = meta.max_q_len if meta.is_prefill else 1
        x, _ = rec.embed_scaled(input_ids, self.embed, a.embed_scale, copy=False)
        y = spare = None
        shared: Dict[str, Any] = {}

        def boundary(norm, wt=None, state=None):
            """The residual takes the pending sublayer output; returns the next sublayer's input."""
            nonlocal x, spare
            new, h = conv.conv_norm(x, y, norm, eps, dt, wt, state, rag, max_q, spare)
            if new is not x:
                x, spare = new, x
            return h

        for li, lw in enumerate(self.layers):
            h = boundary(lw.norm1, lw.canon1, st[li]["canon1"])
            if layer_hook is not None and li > 0:
                layer_hook(li - 1, x)
            y = lw.mix.forward(h, positions, meta, kv_pool[li], eps, state=st[li], rag=rag, shared=shared)
            if meta.kv_hook is not None:
                meta.kv_hook(li)
            if lw.up is not None:
                h = boundary(lw.norm2, lw.canon2, st[li]["canon2"])
                y = mix.linear_partials(mix.gelu_act(mix.linear(h, lw.up)), lw.down)
        h = boundary(self.norm_out)
        if layer_hook is not None:
            layer_hook(len(self.layers) - 1, x)
        return h

    def compute_logits(self, hidden: torch.Tensor, argmax_parts=None) -> torch.Tensor:
        """Logits [rows, vocab] = head(hidden) in the model dtype (what the sampling kernel reads; the logit scale is
        already in ``hidden``)."""
        if argmax_parts is not None:
            raise ValueError("this head writes no per-tile argmax candidates")
        return mix.linear(hidden, self.lm_head)
