"""
Malapel: a decoder-only LM whose layers are listed in ``config.json``; a stretch of them may run several times in a row
with the same weights, every pass with its own cache, and every pass begins by mixing the residual with the embedding
output. Three mixers, all grouped-query attention with rotary positions
(:class:`src.models.fekolorn.SinkAttentionMixer` under different switches):

* ``attention`` — within fixed chunks of positions, q and k RMS-normed over the whole projection, one added to the softmax
  denominator;
* ``attention_2`` — causal, ordinary softmax;
* ``attention_3`` — a sliding window whose keys weigh sigmoid(score + a number per head) each, not normalised.

Feed-forward: dense clamped sigmoid-gated, or a mixture of squared-ReLU experts with softmax routing limited to the best
groups of experts.

Per layer run (T tokens, residual x fp32; norms with a gain of one plus the stored weight, folded once):

    x = rms(embed) * (1 + w)                         embed_norm                    HIP, one launch
    [x | x0] <- x + y                                conv_norm / combine_pre_norm  HIP (a pass of the loop begins)
    x = W_in [x; x0]                                 GEMM with fp32 results
    x += y;  h = rms(x) * (1 + norm1)                conv_norm / combine_pre_norm  HIP, one launch (y: the last output)
    y = W_o attn(W_qkv h)                            GEMM, qkv_prep, sink_attn     HIP, GEMM
    x += y;  h = rms(x) * (1 + norm2)                conv_norm                     HIP, one launch
    y = ff(h)                                        GEMM, gated_act HIP, GEMM; or route_grouped_topk, moe_output_weighted

The weighted sum of a mixture's experts, the residual update and the next norm (or the copy that the loop's projection
reads) are one launch. The model plugs into :class:`src.engine.llm_engine.LLMEngine` like the other families: paged cache
rows from :class:`src.models.datatar.LayerRowPool`, one plane per layer run; it keeps no other per-sequence state.
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass, replace
from typing import Any, Dict, List, NamedTuple, Optional, Tuple

import torch

from src.models.datatar import LayerRowPool
from src.models.fekolorn import SinkAttentionMixer, SinkAttnSpec
from src.ops import conv, mix
from src.parallel.tp import TPContext

# the dense feed-forward's gate is g * sigmoid(GATE_ALPHA * g)
GATE_ALPHA = 1.702


# ------------------------------------------------------------------------------------------ configuration
@dataclass(frozen=True)
class RoutedMlpSpec:
    kind: str                  # "dense" | "moe"
    ff: int                    # width (of one expert)
    limit: float = 0.0         # dense: clamp of gate (above) and up (both sides)
    experts: int = 0
    top: int = 0
    groups: int = 1
    keep: int = 1              # groups whose experts can be chosen
    scale: float = 1.0         # of the chosen experts' scores

    @staticmethod
    def from_config(m: Optional[Dict[str, Any]]) -> Optional["RoutedMlpSpec"]:
        if m is None:
            return None
        if m["kind"] == "dense":
            return RoutedMlpSpec("dense", ff=int(m["ff"]), limit=float(m["limit"]))
        if m["kind"] != "moe":
            raise ValueError(f"unknown feed-forward kind {m['kind']!r}")
        r = m["router"]
        g = r.get("groups") or {}
        count = int(g.get("count") or 1)
        f = RoutedMlpSpec("moe", ff=int(m["expert"]["ff"]), experts=int(r["experts"]), top=int(r["top"]), groups=count,
                          keep=int(g.get("keep") or count), scale=float(r.get("scale", 1.0)))
        if f.experts % count or not 1 <= f.keep <= count or not 1 <= f.top <= f.keep * (f.experts // count):
            raise ValueError("router: groups must divide the experts, and the kept groups hold at least `top` experts")
        return f

    def to_config(self) -> Dict[str, Any]:
        if self.kind == "dense":
            return {"kind": "dense", "ff": self.ff, "limit": self.limit}
        return {"kind": "moe", "expert": {"ff": self.ff},
                "router": {"experts": self.experts, "groups": {"count": self.groups, "keep": self.keep}, "scale": self.scale,
                           "top": self.top}}


def _attn_common(m: Dict[str, Any]) -> Dict[str, Any]:
    rot = m.get("rot") or {}
    return dict(heads=int(m["heads"]), kv_heads=int(m.get("kv_heads") or m["heads"]), dim=int(m["dim"]),
                vdim=int(m.get("vdim") or m["dim"]), scale=float(m["scale"]), rot_dims=int(rot.get("dims") or 0),
                rot_base=float(rot.get("base", 10000.0)), has_sink=False)


def _mask_size(m: Dict[str, Any]) -> int:
    return int((m.get("mask") or {}).get("size") or 0)


# this family's reading of the layer types: the attention's switches from the layer's "mixer" entry
MALAPEL_MIXERS = {
    "attention": lambda m: SinkAttnSpec(**_attn_common(m), seg=_mask_size(m), qk_norm=True, unit_sink=True),
    "attention_2": lambda m: SinkAttnSpec(**_attn_common(m)),
    "attention_3": lambda m: SinkAttnSpec(**_attn_common(m), window=_mask_size(m), sigmoid=True),
}


@dataclass(frozen=True)
class MalLayerSpec:
    type: str
    mixer: SinkAttnSpec
    mlp: Optional[RoutedMlpSpec]


class LayerRun(NamedTuple):
    layer: int
    enter: bool                # a pass of the loop begins right before this run


@dataclass(frozen=True)
class MalapelArch:
    name: str
    vocab_size: int
    hidden_size: int
    layers: tuple
    loop: Optional[Tuple[int, int, int]] = None   # (start, stop, times): layers start .. stop - 1 run `times` times in a row
    rms_eps: float = 1e-5
    max_position: int = 1 << 20   # positions are rotated from inverse-frequency tables: no position table

    def runs(self) -> List[LayerRun]:
        """The layers in the order in which they run; each run has its own plane of the cache."""
        n = len(self.layers)
        start, stop, times = self.loop or (n, n, 0)
        out = [LayerRun(i, False) for i in range(start)]
        for _ in range(times):
            out += [LayerRun(i, i == start) for i in range(start, stop)]
        return out + [LayerRun(i, False) for i in range(stop, n)]

    @property
    def num_layers(self) -> int:
        """Layer runs (planes of the cache), not layers with weights of their own."""
        return len(self.runs())

    @property
    def is_moe(self) -> bool:
        return any(l.mlp is not None and l.mlp.kind == "moe" for l in self.layers)

    @property
    def num_heads(self) -> int:
        return max(l.mixer.heads for l in self.layers)

    def cache_widths(self) -> List[int]:
        return [self.layers[r.layer].mixer.cache_width for r in self.runs()]

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return sum(self.cache_widths()) * dtype_bytes

    @staticmethod
    def from_config(c: Dict[str, Any], name: str = "malapel") -> "MalapelArch":
        layers = []
        for i, lc in enumerate(c["layers"]):
            t = lc["type"]
            if t not in MALAPEL_MIXERS:
                raise ValueError(f"layer {i}: unknown mixer type {t!r} (known: {sorted(MALAPEL_MIXERS)})")
            layers.append(MalLayerSpec(t, MALAPEL_MIXERS[t](lc["mixer"]), RoutedMlpSpec.from_config(lc.get("mlp"))))
        loop = c.get("loop")
        if loop:
            loop = (int(loop["start"]), int(loop["stop"]), int(loop["times"]))
            if not 0 <= loop[0] < loop[1] <= len(layers) or loop[2] < 1:
                raise ValueError("loop: 0 <= start < stop <= layers, times >= 1")
        return MalapelArch(name=name, vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=tuple(layers),
                           loop=loop or None, rms_eps=float((c.get("norm") or {}).get("eps", 1e-5)))

    def to_config(self) -> Dict[str, Any]:
        c: Dict[str, Any] = {"architecture": "Malapel",
                             "layers": [{"type": l.type, "mixer": l.mixer.to_config(),
                                         "mlp": None if l.mlp is None else l.mlp.to_config()} for l in self.layers],
                             "norm": {"eps": self.rms_eps}, "vocab": self.vocab_size, "width": self.hidden_size}
        if self.loop is not None:
            c["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        return c


def malapel_arch_from_dir(path: str, **overrides) -> MalapelArch:
    with open(os.path.join(path, "config.json")) as f:
        c = json.load(f)
    arch = MalapelArch.from_config(c, name=os.path.basename(os.path.normpath(path)))
    return replace(arch, **overrides) if overrides else arch


# ------------------------------------------------------------------------------------------------ weights
def _put(dst: torch.Tensor, src: torch.Tensor) -> bool:
    dst.copy_(src.to(dst.device, dst.dtype).reshape(dst.shape))
    return True


class MalLayerWeights:
    __slots__ = ("norm1", "norm2", "gain1", "gain2", "mix", "gate_up", "down", "router", "w1", "w2")

    def __init__(self):
        for s in self.__slots__:
            setattr(self, s, None)

    def tensors(self) -> List[torch.Tensor]:
        return [t for t in (self.gate_up, self.down, self.router, self.w1, self.w2) if t is not None]


class MalapelLM:
    """The model behind :class:`src.engine.llm_engine.LLMEngine` for ``architecture: Malapel`` checkpoints (same interface
    as the other families: forward / compute_logits / load_state_dict)."""

    needs_decode_partials = False   # the runner's split-KV scratch of the GQA decode kernel is not used
    graph_capturable = True

    def __init__(self, arch: MalapelArch, device, dtype=torch.bfloat16, tp: Optional[TPContext] = None, seed: int = 0,
                 init_std: float = 0.05, max_position: Optional[int] = None, random_init: bool = True, **_):
        if tp is not None and tp.enabled:
            raise ValueError("Malapel runs on one GPU (no tensor-parallel layout is defined for its mixers)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Malapel runs in bfloat16 or float32")
        self.arch, self.device, self.dtype = arch, torch.device(device), dtype
        self.tp = tp or TPContext()
        self.hq, self.hkv = arch.num_heads, 1
        self.max_position = max_position or arch.max_position
        self.runs = arch.runs()
        gen = None
        if random_init:
            gen = torch.Generator(device=self.device)
            gen.manual_seed(seed)
        h, f32 = arch.hidden_size, torch.float32

        def rnd(*shape, scale=init_std, dt=dtype):
            t = torch.empty(*shape, dtype=dt, device=self.device)
            return t.normal_(0.0, scale, generator=gen) if gen is not None else t.zero_()

        self.embed = rnd(arch.vocab_size, h, scale=1.0)
        self.embed_norm = rnd(h, scale=0.1, dt=f32)
        self.loop_in = rnd(h, 2 * h) if arch.loop is not None else None   # [x; x0], x first
        self.layers: List[MalLayerWeights] = []
        for spec in arch.layers:
            lw, f = MalLayerWeights(), spec.mlp
            lw.norm1 = rnd(h, scale=0.1, dt=f32)
            lw.mix = SinkAttentionMixer(spec.mixer, h, self.device, dtype, gen, init_std)
            if f is not None:
                lw.norm2 = rnd(h, scale=0.1, dt=f32)
                if f.kind == "dense":
                    lw.gate_up, lw.down = rnd(2 * f.ff, h), rnd(h, f.ff)
                else:
                    lw.router = rnd(f.experts, h, scale=init_std * 4)
                    lw.w1, lw.w2 = rnd(f.experts, f.ff, h), rnd(f.experts, h, f.ff)
            self.layers.append(lw)
        self.norm = rnd(h, scale=0.1, dt=f32)
        self.lm_head = rnd(arch.vocab_size, h)
        self.embed_gain = self.gain = None
        self._fold_gains()

    # ------------------------------------------------------------------ weights
    def _slots(self, li: int) -> Dict[str, torch.Tensor]:
        """Layer li's tensors besides its mixer's, under their names after ``l<li>.`` (views where several are fused)."""
        lw, f = self.layers[li], self.arch.layers[li].mlp
        out = {"norm1": lw.norm1}
        if f is None:
            return out
        out["norm2"] = lw.norm2
        if f.kind == "dense":
            out.update({"mlp.gate": lw.gate_up[: f.ff], "mlp.up": lw.gate_up[f.ff:], "mlp.down": lw.down})
        else:
            out["mlp.router"] = lw.router
            for e in range(f.experts):
                out[f"mlp.e{e}.up"], out[f"mlp.e{e}.down"] = lw.w1[e], lw.w2[e]
        return out

    def _top(self) -> Dict[str, torch.Tensor]:
        out = {"embed": self.embed, "embed.norm": self.embed_norm, "head": self.lm_head, "final.norm": self.norm}
        if self.loop_in is not None:
            out["loop.in"] = self.loop_in
        return out

    def load_state_dict(self, tensors: Dict[str, torch.Tensor], fold: bool = True) -> int:
        """Tensors under the checkpoint's names: ``embed``, ``embed.norm``, ``loop.in``, ``head``, ``final.norm`` and, for
        layer i, ``l<i>.norm1|norm2``, ``l<i>.mix.<name>`` (the mixer's own), ``l<i>.mlp.gate|up|down`` (dense) or
        ``l<i>.mlp.router``, ``l<i>.mlp.e<j>.up|down`` (moe)."""
        n = 0
        top = self._top()
        slots = [self._slots(i) for i in range(len(self.layers))]
        for name, t in tensors.items():
            dst = top.get(name)
            if dst is None and name.startswith("l") and "." in name and name[1:name.index(".")].isdigit():
                li, rest = int(name[1:name.index(".")]), name[name.index(".") + 1:]
                if li >= len(self.layers):
                    continue
                if rest.startswith("mix."):
                    n += bool(self.layers[li].mix.load(rest[4:], t))
                    continue
                dst = slots[li].get(rest)
            if dst is not None:
                n += _put(dst, t)
        if fold:
            self.fold_norm_weights()
        return n

    def _fold_gains(self) -> None:
        self.embed_gain, self.gain = 1.0 + self.embed_norm, 1.0 + self.norm
        for lw in self.layers:
            lw.gain1 = 1.0 + lw.norm1
            lw.gain2 = 1.0 + lw.norm2 if lw.norm2 is not None else None

    def fold_norm_weights(self, layers=None) -> None:
        """Called once the weights are in: the norms' gains (one plus the stored weight) and the mixers' derived tensors."""
        for lw in self.layers:
            lw.mix.finalize()
        self._fold_gains()

    def state_dict(self) -> Dict[str, torch.Tensor]:
        out = self._top()
        for i, lw in enumerate(self.layers):
            p = f"l{i}."
            out.update({p + k: v for k, v in self._slots(i).items()})
            out.update({p + "mix." + k: v for k, v in lw.mix.state().items()})
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
        ts = [t for t in (self.embed, self.lm_head, self.loop_in) if t is not None]
        for lw in self.layers:
            ts += lw.mix.tensors() + lw.tensors()
        return sum(t.numel() * t.element_size() for t in ts)

    # ------------------------------------------------------------------- cache
    def kv_bytes_per_block(self, block_size: int) -> int:
        return max(1, self.arch.kv_bytes_per_token(self.embed.element_size())) * block_size

    def make_kv_pool(self, num_blocks: int, block_size: int) -> LayerRowPool:
        """One plane per layer run: a looped layer's passes keep their keys and values apart."""
        return LayerRowPool(self.arch.cache_widths(), num_blocks, block_size, self.device, self.dtype)

    def activation_bytes(self, tokens: int) -> int:
        """Rough peak of one step's activations (projections, expert rows, fp32 residual + logits slack)."""
        a = self.arch
        widest = 0
        for l in a.layers:
            w, f = 2 * l.mixer.channels + l.mixer.heads * l.mixer.vdim, l.mlp
            if f is not None:
                w = max(w, 3 * f.ff if f.kind == "dense" else 2 * f.top * (a.hidden_size + f.ff))
            widest = max(widest, w)
        return tokens * (20 * a.hidden_size + 4 * widest) + (1 << 30)

    # ----------------------------------------------------------------- forward
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, meta, kv_pool,
                layer_hook=None) -> torch.Tensor:
        """Final-norm hidden states [T, W] in the model dtype. ``kv_pool``: one cache tensor per layer run.
        ``layer_hook(run, residual)``: called with the fp32 residual after every layer run (a buffer that later runs
        update)."""
        eps, dt, W = self.arch.rms_eps, self.dtype, self.arch.hidden_size
        T = input_ids.shape[0]
        both = None   # [x | x0] in the model dtype, what the loop's projection reads; x0 stays for all passes
        if self.loop_in is not None:
            both = torch.empty(T, 2 * W, dtype=dt, device=input_ids.device)
        x = mix.embed_norm(input_ids, self.embed, self.embed_gain, eps, copy=None if both is None else both[:, W:])

        def target(r: int) -> Tuple[Optional[torch.Tensor], torch.Tensor]:
            """What run r (the model's end, after the last) takes from the residual: (gain, where): the normed rows, or at
            the start of a pass (gain None) the residual itself as the left half of the loop's input."""
            if r < len(self.runs):
                if self.runs[r].enter:
                    return None, both[:, :W]
                return self.layers[self.runs[r].layer].gain1, torch.empty(T, W, dtype=dt, device=x.device)
            return self.gain, torch.empty(T, W, dtype=dt, device=x.device)

        def arrive(r: int, h: torch.Tensor) -> torch.Tensor:
            """Run r's input once the residual is up to date and its target ``h`` is written."""
            nonlocal x
            if layer_hook is not None and r > 0:
                layer_hook(r - 1, x)
            if r < len(self.runs) and self.runs[r].enter:
                x, h = conv.conv_norm(None, mix.linear_f32(both, self.loop_in), self.layers[self.runs[r].layer].gain1, eps, dt,
                                      spare=x)
            return h

        def take(r: int, y: Optional[torch.Tensor]) -> torch.Tensor:
            """The residual takes the pending sublayer output; returns run r's input."""
            nonlocal x
            gain, h = target(r)
            keep = gain is not None or layer_hook is not None   # (at the start of a pass x is replaced)
            new, _ = conv.conv_norm(x, y, gain, eps, dt, out=h, keep=keep)
            x = new if keep else x
            return arrive(r, h)

        h = take(0, None)
        for r, (li, _) in enumerate(self.runs):
            lw, f = self.layers[li], self.arch.layers[li].mlp
            u = lw.mix.heads_out(mix.linear(h, lw.mix.qkv), positions, meta, kv_pool[r], eps, {})
            y = mix.linear_partials(u, lw.mix.o)
            if meta.kv_hook is not None:
                meta.kv_hook(r)
            if f is None:
                h = take(r + 1, y)
                continue
            x, h = conv.conv_norm(x, y, lw.gain2, eps, dt)
            if f.kind == "dense":
                z = mix.gated_act(mix.linear(h, lw.gate_up), mix.ACT_CLAMPED, f.limit, GATE_ALPHA)
                h = take(r + 1, mix.linear_partials(z, lw.down))
            else:
                w, ids = mix.route_grouped_topk(h, lw.router, f.top, f.groups, f.keep, f.scale)
                gain, out = target(r + 1)
                mix.moe_output_weighted(h, lw.w1, lw.w2, w, ids, mix.ACT_RELU2, 0.0, 0.0, pre_norm=(x, gain, eps, out))
                h = arrive(r + 1, out)
        return h

    def compute_logits(self, hidden: torch.Tensor, argmax_parts=None) -> torch.Tensor:
        """Logits [rows, vocab] = head(hidden) in the model dtype (what the sampling kernel reads)."""
        if argmax_parts is not None:
            raise ValueError("this head writes no per-tile argmax candidates")
        return mix.linear(hidden, self.lm_head)
