#!/usr/bin/env python3
"""
Rerozen beside the framework's closest existing model at equal size, random weights, one GPU
(``python bench.py --rerozen-compare`` runs this; the default bench is unchanged).

Served through the same engine (scheduler, paged cache, state slots, runner, hipGraph decode, sampling) beside
Fekolorn, whose ``parallel`` layers also put rotary grouped-query attention next to a gated delta rule (one residual
stream, an attention window of the chunk's size):

* prefill throughput: ``batch`` prompts of ``prompt`` tokens, prompt tokens / s of the prefill steps;
* decode throughput: ``gen`` tokens per sequence, generated tokens / s of the decode steps;

and the new design's kernels alone beside their like in the other families (events around the op, median of
``iters``), each as a fraction of the roofline that binds it:

* the recurrences with a decay per key channel beside the same recurrences with a decay per head: FLOP/s over the
  157 TFLOP/s fp32 vector peak at prefill, state bytes / time over the 8 TB/s HBM3E peak at decode;
* chunked attention: matrix FLOP/s over the visible pairs over the 2.5 PFLOP/s dense bf16 peak (prefill), cache bytes /
  time over the HBM peak (decode), beside a window of the same size and full context;
* the row kernels (residual + norm + input convolution, q/k/v preparation, gates, GELU): bytes moved / time over the HBM
  peak at prefill, time at decode.

Prints one JSON line per measurement and a final summary line.
"""

from __future__ import annotations

import argparse
import json
import math
import os
import sys
import time

import torch

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
if ROOT not in sys.path:
    sys.path.insert(0, ROOT)


def _sibling(name):
    """A module of this folder by file (the folder shares its name with bench.py and is no package)."""
    import importlib.util

    spec = importlib.util.spec_from_file_location(name, os.path.join(ROOT, "bench", name + ".py"))
    mod = importlib.util.module_from_spec(spec)
    spec.loader.exec_module(mod)
    return mod


_dc = _sibling("design_compare")
PEAK_BF16, PEAK_HBM, _time, serve = _dc.PEAK_BF16, _dc.PEAK_HBM, _dc._time, _dc.serve
PEAK_FP32_VALU = 157.3e12

# width, layers; attention heads / key-value heads / head size / chunk; delta rule heads / kv heads / sizes; gated linear
# attention heads / sizes; low-rank widths; taps; feed-forward width
SIZES = {
    "2k": dict(hidden=2048, layers=4, heads=16, kv_heads=4, dim=128, vdim=128, chunk=512, d_heads=16, d_kv=4, d_dim=128,
               d_vdim=128, l_heads=16, l_dim=64, l_vdim=128, rank=64, conv=4, taps=4, ff=8192, vocab=32000),
    "4k": dict(hidden=4096, layers=4, heads=32, kv_heads=8, dim=128, vdim=128, chunk=512, d_heads=32, d_kv=8, d_dim=128,
               d_vdim=128, l_heads=32, l_dim=64, l_vdim=128, rank=128, conv=4, taps=4, ff=16384, vocab=32000),
}


def rerozen_arch(z):
    from src.models.fekolorn import SinkAttnSpec
    from src.models.rerozen import ChannelDeltaSpec, GatedLinearSpec, RerLayerSpec, RerozenArch, ScaledPairSpec

    att = dict(heads=z["heads"], kv_heads=z["kv_heads"], dim=z["dim"], vdim=z["vdim"], scale=1.0 / math.sqrt(z["dim"]),
               seg=z["chunk"], rot_dims=z["dim"] // 2, rot_base=5e5, has_sink=False, head_gate=True)
    delta = ScaledPairSpec(SinkAttnSpec(**att, conv=z["conv"], rot_yarn=(8.0, 4096.0, 32.0, 1.0), rot_values=True, unit_sink=True),
                           ChannelDeltaSpec(z["d_heads"], z["d_kv"], z["d_dim"], z["d_vdim"], z["conv"], rank=z["rank"]), 0.6, 0.5)
    lin = ScaledPairSpec(SinkAttnSpec(**att, qkv_bias=True, qk_norm=True, head_norm=True),
                         GatedLinearSpec(z["l_heads"], z["l_dim"], z["l_vdim"], 16.0, rank=z["rank"]), 0.8, 0.5)
    layers = tuple(RerLayerSpec("parallel_2", delta, z["ff"]) if i % 2 == 0 else RerLayerSpec("parallel", lin, z["ff"])
                   for i in range(z["layers"]))
    return RerozenArch("rerozen-bench", z["vocab"], z["hidden"], layers, taps=z["taps"], embed_scale=math.sqrt(z["hidden"]))


def fekolorn_arch(z):
    from src.models.fekolorn import FekLayerSpec, FekolornArch, GatedDeltaSpec, ParallelSpec, PolyMlpSpec, SinkAttnSpec

    left = SinkAttnSpec(z["heads"], z["kv_heads"], z["dim"], z["vdim"], 1.0 / math.sqrt(z["dim"]), window=z["chunk"],
                        rot_dims=z["dim"] // 2, v_unit=True)
    right = GatedDeltaSpec(z["d_heads"], z["d_kv"], z["d_dim"], z["d_vdim"], z["conv"])
    layers = tuple(FekLayerSpec("parallel", ParallelSpec(left, right, 0.6, 0.9), PolyMlpSpec(z["ff"])) for _ in range(z["layers"]))
    return FekolornArch("fekolorn-bench", z["vocab"], z["hidden"], layers)


def kernels(z, a, size):
    from src.ops import conv, lin, mix, rec, seq

    dev, bf = "cuda", torch.bfloat16
    bs, S, L = 16, a.batch, a.prompt
    W = z["hidden"]
    T = S * L
    cu = (torch.arange(S + 1, dtype=torch.int32, device=dev) * L)
    sl = torch.arange(S, dtype=torch.int32, device=dev)
    rags = (("prefill", T, seq.Ragged(torch.arange(L, device=dev).repeat(S), cu, sl)),
            ("decode", S, seq.Ragged(torch.full((S,), L - 1, device=dev), None, sl)))
    res = []

    def emit(design, kernel, mode, t, **fracs):
        r = {"design": design, "kernel": kernel, "mode": mode, "ms": round(t * 1e3, 4), **fracs, "bench": "kernel", "size": size}
        res.append(r)
        print(json.dumps(r), flush=True)

    def bw(nbytes, t):
        return {"hbm_frac_of_peak": round(nbytes / t / PEAK_HBM, 4)}

    def timed(fn):
        return _time(fn, a.iters)

    # ---- delta rule: decay per key channel beside decay per head
    H, G, D, V = z["d_heads"], z["d_kv"], z["d_dim"], z["d_vdim"]
    C = 2 * G * D + H * V
    state = torch.zeros(S + 1, H, D, V, device=dev)
    nv, zb, al = torch.ones(V, device=dev), torch.full((H * D,), -2.5, device=dev), torch.zeros(H, device=dev)
    for mode, T2, rag in rags:
        qkv32 = torch.randn(T2, C, device=dev) * 0.1
        bg = torch.rand(T2, 2 * H, device=dev)
        beta = bg[:, :H].contiguous()
        low = torch.randn(T2, H * D + H * V, device=dev).to(bf)
        gate = low[:, H * D:]
        for design, label, fn in (
                ("rerozen", "gated_delta (decay per key channel)", lambda: seq.gated_delta(
                    qkv32, beta, gate, nv, 1e-6, state, H, G, D, V, rag, z=low[:, : H * D], z_bias=zb, A_log=al, gate_sigmoid=True)),
                ("fekolorn", "gated_delta (decay per head)", lambda: seq.gated_delta(qkv32, bg, gate, nv, 1e-6, state, H, G, D, V, rag))):
            t = timed(fn)
            fr = {"valu_fp32_frac_of_peak": round(T2 * H * (6 if design == "fekolorn" else 7) * D * V / t / PEAK_FP32_VALU, 4)}
            emit(design, label, mode, t, **(fr if mode == "prefill" else bw(S * H * D * V * 8, t)))
        p = torch.randn(T2, C + 2 * H, device=dev).to(bf)
        cst = torch.zeros(S + 1, z["conv"] - 1, C, device=dev)
        cw = torch.randn(C, z["conv"], device=dev) * 0.3
        cwt = cw.t().contiguous()
        t = timed(lambda: seq.delta_prep(p[:, :C], p[:, C: C + H], None, cw, cst, None, None, H, G, D, V, rag, conv_wt=cwt))
        emit("rerozen", "delta_prep (write strength only)", mode, t, **bw(T2 * C * 6, t))
        t = timed(lambda: seq.delta_prep(p[:, :C], p[:, C: C + H], p[:, C + H:], cw, cst, al, al, H, G, D, V, rag, conv_wt=cwt))
        emit("fekolorn", "delta_prep", mode, t, **bw(T2 * C * 6, t))
    # ---- gated linear attention: decay per key channel beside decay per head, and their read-out
    H, D, V = z["l_heads"], z["l_dim"], z["l_vdim"]
    state = torch.zeros(S + 1, H, D, V, device=dev)
    zb = torch.ones(H * D, device=dev)
    for mode, T2, rag in rags:
        x = (torch.randn(T2, 2 * H * D + H * V, device=dev) * 0.3).to(bf)
        low = torch.randn(T2, H * D, device=dev).to(bf)
        ab = torch.rand(T2, H, 3, device=dev) * 0.5 + 0.4
        for design, label, fn in (
                ("rerozen", "gated_linear_attn (decay per key channel)", lambda: rec.gated_linear_attn(
                    x, 0, H * D, 2 * H * D, None, state, None, H, H, D, V, 0.125, rag, z=low, z_bias=zb, tau=16.0)),
                ("kogerax", "gated_linear_attn (decay per head)", lambda: rec.gated_linear_attn(
                    x, 0, H * D, 2 * H * D, ab, state, None, H, H, D, V, 0.125, rag))):
            t = timed(fn)
            fr = {"valu_fp32_frac_of_peak": round(T2 * H * 4 * D * V / t / PEAK_FP32_VALU, 4)}
            emit(design, label, mode, t, **(fr if mode == "prefill" else bw(S * H * D * V * 8, t)))
        o32, g = torch.randn(T2, H * V, device=dev), torch.randn(T2, H * V, device=dev).to(bf)
        w1, wh = torch.ones(V, device=dev), torch.ones(H * V, device=dev)
        nq, abe = torch.randn(T2, H, device=dev), torch.rand(T2, H, 3, device=dev)
        t = timed(lambda: rec.head_norm_gate(o32, None, None, g, w1, H, V, 1e-6, gate_silu=True, mult=0.5))
        emit("rerozen", "head_norm_gate (SiLU)", mode, t, **bw(T2 * H * V * 8, t))
        t = timed(lambda: rec.head_norm_gate(o32, nq, abe, g, wh, H, V, 1e-6))
        emit("kogerax", "head_norm_gate (normaliser, sigmoid)", mode, t, **bw(T2 * H * V * 8, t))
    # ---- residual + norm (+ input convolution)
    for mode, T2, rag in rags:
        x, spare = torch.randn(T2, W, device=dev), torch.empty(T2, W, device=dev)
        y = torch.randn(T2, W, device=dev).to(bf)
        w, cwt = torch.ones(W, device=dev), torch.randn(z["taps"], W, device=dev) * 0.3
        cst = torch.zeros(S + 1, z["taps"] - 1, W, device=dev)
        mq = L if mode == "prefill" else 1
        t = timed(lambda: conv.conv_norm(x, y, w, 1e-6, bf, cwt, cst, rag, mq, spare))
        emit("rerozen", "conv_norm (residual, norm, convolution)", mode, t, **bw(T2 * W * 12, t))
        t = timed(lambda: conv.conv_norm(x, y, w, 1e-6, bf))
        emit("rerozen", "conv_norm (residual, norm)", mode, t, **bw(T2 * W * 12, t))
        xs, gain = torch.randn(T2, 1, W, device=dev), torch.ones(1, device=dev)
        t = timed(lambda: seq.stream_mix_norm(xs, y, None, 1.0, 1.0, None, None, None, gain, 1e-6, bf))
        emit("fekolorn", "stream_mix_norm (one stream)", mode, t, **bw(T2 * W * 12, t))
        t = timed(lambda: lin.post_pre_norm(x, y, None, w, w, 1e-6, bf))
        emit("bapivik", "post_pre_norm", mode, t, **bw(T2 * W * 12, t))
    # ---- feed-forward activation
    for mode, T2, _ in rags:
        zf = torch.randn(T2, z["ff"], device=dev).to(bf)
        coef, b = torch.tensor([0.5, 0.3, 0.2, 0.1], device=dev), torch.zeros(z["ff"], device=dev).to(bf)
        t = timed(lambda: mix.gelu_act(zf))
        emit("rerozen", "gelu_act", mode, t, **bw(T2 * z["ff"] * 4, t))
        t = timed(lambda: seq.poly_norm_act(zf, coef, 1e-6))
        emit("fekolorn", "poly_norm_act", mode, t, **bw(T2 * z["ff"] * 4, t))
        t = timed(lambda: lin.bias_relu2(zf, b))
        emit("bapivik", "bias_relu2", mode, t, **bw(T2 * z["ff"] * 4, t))
    # ---- attention in chunks, its preparation and its gate; values as wide as the keys and twice as wide
    H, G, D = z["heads"], z["kv_heads"], z["dim"]
    nb = S * (L // bs)
    bt = torch.arange(nb, dtype=torch.int32, device=dev).view(S, L // bs)
    ctx = torch.full((S,), L, dtype=torch.int32, device=dev)
    scale = 1.0 / math.sqrt(D)
    sink = torch.zeros(H, device=dev)
    n = min(z["chunk"], L)
    visible = {"chunk": S * sum(i % n + 1 for i in range(L)), "window": S * sum(min(i + 1, n) for i in range(L)),
               "full": S * L * (L + 1) // 2}
    last = {"chunk": (L - 1) % n + 1, "window": n, "full": L}
    for V in (z["vdim"], 2 * z["vdim"]):
        cache = (torch.randn(nb, bs, G * (D + V), device=dev) * 0.5).to(bf)
        for mode, T2, rag in rags:
            q = (torch.randn(T2, H * D, device=dev) * 0.1).to(bf)
            cuq, mq = (cu, L) if mode == "prefill" else (None, 1)
            for design, kind, win, seg in (("rerozen", "chunk", 0, n), ("kogerax", "window", n, 0), ("fekolorn", "full", 0, 0)):
                if V != z["vdim"] and kind == "window":
                    continue
                t = timed(lambda: seq.sink_attn(q, cache, bt, cuq, ctx, rag.positions, sink, None, mq, H, G, D, V, win, scale, seg=seg))
                fr = {"flops_frac_of_peak": round(2 * visible[kind] * H * (D + V) / t / PEAK_BF16, 4)} if mode == "prefill" \
                    else bw(S * last[kind] * G * (D + V) * 2, t)
                emit(design, f"sink_attn ({kind}{'' if kind == 'full' else ' of ' + str(n)}, values {V})", mode, t, **fr)
            Cq = (H + G) * D + G * V
            p = torch.randn(T2, Cq, device=dev).to(bf)
            qs, ks, vs = p[:, : H * D], p[:, H * D: (H + G) * D], p[:, (H + G) * D:]
            slots = torch.arange(T2, device=dev)
            inv, vinv = mix.rope_inv_freq(5e5, D // 2, dev), mix.rope_inv_freq(5e5, V, dev)
            cwt = torch.randn(z["conv"], Cq, device=dev) * 0.3
            cst = torch.zeros(S + 1, z["conv"] - 1, Cq, device=dev)
            nbytes = T2 * Cq * 4
            t = timed(lambda: seq.qkv_prep(qs, ks, vs, cache, H, G, D, V, rag.positions, slots, 1e-6, rot_dims=D // 2,
                                           inv_freq=inv, conv_wt=cwt, conv_state=cst, rag=rag, rot_gain=1.2, v_inv_freq=vinv))
            emit("rerozen", f"qkv_prep (convolution, rotary, turned values {V})", mode, t, **bw(nbytes, t))
            bias, ones = torch.zeros(Cq, device=dev), torch.ones(D, device=dev)
            t = timed(lambda: seq.qkv_prep(qs, ks, vs, cache, H, G, D, V, rag.positions, slots, 1e-6, rot_dims=D // 2,
                                           inv_freq=inv, bias=bias, q_norm=ones, k_norm=ones, head_norm=True))
            emit("rerozen", f"qkv_prep (bias, head norm, rotary, values {V})", mode, t, **bw(nbytes, t))
            t = timed(lambda: seq.qkv_prep(qs, ks, vs, cache, H, G, D, V, rag.positions, slots, 1e-6, rot_dims=D // 2,
                                           inv_freq=inv, v_unit=True))
            emit("fekolorn", f"qkv_prep (rotary, unit values {V})", mode, t, **bw(nbytes, t))
            o, gt = torch.randn(T2, H * V, device=dev).to(bf), torch.randn(T2, H, device=dev).to(bf)
            oh = o.view(H, T2, V)
            t = timed(lambda: conv.rot_head_gate(o, gt, H, V, 0.6, rag.positions, vinv))
            emit("rerozen", f"rot_head_gate (turned back, values {V})", mode, t, **bw(T2 * H * V * 4, t))
            t = timed(lambda: conv.rot_head_gate(o, gt, H, V, 0.6))
            emit("rerozen", f"rot_head_gate (gate only, values {V})", mode, t, **bw(T2 * H * V * 4, t))
            t = timed(lambda: lin.head_gate(oh, gt))
            emit("bapivik", f"head_gate (values {V})", mode, t, **bw(T2 * H * V * 4, t))
    return res


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--sizes", default=",".join(SIZES))
    ap.add_argument("--batch", type=int, default=32)
    ap.add_argument("--prompt", type=int, default=1024)
    ap.add_argument("--gen", type=int, default=64)
    ap.add_argument("--steps", type=int, default=2)
    ap.add_argument("--warmup", type=int, default=1)
    ap.add_argument("--iters", type=int, default=10)
    ap.add_argument("--skip-serving", action="store_true")
    ap.add_argument("--skip-kernels", action="store_true")
    ap.add_argument("--models", default="rerozen,fekolorn", help="which models to serve")
    a = ap.parse_args(argv)
    assert torch.cuda.is_available(), "needs a GPU"
    from src.models.fekolorn import FekolornLM
    from src.models.rerozen import RerozenLM

    t0 = time.time()
    summary = []
    for size in a.sizes.split(","):
        z = SIZES[size]
        if not a.skip_kernels:
            summary += kernels(z, a, size)
        if a.skip_serving:
            continue
        if "rerozen" in a.models.split(","):
            summary.append(serve(RerozenLM(rerozen_arch(z), "cuda:0", seed=1, init_std=0.02), a, "rerozen", size))
        if "fekolorn" in a.models.split(","):
            summary.append(serve(FekolornLM(fekolorn_arch(z), "cuda:0", seed=1, init_std=0.02), a, "fekolorn", size))
    print(json.dumps({"bench": "rerozen_compare_summary", "seconds": round(time.time() - t0, 1), "rows": summary}),
          flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
