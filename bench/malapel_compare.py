#!/usr/bin/env python3
"""
Malapel beside the framework's closest existing model at equal size, random weights, one GPU
(``python bench.py --malapel-compare`` runs this; the default bench is unchanged).

Served through the same engine (scheduler, paged cache, runner, hipGraph decode, sampling) beside Datatar, which also
alternates the clamped gated feed-forward with a routed mixture over an fp32 residual (its attention is latent; as many
layers as Malapel has layer runs, and gated experts of the same width):

* prefill throughput: ``batch`` prompts of ``prompt`` tokens, prompt tokens / s of the prefill steps;
* decode throughput: ``gen`` tokens per sequence, generated tokens / s of the decode steps;

and the new design's kernels alone beside their like in the other families (events around the op, median of ``iters``),
each as a fraction of the roofline that binds it:

* attention with sigmoid weights in a window, in chunks and over everything, beside the softmax window and the Llama path's
  kernels: matrix FLOP/s over the visible pairs over the 2.5 PFLOP/s dense bf16 peak (prefill), cache bytes / time over the
  8 TB/s HBM3E peak (decode);
* the mixture: its products' FLOP/s over the bf16 peak (prefill), weight bytes / time over the HBM peak (decode), beside
  gated experts;
* the row kernels (residual + norm, embedding norm, q/k/v preparation, activations, expert sums, routing): bytes moved /
  time over the HBM peak at prefill, time at decode.

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

# width; attention heads / key-value heads / head size / window and chunk; dense width; experts / groups / kept groups / chosen
# / expert width; Datatar's latent attention
SIZES = {
    "2k": dict(hidden=2048, heads=16, kv_heads=4, dim=128, vdim=128, window=512, ff=8192, experts=16, groups=4, keep=2, top=4,
               expert_ff=1024, vocab=32000, l_dim=96, l_rot=32, l_rank=256, l_qrank=768),
    "4k": dict(hidden=4096, heads=32, kv_heads=8, dim=128, vdim=128, window=512, ff=14336, experts=32, groups=8, keep=4, top=4,
               expert_ff=2048, vocab=32000, l_dim=96, l_rot=32, l_rank=256, l_qrank=1536),
}
LOOP = (1, 3, 2)   # four layers, six layer runs


def malapel_arch(z):
    from src.models.fekolorn import SinkAttnSpec
    from src.models.malapel import MalapelArch, MalLayerSpec, RoutedMlpSpec

    att = dict(heads=z["heads"], kv_heads=z["kv_heads"], dim=z["dim"], vdim=z["vdim"], scale=1.0 / math.sqrt(z["dim"]),
               rot_dims=z["dim"], rot_base=5e5, has_sink=False)
    win = SinkAttnSpec(**att, window=z["window"], sigmoid=True)
    chunk = SinkAttnSpec(**att, seg=z["window"], qk_norm=True, unit_sink=True)
    dense = RoutedMlpSpec("dense", z["ff"], limit=7.0)
    moe = RoutedMlpSpec("moe", z["expert_ff"], experts=z["experts"], top=z["top"], groups=z["groups"], keep=z["keep"], scale=2.5)
    layers = (MalLayerSpec("attention_3", win, dense), MalLayerSpec("attention", chunk, moe),
              MalLayerSpec("attention_2", SinkAttnSpec(**att), dense), MalLayerSpec("attention_3", win, moe))
    return MalapelArch("malapel-bench", z["vocab"], z["hidden"], layers, loop=LOOP)


def datatar_arch(z):
    from src.models.datatar import DatatarArch, LatentAttnSpec, LayerSpec, MlpSpec

    m = LatentAttnSpec(heads=z["heads"], dim=z["l_dim"], rot_dim=z["l_rot"], vdim=z["vdim"], kv_rank=z["l_rank"],
                       q_rank=z["l_qrank"], scale=1.0 / math.sqrt(z["l_dim"] + z["l_rot"]), window=z["window"],
                       rot_base=10000.0, rot_dims=z["l_rot"])
    dense = MlpSpec("dense", ff=z["ff"], limit=7.0)
    moe = MlpSpec("moe", experts=z["experts"], top=z["top"], expert_ff=z["expert_ff"])
    runs = 4 + (LOOP[1] - LOOP[0]) * (LOOP[2] - 1)
    return DatatarArch("datatar-bench", z["vocab"], z["hidden"],
                       tuple(LayerSpec("latent_attention", m, moe if i % 2 else dense) for i in range(runs)))


def kernels(z, a, size):
    from src import ops
    from src.ops import conv, lin, mix, rec, seq

    dev, bf = "cuda", torch.bfloat16
    bs, S, L = 16, a.batch, a.prompt
    W = z["hidden"]
    T = S * L
    cu = torch.arange(S + 1, dtype=torch.int32, device=dev) * L
    modes = (("prefill", T, torch.arange(L, device=dev).repeat(S)), ("decode", S, torch.full((S,), L - 1, device=dev)))
    res = []

    def emit(design, kernel, mode, t, **fracs):
        r = {"design": design, "kernel": kernel, "mode": mode, "ms": round(t * 1e3, 4), **fracs, "bench": "kernel", "size": size}
        res.append(r)
        print(json.dumps(r), flush=True)

    def bw(nbytes, t):
        return {"hbm_frac_of_peak": round(nbytes / t / PEAK_HBM, 4)}

    def timed(fn):
        return _time(fn, a.iters)

    # ---- attention
    H, G, D, V = z["heads"], z["kv_heads"], z["dim"], z["vdim"]
    nb = S * (L // bs)
    bt = torch.arange(nb, dtype=torch.int32, device=dev).view(S, L // bs)
    ctx = torch.full((S,), L, dtype=torch.int32, device=dev)
    scale = 1.0 / math.sqrt(D)
    sink, pb = torch.zeros(H, device=dev), torch.full((H,), -5.0, device=dev)
    n = min(z["window"], L)
    visible = {"window": S * sum(min(i + 1, n) for i in range(L)), "chunk": S * sum(i % n + 1 for i in range(L)),
               "full": S * L * (L + 1) // 2}
    last = {"window": n, "chunk": (L - 1) % n + 1, "full": L}
    cache = (torch.randn(nb, bs, G * (D + V), device=dev) * 0.5).to(bf)
    for mode, T2, pos in modes:
        q = (torch.randn(T2, H * D, device=dev) * 0.1).to(bf)
        cuq, mq = (cu, L) if mode == "prefill" else (None, 1)
        for design, label, kind, kw in (
                ("malapel", f"sink_attn (sigmoid, window {n})", "window", dict(window=n, sigmoid=True, head_bias=pb)),
                ("kogerax", f"sink_attn (softmax, window {n})", "window", dict(window=n)),
                ("malapel", f"sink_attn (unit sink, chunks of {n})", "chunk", dict(window=0, seg=n, sink=sink)),
                ("malapel", "sink_attn (sigmoid, everything)", "full", dict(window=0, sigmoid=True, head_bias=pb)),
                ("malapel", "sink_attn (softmax, everything)", "full", dict(window=0))):
            kw = dict(kw)
            win, sk = kw.pop("window"), kw.pop("sink", None)
            t = timed(lambda: seq.sink_attn(q, cache, bt, cuq, ctx, pos, sk, None, mq, H, G, D, V, win, scale, **kw))
            fr = {"flops_frac_of_peak": round(2 * visible[kind] * H * (D + V) / t / PEAK_BF16, 4)} if mode == "prefill" \
                else bw(S * last[kind] * G * (D + V) * 2, t)
            emit(design, label, mode, t, **fr)
        C = (H + G) * D + G * V
        p = torch.randn(T2, C, device=dev).to(bf)
        slots = torch.arange(T2, device=dev)
        inv = mix.rope_inv_freq(5e5, D, dev)
        qn, kn = torch.ones(H * D, device=dev), torch.ones(G * D, device=dev)
        args = (p[:, : H * D], p[:, H * D: (H + G) * D], p[:, (H + G) * D:], cache, H, G, D, V, pos, slots, 1e-5)
        for design, label, kw in (("malapel", "qkv_prep (whole norm, rotary)", dict(q_norm=qn, k_norm=kn)),
                                  ("malapel", "qkv_prep (rotary)", {}), ("fekolorn", "qkv_prep (rotary, unit values)", dict(v_unit=True))):
            t = timed(lambda: seq.qkv_prep(*args, rot_dims=D, inv_freq=inv, **kw))
            emit(design, label, mode, t, **bw(T2 * C * 4, t))
    if ops.native_available() and D == 128 and V == 128:
        kc, vc = ((torch.randn(nb, G, bs, D, device=dev) * 0.5).to(bf) for _ in range(2))
        q = (torch.randn(T, H * D, device=dev) * 0.1).to(bf)
        t = timed(lambda: ops.attn_prefill(q, kc, vc, bt, cu, ctx, L, H, G, scale))
        emit("llama", "attn_prefill", "prefill", t, flops_frac_of_peak=round(2 * visible["full"] * H * 2 * D / t / PEAK_BF16, 4))
    # ---- residual, norms, embedding
    x, w = torch.randn(T, W, device=dev), torch.ones(W, device=dev)
    both = torch.empty(T, 2 * W, dtype=bf, device=dev)
    table, g16 = torch.randn(z["vocab"], W, device=dev).to(bf), torch.zeros(W, device=dev).to(bf)
    w_in = (torch.randn(W, 2 * W, device=dev) * 0.02).to(bf)
    for mode, T2, _ in modes:
        ids, y = torch.randint(0, z["vocab"], (T2,), device=dev), torch.randn(T2, W, device=dev).to(bf)
        act = torch.empty(T2, W, dtype=bf, device=dev)
        x2, both2 = x[:T2], both[:T2]
        t = timed(lambda: conv.conv_norm(x2, y, w, 1e-5, bf))
        emit("malapel", "conv_norm (residual, norm)", mode, t, **bw(T2 * W * 12, t))
        t = timed(lambda: conv.conv_norm(x2, y, None, 1e-5, bf, out=both2[:, :W], keep=False))
        emit("malapel", "conv_norm (residual into the loop's input)", mode, t, **bw(T2 * W * 8, t))
        t = timed(lambda: mix.post_norm_residual(x2, y, g16, 1e-5, True, act=act))
        emit("datatar", "post_norm_residual", mode, t, **bw(T2 * W * 12, t))
        t = timed(lambda: mix.embed_norm(ids, table, w, 1e-5, copy=both2[:, W:]))
        emit("malapel", "embed_norm", mode, t, **bw(T2 * W * 8, t))
        t = timed(lambda: rec.embed_scaled(ids, table, 2.0))
        emit("kogerax", "embed_scaled", mode, t, **bw(T2 * W * 8, t))
        t = timed(lambda: mix.linear_f32(both2, w_in))
        fr = {"flops_frac_of_peak": round(4 * T2 * W * W / t / PEAK_BF16, 4)} if mode == "prefill" else bw(4 * W * W, t)
        emit("malapel", "loop projection (fp32 results)", mode, t, **fr)
        t = timed(lambda: mix.linear(both2, w_in))
        fr = {"flops_frac_of_peak": round(4 * T2 * W * W / t / PEAK_BF16, 4)} if mode == "prefill" else bw(4 * W * W, t)
        emit("all", "the same product, bf16 results", mode, t, **fr)
        gu = torch.randn(T2, 2 * z["ff"], device=dev).to(bf)
        t = timed(lambda: mix.gated_act(gu, mix.ACT_CLAMPED, 7.0, 1.702))
        emit("malapel / datatar", "gated_act (clamped)", mode, t, **bw(T2 * z["ff"] * 6, t))
        del gu
    # ---- mixture: routing, experts, weighted sum
    E, K, F, ng, keep = z["experts"], z["top"], z["expert_ff"], z["groups"], z["keep"]
    router = (torch.randn(E, W, device=dev) * 0.05).to(bf)
    w1, w2 = ((torch.randn(*s, device=dev) * 0.02).to(bf) for s in ((E, F, W), (E, W, F)))
    w13 = (torch.randn(E, 2 * F, W, device=dev) * 0.02).to(bf)
    for mode, T2, _ in modes:
        h = torch.randn(T2, W, device=dev).to(bf)
        t = timed(lambda: mix.route_grouped_topk(h, router, K, ng, keep, 2.5))
        emit("malapel", "route_grouped_topk", mode, t, **bw(T2 * W * 2, t))
        t = timed(lambda: mix.route_softmax_topk(h, router, K, E))
        emit("kogerax", "route_softmax_topk", mode, t, **bw(T2 * W * 2, t))
        t = timed(lambda: mix.route_sigmoid_topk(h, router, K))
        emit("datatar", "route_sigmoid_topk", mode, t, **bw(T2 * W * 2, t))
        zr = torch.randn(T2 * K, F, device=dev).to(bf)
        t = timed(lambda: mix.relu2_act(zr))
        emit("malapel", "relu2_act", mode, t, **bw(T2 * K * F * 4, t))
        t = timed(lambda: lin.bias_relu2(zr, zr[0]))
        emit("bapivik", "bias_relu2", mode, t, **bw(T2 * K * F * 4, t))
        del zr
        p, ids = mix.route_grouped_topk(h, router, K, ng, keep, 2.5)
        ys = torch.randn(T2 * K, W, device=dev).to(bf)
        act = torch.empty(T2, W, dtype=bf, device=dev)
        kern = mix._kern()
        t = timed(lambda: kern.combine_pre_norm(x[:T2], act, ys, None, h, p, ids, E, None, None, w, False, 1e-5, 1.0))
        emit("malapel", "combine_pre_norm (sum, residual, next norm)", mode, t, **bw(T2 * W * (2 * K + 10), t))
        t = timed(lambda: kern.combine_weighted(None, x[:T2], act, ys, None, h, p, ids, E, None, None, g16, True, 1e-5, 1.0))
        emit("kogerax", "combine_weighted (sum, norm, residual)", mode, t, **bw(T2 * W * (2 * K + 10), t))
        del ys
        used = int(ids.unique().numel())
        pre = (x[:T2], w, 1e-5, act)
        post = (x[:T2], g16, 1e-5, True, act)
        for design, label, mats, fn in (
                ("malapel", "mixture (squared ReLU)", 2, lambda: mix.moe_output_weighted(h, w1, w2, p, ids, mix.ACT_RELU2, 0.0, 0.0, pre_norm=pre)),
                ("kogerax", "mixture (clamped gate)", 3, lambda: mix.moe_output_weighted(h, w13, w2, p, ids, mix.ACT_CLAMPED, 7.0, 1.702, post_norm=post + (1.0,))),
                ("datatar", "mixture (SiLU gate)", 3, lambda: mix.moe_input_scaled(h, w13, w2, p, ids, post_norm=post))):
            t = timed(fn)
            fr = {"flops_frac_of_peak": round(2 * T2 * K * mats * W * F / t / PEAK_BF16, 4)} if mode == "prefill" \
                else bw(used * mats * W * F * 2, t)
            emit(design, label, mode, t, **fr)
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
    ap.add_argument("--models", default="malapel,datatar", help="which models to serve")
    a = ap.parse_args(argv)
    assert torch.cuda.is_available(), "needs a GPU"
    from src.models.datatar import DatatarLM
    from src.models.malapel import MalapelLM

    t0 = time.time()
    summary = []
    for size in a.sizes.split(","):
        z = SIZES[size]
        if not a.skip_kernels:
            summary += kernels(z, a, size)
            torch.cuda.empty_cache()
        if a.skip_serving:
            continue
        for name, cls, arch in (("malapel", MalapelLM, malapel_arch), ("datatar", DatatarLM, datatar_arch)):
            if name in a.models.split(","):
                summary.append(serve(cls(arch(z), "cuda:0", seed=1, init_std=0.02), a, name, size))
    print(json.dumps({"bench": "malapel_compare_summary", "seconds": round(time.time() - t0, 1), "rows": summary}),
          flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
