"""
A plain, slow implementation of the Rerozen design in float64, written from its equations: dense masks, explicit
loops over time, no cache, no batching, one function per mechanism. It shares no code with ``src/`` and is what
``tests/test_rerozen.py`` compares the engine with. It also makes the tests' configurations and random weights.

Notation: ``h`` [T, W] is a mixer's input, weights are stored [out, in] and applied as ``h @ W.T``; positions count
from 0; rms(x) = x / sqrt(mean(x^2) + eps).
"""

from __future__ import annotations

import math
from typing import Any, Dict, List, Optional

import torch

F64 = torch.float64


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.where(x > 30.0, x, torch.log1p(torch.exp(torch.clamp(x, max=30.0))))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


# ---------------------------------------------------------------------------------------------- convolutions
def causal_conv(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x [T, C], w [C, taps]; the last column multiplies the current row, rows before the first are zero."""
    T, C = x.shape
    taps = w.shape[1]
    out = torch.zeros(T, C, dtype=F64)
    for t in range(T):
        for j in range(taps):
            src = t - (taps - 1) + j
            if src >= 0:
                out[t] += w[:, j] * x[src]
    return out


def input_conv(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """What a sublayer reads: its normed input plus a causal convolution of it."""
    return h + causal_conv(h, w)


# ------------------------------------------------------------------------------------------------- positions
def rotary_frequencies(rot: Dict[str, Any]) -> torch.Tensor:
    """base^(-2i/dims), i < dims / 2; with YaRN scaling a ramp over i blends f (fast pairs) into f / factor."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if sc:
        def pair_of(turns):     # the (fractional) pair that makes `turns` full turns over the original length
            return dims * math.log(float(sc["original"]) / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

        lo = max(math.floor(pair_of(float(sc["fast"]))), 0)
        hi = min(math.ceil(pair_of(float(sc["slow"]))), dims - 1)
        for i in range(len(f)):
            r = min(1.0, max(0.0, (i - lo) / max(hi - lo, 0.001)))
            f[i] = f[i] / float(sc["factor"]) * r + f[i] * (1.0 - r)
    return torch.tensor(f, dtype=F64)


def rotary_gain(rot: Dict[str, Any]) -> float:
    """What YaRN multiplies cosines and sines with; 1 without scaling."""
    sc = rot.get("scaling")
    return 0.1 * math.log(float(sc["factor"])) + 1.0 if sc else 1.0


def rotate(x: torch.Tensor, freqs: torch.Tensor, gain: float = 1.0, sign: float = 1.0) -> torch.Tensor:
    """x [T, heads, n]: dimension i turns together with i + len(freqs), by sign * position * freqs[i]; dimensions from
    2 len(freqs) on pass unchanged."""
    T, n = x.shape[0], freqs.numel()
    ang = sign * torch.arange(T, dtype=F64)[:, None] * freqs[None, :]
    c, s = (torch.cos(ang) * gain)[:, None, :], (torch.sin(ang) * gain)[:, None, :]
    u, v = x[..., :n], x[..., n: 2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * n:]], -1)


# ------------------------------------------------------------------------------------------------- attention
def chunk_mask(T: int, size: int) -> torch.Tensor:
    """[T, T] bool: row i sees column j <= i of its own chunk of ``size`` positions (0: every j <= i)."""
    i = torch.arange(T)
    ok = i[:, None] >= i[None, :]
    if size:
        ok = ok & ((i // size)[:, None] == (i // size)[None, :])
    return ok


def attend(q, k, v, scale: float, size: int, plus_one: bool) -> torch.Tensor:
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]; ``plus_one``: the softmax denominator has one more term 1."""
    T, H = q.shape[0], q.shape[1]
    G = k.shape[1]
    ok = chunk_mask(T, size)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * scale
        s = s.masked_fill(~ok, -math.inf)
        m = s.max(-1, keepdim=True).values.clamp_min(0.0)
        p = torch.exp(s - m)
        den = p.sum(-1, keepdim=True) + (torch.exp(-m) if plus_one else 0.0)
        out[:, hd] = (p / den) @ v[:, g]
    return out


def _heads(h, w, m):
    H, D, V = m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads") or H
    T = h.shape[0]

    def proj(name):
        y = h @ w[name].T
        if name + ".b" in w:
            y = y + w[name + ".b"]
        if name + ".conv" in w:
            y = causal_conv(y, w[name + ".conv"])
        return y

    return proj("q").view(T, H, D), proj("k").view(T, G, D), proj("v").view(T, G, V)


def head_gated_out(h, o, w) -> torch.Tensor:
    """o [T, H, V]: one sigmoid gate per head, then the output projection."""
    gate = sigmoid(h @ w["g"].T)
    return (o * gate[:, :, None]).reshape(o.shape[0], -1) @ w["o"].T


def chunked_attention(h, w: Dict[str, torch.Tensor], m: Dict[str, Any], eps: float) -> torch.Tensor:
    """Biased projections, per-head q / k norm, rotary q / k, chunks, ordinary softmax, head gates."""
    q, k, v = _heads(h, w, m)
    q, k = rms(q, eps) * w["q.norm"], rms(k, eps) * w["k.norm"]
    if m.get("rot"):
        fr, gain = rotary_frequencies(m["rot"]), rotary_gain(m["rot"])
        q, k = rotate(q, fr, gain), rotate(k, fr, gain)
    o = attend(q, k, v, float(m["scale"]), (m.get("mask") or {}).get("size") or 0, plus_one=False)
    return head_gated_out(h, o, w)


def rotated_value_attention(h, w: Dict[str, torch.Tensor], m: Dict[str, Any], eps: float) -> torch.Tensor:
    """Convolved projections, rotary q / k, values turned by their position and the output turned back by the query's,
    chunks, softmax with one more unit in the denominator, head gates."""
    q, k, v = _heads(h, w, m)
    fr, gain = rotary_frequencies(m["rot"]), rotary_gain(m["rot"])
    q, k = rotate(q, fr, gain), rotate(k, fr, gain)
    vf = rotary_frequencies({"dims": m["vdim"], "base": m["rot"]["base"]})
    o = attend(q, k, rotate(v, vf), float(m["scale"]), (m.get("mask") or {}).get("size") or 0, plus_one=True)
    return head_gated_out(h, rotate(o, vf, sign=-1.0), w)


# ------------------------------------------------------------------------------------------------ recurrences
def gated_linear(h, w: Dict[str, torch.Tensor], m: Dict[str, Any], eps: float) -> torch.Tensor:
    """S <- diag(a) S + k v^T, o = S^T q, a decay per key channel from a low-rank projection; per-head norm, SiLU gate."""
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w["q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w["k"].T).view(T, H, D)
    v = (h @ w["v"].T).view(T, H, V)
    z = (h @ w["a1"].T @ w["a2"].T + w["a2.b"]).view(T, H, D)
    a = sigmoid(z) ** (1.0 / float(m["tau"]))
    o = torch.zeros(T, H, V, dtype=F64)
    for hd in range(H):
        S = torch.zeros(D, V, dtype=F64)
        for t in range(T):
            S = a[t, hd][:, None] * S + torch.outer(k[t, hd], v[t, hd])
            o[t, hd] = S.T @ q[t, hd]
    o = (rms(o, eps) * w["norm"]).reshape(T, H * V) * silu(h @ w["g"].T)
    return o @ w["o"].T


def channel_delta(h, w: Dict[str, torch.Tensor], m: Dict[str, Any], eps: float) -> torch.Tensor:
    """Delta rule with a decay per key channel: S <- diag(g) S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q."""
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads") or H
    q = silu(causal_conv(h @ w["q"].T, w["q.conv"])).view(T, G, D)
    k = silu(causal_conv(h @ w["k"].T, w["k.conv"])).view(T, G, D)
    v = silu(causal_conv(h @ w["v"].T, w["v.conv"])).view(T, H, V)
    q, k = unit(q) * D ** -0.5, unit(k)
    beta = sigmoid(h @ w["b"].T)
    dec = softplus(h @ w["a1"].T @ w["a2"].T + w["dt_bias"]).view(T, H, D)
    dec = torch.exp(-torch.exp(w["A_log"])[None, :, None] * dec)
    o = torch.zeros(T, H, V, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        S = torch.zeros(D, V, dtype=F64)
        for t in range(T):
            S = dec[t, hd][:, None] * S
            u = beta[t, hd] * (v[t, hd] - S.T @ k[t, g])
            S = S + torch.outer(k[t, g], u)
            o[t, hd] = S.T @ q[t, g]
    gate = sigmoid(h @ w["g1"].T @ w["g2"].T)
    o = (rms(o, eps) * w["norm"]).reshape(T, H * V) * gate
    return o @ w["o"].T


def _pair(left, right):
    def f(h, w, m, eps):
        def side(p):
            return {k[len(p):]: v for k, v in w.items() if k.startswith(p)}

        return (float(m["left_scale"]) * left(h, side("left."), m["left"], eps) +
                float(m["right_scale"]) * right(h, side("right."), m["right"], eps))
    return f


MIXERS = {"parallel": _pair(chunked_attention, gated_linear), "parallel_2": _pair(rotated_value_attention, channel_delta)}


def feed_forward(h, w) -> torch.Tensor:
    return gelu_erf(h @ w["up"].T) @ w["down"].T


# ----------------------------------------------------------------------------------------------------- model
def forward(config: Dict[str, Any], weights: Dict[str, torch.Tensor], tokens: List[int], keep_layers: bool = False):
    """Logits [T, vocab] of one sequence (float64); with ``keep_layers`` also the stream after every layer."""
    W = {k: v.to(F64) for k, v in weights.items()}
    eps = float(config["norm"]["eps"])

    def sub(prefix):
        return {k[len(prefix):]: v for k, v in W.items() if k.startswith(prefix)}

    x = W["embed"][torch.tensor(tokens)] * float((config.get("embedding") or {}).get("scale", 1.0))
    kept = []
    for i, lc in enumerate(config["layers"]):
        p = f"l{i}."
        h = input_conv(rms(x, eps) * W[p + "norm1"], W[p + "canon1"])
        x = x + MIXERS[lc["type"]](h, sub(p + "mix."), lc["mixer"], eps)
        if lc.get("mlp") is not None:
            h = input_conv(rms(x, eps) * W[p + "norm2"], W[p + "canon2"])
            x = x + feed_forward(h, sub(p + "mlp."))
        kept.append(x.clone())
    logits = (rms(x, eps) * W["final.norm"]) @ W["head"].T * float(config.get("logit_scale", 1.0))
    return (logits, torch.stack(kept)) if keep_layers else logits


# ---------------------------------------------------------------------------------- configurations + weights
def tensor_shapes(config: Dict[str, Any], rank: int = 5, gate_rank: Optional[int] = None) -> Dict[str, tuple]:
    """``rank`` / ``gate_rank``: widths of the low-rank decay and gate projections (only the tensors' shapes carry them)."""
    Wd, K, out = int(config["width"]), int(config["canon"]["taps"]), {}
    gate_rank = gate_rank or rank + 2
    out["embed"] = (int(config["vocab"]), Wd)
    for i, lc in enumerate(config["layers"]):
        p, l, r = f"l{i}.", lc["mixer"]["left"], lc["mixer"]["right"]
        two = lc["type"] == "parallel_2"
        out[p + "norm1"], out[p + "canon1"] = (Wd,), (Wd, K)
        H, G, D, V = l["heads"], l.get("kv_heads") or l["heads"], l["dim"], l["vdim"]
        q = p + "mix.left."
        for nm, n in (("q", H * D), ("k", G * D), ("v", G * V)):
            out[q + nm] = (n, Wd)
            if two:
                out[q + nm + ".conv"] = (n, l["conv"])
            else:
                out[q + nm + ".b"] = (n,)
        if not two:
            out[q + "q.norm"], out[q + "k.norm"] = (D,), (D,)
        out[q + "g"], out[q + "o"] = (H, Wd), (Wd, H * V)
        H, D, V = r["heads"], r["dim"], r["vdim"]
        G = (r.get("kv_heads") or H) if two else H
        q = p + "mix.right."
        for nm, n in (("q", G * D), ("k", G * D), ("v", H * V)):
            out[q + nm] = (n, Wd)
            if two:
                out[q + nm + ".conv"] = (n, r["conv"])
        out[q + "a1"], out[q + "a2"] = (rank, Wd), (H * D, rank)
        if two:
            out[q + "b"], out[q + "A_log"], out[q + "dt_bias"] = (H, Wd), (H,), (H * D,)
            out[q + "g1"], out[q + "g2"] = (gate_rank, Wd), (H * V, gate_rank)
        else:
            out[q + "a2.b"], out[q + "g"] = (H * D,), (H * V, Wd)
        out[q + "norm"], out[q + "o"] = (V,), (Wd, H * V)
        if lc.get("mlp") is not None:
            out[p + "norm2"], out[p + "canon2"] = (Wd,), (Wd, K)
            out[p + "mlp.up"], out[p + "mlp.down"] = (lc["mlp"]["ff"], Wd), (Wd, lc["mlp"]["ff"])
    out["final.norm"], out["head"] = (Wd,), (int(config["vocab"]), Wd)
    return out


def make_weights(config: Dict[str, Any], seed: int = 0, dtype=torch.float32, **ranks) -> Dict[str, torch.Tensor]:
    """Random weights of sizes that keep every mechanism visible: gates neither saturated nor dead, decays that reach
    back tens of tokens, peaked attention. Values are rounded to bf16 so both dtypes load the same."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(config, **ranks).items():
        leaf = name.split(".")[-1]
        if name == "embed":
            t = torch.randn(shape, generator=g) * 0.5
        elif name == "head":
            t = torch.randn(shape, generator=g) * (2.0 / math.sqrt(shape[1]))
        elif leaf in ("norm", "norm1", "norm2"):
            t = 1.0 + torch.randn(shape, generator=g) * 0.2
        elif leaf in ("canon1", "canon2"):
            t = torch.randn(shape, generator=g) * 0.35
        elif leaf == "conv":
            t = torch.randn(shape, generator=g) * 0.5
        elif leaf == "A_log":
            t = torch.log(0.1 + 1.0 * torch.rand(shape, generator=g))
        elif leaf == "dt_bias":
            t = torch.randn(shape, generator=g) * 0.7 - 2.5
        elif name.endswith("a2.b"):
            t = torch.randn(shape, generator=g) * 1.0 + 1.0
        elif leaf == "b" and len(shape) == 1:
            t = torch.randn(shape, generator=g) * 0.3
        else:
            t = torch.randn(shape, generator=g) * (1.3 / math.sqrt(shape[-1]))
        out[name] = t.to(torch.bfloat16).to(dtype)
    return out


# layer entries of a configuration
def _left(heads, kv_heads, dim, vdim, chunk, rot_dims, rot_base, scale) -> Dict[str, Any]:
    m: Dict[str, Any] = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk:
        m["mask"] = {"size": chunk}
    if rot_dims:
        m["rot"] = {"base": rot_base, "dims": rot_dims}
    return m


def gla_layer(heads=4, kv_heads=2, dim=12, vdim=8, chunk=11, rot_dims=8, rot_base=100.0, scale=0.4, r_heads=3, r_dim=6,
              r_vdim=10, tau=4.0, left_scale=0.7, right_scale=0.45, ff: Optional[int] = 40) -> Dict[str, Any]:
    return {"type": "parallel", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"left": _left(heads, kv_heads, dim, vdim, chunk, rot_dims, rot_base, scale), "left_scale": left_scale,
                      "right": {"heads": r_heads, "dim": r_dim, "vdim": r_vdim, "tau": tau}, "right_scale": right_scale}}


def delta_layer(heads=4, kv_heads=2, dim=8, vdim=12, chunk=7, rot_dims=6, rot_base=50.0, scaling=(4.0, 8.0, 1.0, 60),
                scale=0.35, conv=3, r_heads=4, r_kv_heads=2, r_dim=10, r_vdim=6, r_conv=4, left_scale=0.5, right_scale=0.8,
                ff: Optional[int] = 40) -> Dict[str, Any]:
    left = _left(heads, kv_heads, dim, vdim, chunk, rot_dims, rot_base, scale)
    left["conv"] = conv
    if scaling:
        left["rot"]["scaling"] = dict(zip(("factor", "fast", "slow", "original"), scaling))
    return {"type": "parallel_2", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"left": left, "left_scale": left_scale, "right_scale": right_scale,
                      "right": {"heads": r_heads, "kv_heads": r_kv_heads, "dim": r_dim, "vdim": r_vdim, "conv": r_conv}}}


def make_config(layers, vocab=67, width=32, eps=1e-5, embed_scale=3.0, taps=4, logit_scale=0.6) -> Dict[str, Any]:
    return {"architecture": "Rerozen", "canon": {"taps": taps}, "embedding": {"scale": embed_scale}, "layers": layers,
            "logit_scale": logit_scale, "norm": {"eps": eps}, "vocab": vocab, "width": width}
