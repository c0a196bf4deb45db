"""
A plain, slow implementation of the Malapel design in float64, written from its equations: explicit masks, no cache, no
batching, one function per mechanism. It shares no code with ``src/`` and is what ``tests/test_malapel.py`` compares the
engine with. It also makes the tests' configurations and random weights.

Notation: ``h`` [T, W] is a sublayer's input, weights are stored [out, in] and applied as ``h @ W.T``; positions count
from 0; rms(x) = x / sqrt(mean(x^2) + eps).
"""

from __future__ import annotations

from typing import Any, Dict, List, Optional

import torch

F64 = torch.float64
GATE_SLOPE = 1.702


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm1p(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """RMS norm with a gain of one plus the stored weight."""
    return rms(x, eps) * (1.0 + w)


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


# ------------------------------------------------------------------------------------------------- positions
def rotary_frequencies(rot: Dict[str, Any]) -> torch.Tensor:
    dims = int(rot["dims"])
    return torch.tensor([float(rot["base"]) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)


def rotate(x: torch.Tensor, freqs: torch.Tensor) -> torch.Tensor:
    """x [T, heads, dim]: dimension i is paired with i + n (n = len(freqs)) and the pair turns by position * f_i; the
    dimensions from 2n on pass unchanged."""
    n = freqs.numel()
    ang = torch.arange(x.shape[0], dtype=F64)[:, None] * freqs[None, :]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., :n], x[..., n: 2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * n:]], -1)


# ----------------------------------------------------------------------------------------------------- masks
def causal_mask(T: int) -> torch.Tensor:
    i = torch.arange(T)
    return i[None, :] <= i[:, None]


def window_mask(T: int, size: int) -> torch.Tensor:
    """Distances 0 .. size - 1."""
    i = torch.arange(T)
    return causal_mask(T) & (i[:, None] - i[None, :] < size)


def chunk_mask(T: int, size: int) -> torch.Tensor:
    """Earlier positions with the same quotient by ``size``."""
    i = torch.arange(T)
    return causal_mask(T) & (i[:, None] // size == i[None, :] // size)


# ----------------------------------------------------------------------------------- weights from the scores
def softmax_weights(s: torch.Tensor, ok: torch.Tensor) -> torch.Tensor:
    e = torch.where(ok, torch.exp(s - s.masked_fill(~ok, -torch.inf).amax(-1, keepdim=True)), torch.zeros_like(s))
    return e / e.sum(-1, keepdim=True)


def softmax_one_weights(s: torch.Tensor, ok: torch.Tensor) -> torch.Tensor:
    """exp(s_j) / (1 + sum exp(s_j)): a further term of score 0 in the denominator, with no value."""
    m = s.masked_fill(~ok, -torch.inf).amax(-1, keepdim=True).clamp_min(0.0)
    e = torch.where(ok, torch.exp(s - m), torch.zeros_like(s))
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def sigmoid_weights(s: torch.Tensor, ok: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """s [H, T, T], bias [H]: every visible key weighs sigmoid(s + bias), whatever the others weigh."""
    return torch.where(ok, sigmoid(s + bias[:, None, None]), torch.zeros_like(s))


# ---------------------------------------------------------------------------------------------------- mixers
def attention(h: torch.Tensor, w: Dict[str, torch.Tensor], m: Dict[str, Any], kind: str, eps: float) -> torch.Tensor:
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    G = m["kv_heads"]
    q, k, v = h @ w["q"].T, h @ w["k"].T, (h @ w["v"].T).view(T, G, V)
    if kind == "attention":
        q, k = rms(q, eps) * w["q.norm"], rms(k, eps) * w["k.norm"]
    q, k = q.view(T, H, D), k.view(T, G, D)
    if m.get("rot"):
        fr = rotary_frequencies(m["rot"])
        q, k = rotate(q, fr), rotate(k, fr)
    of = torch.arange(H) // (H // G)                       # the key / value head of each query head
    s = torch.einsum("ihd,jhd->hij", q, k[:, of]) * m["scale"]
    if kind == "attention":
        p = softmax_one_weights(s, chunk_mask(T, m["mask"]["size"]))
    elif kind == "attention_2":
        p = softmax_weights(s, causal_mask(T))
    else:
        p = sigmoid_weights(s, window_mask(T, m["mask"]["size"]), w["pb"])
    return torch.einsum("hij,jhv->ihv", p, v[:, of]).reshape(T, H * V) @ w["o"].T


# ---------------------------------------------------------------------------------------------- feed-forward
def dense(h: torch.Tensor, w: Dict[str, torch.Tensor], m: Dict[str, Any]) -> torch.Tensor:
    lim = m["limit"]
    g = torch.clamp(h @ w["gate"].T, max=lim)
    u = torch.clamp(h @ w["up"].T, -lim, lim)
    return (g * sigmoid(GATE_SLOPE * g) * (u + 1.0)) @ w["down"].T


def route(z: torch.Tensor, r: Dict[str, Any]):
    """Logits [T, E] -> dense weights [T, E], zero for experts that were not chosen."""
    T, E = z.shape
    s = torch.softmax(z, -1)
    g = r.get("groups") or {"count": 1, "keep": 1}
    per = E // g["count"]
    out = torch.zeros_like(s)
    for t in range(T):
        best = sorted(range(g["count"]), key=lambda a: -float(s[t, a * per: (a + 1) * per].max()))[: g["keep"]]
        open_ = [e for e in range(E) if e // per in best]
        for e in sorted(open_, key=lambda e: -float(s[t, e]))[: r["top"]]:
            out[t, e] = s[t, e] * r.get("scale", 1.0)
    return out


def relu_squared(z: torch.Tensor) -> torch.Tensor:
    return torch.relu(z) ** 2


def mixture(h: torch.Tensor, w: Dict[str, torch.Tensor], m: Dict[str, Any]) -> torch.Tensor:
    p = route(h @ w["router"].T, m["router"])
    y = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        y = y + p[:, e: e + 1] * (relu_squared(h @ w[f"e{e}.up"].T) @ w[f"e{e}.down"].T)
    return y


# ----------------------------------------------------------------------------------------------------- model
def runs(config: Dict[str, Any]) -> List[Dict[str, Any]]:
    """The layers in the order in which they run; ``enter``: a pass of the loop begins right before."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [{"layer": i, "enter": False} for i in range(n)]
    out = [{"layer": i, "enter": False} for i in range(loop["start"])]
    for _ in range(loop["times"]):
        out += [{"layer": i, "enter": i == loop["start"]} for i in range(loop["start"], loop["stop"])]
    return out + [{"layer": i, "enter": False} for i in range(loop["stop"], n)]


def forward(config: Dict[str, Any], weights: Dict[str, torch.Tensor], tokens: List[int], hook=None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence. ``hook(run, x)``: the residual after every layer run."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps = float(config["norm"]["eps"])
    x = x0 = norm1p(w["embed"][torch.tensor(tokens)], w["embed.norm"], eps)
    for n, r in enumerate(runs(config)):
        i, p = r["layer"], f"l{r['layer']}."
        layer = config["layers"][i]
        if r["enter"]:
            x = torch.cat([x, x0], 1) @ w["loop.in"].T
        wm = {k[len(p) + 4:]: v for k, v in w.items() if k.startswith(p + "mix.")}
        x = x + attention(norm1p(x, w[p + "norm1"], eps), wm, layer["mixer"], layer["type"], eps)
        f = layer.get("mlp")
        if f is not None:
            wf = {k[len(p) + 4:]: v for k, v in w.items() if k.startswith(p + "mlp.")}
            x = x + (dense if f["kind"] == "dense" else mixture)(norm1p(x, w[p + "norm2"], eps), wf, f)
        if hook is not None:
            hook(n, x)
    return norm1p(x, w["final.norm"], eps) @ w["head"].T


# --------------------------------------------------------------------------------------- test configurations
def _mixer(heads, kv_heads, dim, vdim, rot_dims, base, scale, size=None) -> Dict[str, Any]:
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if rot_dims:
        m["rot"] = {"base": base, "dims": rot_dims}
    if size:
        m["mask"] = {"size": size}
    return m


def dense_mlp(ff=40, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe_mlp(experts=8, top=3, ff=20, count=4, keep=2, scale=1.5):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "scale": scale, "groups": {"count": count, "keep": keep}}}


def chunk_layer(heads=4, kv_heads=2, dim=12, vdim=10, rot_dims=8, base=300.0, scale=0.4, size=13, mlp=None):
    return {"type": "attention", "mixer": _mixer(heads, kv_heads, dim, vdim, rot_dims, base, scale, size), "mlp": mlp}


def full_layer(heads=3, kv_heads=3, dim=10, vdim=14, rot_dims=10, base=1000.0, scale=0.35, mlp=None):
    return {"type": "attention_2", "mixer": _mixer(heads, kv_heads, dim, vdim, rot_dims, base, scale), "mlp": mlp}


def window_layer(heads=6, kv_heads=2, dim=8, vdim=9, rot_dims=4, base=200.0, scale=0.45, size=17, mlp=None):
    return {"type": "attention_3", "mixer": _mixer(heads, kv_heads, dim, vdim, rot_dims, base, scale, size), "mlp": mlp}


def make_config(layers, vocab=71, width=36, eps=2e-5, loop=None) -> Dict[str, Any]:
    c = {"architecture": "Malapel", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if loop is not None:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def make_weights(config: Dict[str, Any], seed: int = 0, std: Optional[float] = None) -> Dict[str, torch.Tensor]:
    """Random weights under the checkpoint's names, rounded to bfloat16 (what a checkpoint stores)."""
    g = torch.Generator().manual_seed(seed)
    W, Vc = config["width"], config["vocab"]
    std = std or 1.0 / W ** 0.5

    def rnd(*shape, scale=None, shift=0.0):
        return (torch.randn(*shape, generator=g) * (std if scale is None else scale) + shift).to(torch.bfloat16)

    out = {"embed": rnd(Vc, W, scale=1.0), "embed.norm": rnd(W, scale=0.2), "final.norm": rnd(W, scale=0.2),
           "head": rnd(Vc, W)}
    if config.get("loop"):
        out["loop.in"] = rnd(W, 2 * W, scale=0.7 * std)
    for i, layer in enumerate(config["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = rnd(W, scale=0.2)
        out[p + "mix.q"], out[p + "mix.k"], out[p + "mix.v"] = rnd(H * D, W), rnd(G * D, W), rnd(G * V, W)
        out[p + "mix.o"] = rnd(W, H * V, scale=0.7 / (H * V) ** 0.5)
        if layer["type"] == "attention":
            out[p + "mix.q.norm"], out[p + "mix.k.norm"] = rnd(H * D, scale=0.2, shift=1.0), rnd(G * D, scale=0.2, shift=1.0)
        if layer["type"] == "attention_3":
            out[p + "mix.pb"] = rnd(H, scale=0.6, shift=-1.5)
        if f is None:
            continue
        out[p + "norm2"] = rnd(W, scale=0.2)
        if f["kind"] == "dense":
            F = f["ff"]
            out[p + "mlp.gate"], out[p + "mlp.up"] = rnd(F, W, scale=1.5 * std), rnd(F, W, scale=1.5 * std)
            out[p + "mlp.down"] = rnd(W, F, scale=0.7 / F ** 0.5)
        else:
            F = f["expert"]["ff"]
            out[p + "mlp.router"] = rnd(f["router"]["experts"], W, scale=2.0 * std)
            for e in range(f["router"]["experts"]):
                out[p + f"mlp.e{e}.up"] = rnd(F, W)
                out[p + f"mlp.e{e}.down"] = rnd(W, F, scale=1.0 / F ** 0.5)
    return out
