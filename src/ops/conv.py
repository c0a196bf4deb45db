"""
Ops for layers whose sublayers read a convolved input, on the ``src/_Cmix`` HIP extension
(``csrc/kernels/conv_mix.hip``):

* :func:`conv_norm` — residual sum, RMS norm and a short causal convolution over the normed rows in one launch; the
  convolution's last inputs are per-sequence state;
* :func:`rot_head_gate` — the epilogue of attention over rotated values: the output turned back by the query's position,
  a sigmoid gate per head, a constant factor.

A step is a ragged batch (:class:`src.ops.seq.Ragged`); a sequence whose first row of the step is at position 0 starts
from zeros whatever its slot holds. GPU tensors always run the HIP kernels (a missing extension raises); CPU tensors run
the plain-PyTorch semantics below, which lets the engine's control flow run in CPU-only tests.
"""

from __future__ import annotations

from typing import Optional, Tuple

import torch

from .mix import _kern
from .seq import Ragged


def conv_norm(resid: Optional[torch.Tensor], y: Optional[torch.Tensor], w: Optional[torch.Tensor], eps: float,
              out_dtype: torch.dtype, conv_wt: Optional[torch.Tensor] = None, conv_state: Optional[torch.Tensor] = None,
              rag: Optional[Ragged] = None, max_q: int = 1, spare: Optional[torch.Tensor] = None,
              out: Optional[torch.Tensor] = None, keep: bool = True) -> Tuple[Optional[torch.Tensor], torch.Tensor]:
    """(x, h): x = resid + y (fp32 [T, W]; ``resid`` itself without y), n = rms(x) * w and
    h[t] = n[t] + sum_j conv_wt[j] * n[t - (taps - 1) + j] in ``out_dtype`` — over the row's own sequence, the rows
    before the step from conv_state [slots, taps - 1, W] (fp32, the most recent last), zeros before the sequence's start;
    without ``conv_wt`` h = n. ``y`` may be fp32 partial sums [n, T, W] (:func:`src.ops.mix.linear_partials`). conv_state takes the sequence's last taps - 1 rows of n. ``max_q``: most rows of one
    sequence in the step. x is written in place where no other row of the step reads the row, else into ``spare``
    (a buffer like ``resid``, or a new one); the one not returned is free afterwards. Without a convolution: ``resid`` None
    stands for zeros (x = y, in ``spare`` or a new buffer), ``w`` None for no norm (h = x), ``keep`` off leaves x unwritten
    (h alone is wanted; x is returned as None), and ``out`` is where h goes ([T, W], any row stride)."""
    like = resid if resid is not None else y
    T, W = like.shape[-2:]
    if like.is_cuda:
        h = out if out is not None else torch.empty(T, W, dtype=out_dtype, device=like.device)
        x = resid if keep else None
        if keep and (resid is None or (y is not None and conv_wt is not None and rag.cu_q is not None)):
            x = spare if spare is not None else torch.empty(T, W, dtype=torch.float32, device=like.device)
        if conv_wt is None:
            _kern().conv_norm(h, resid, x, y, w, float(eps), None, None, 1, None, None, None)
        else:
            _kern().conv_norm(h, resid, x, y, w, float(eps), conv_wt, conv_state, max_q, rag.positions, rag.cu_q,
                              rag.state_slots)
        return x, h
    x = resid
    if y is not None:
        yf = y.sum(0) if y.dim() == 3 else y.float()
        x = yf.clone() if resid is None else resid + yf
    n = x if w is None else x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w
    if conv_wt is None:
        h = n.to(out_dtype) if out is None else out.copy_(n)
        return (x if keep else None), h
    taps = conv_wt.shape[0]
    h = n.clone()
    pos = rag.positions.tolist()
    for q0, k, slot in rag.spans(T):
        hist = conv_state[slot].clone() if pos[q0] > 0 else torch.zeros(taps - 1, W)
        if 0 < pos[q0] < taps - 1:
            hist[: taps - 1 - pos[q0]] = 0
        s = torch.cat([hist, n[q0:q0 + k]], 0)
        h[q0:q0 + k] += (s.unfold(0, taps, 1) * conv_wt.t()[None]).sum(-1)
        if taps > 1:
            conv_state[slot] = s[-(taps - 1):]
    return x, h.to(out_dtype)


def rot_head_gate(o: torch.Tensor, g: torch.Tensor, heads: int, vdim: int, mult: float = 1.0,
                  positions: Optional[torch.Tensor] = None, inv_freq: Optional[torch.Tensor] = None,
                  out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """mult * sigmoid(g[t, h]) * o[t, h, :] for o [T, H * vdim], g [T, H] (any row stride); with ``inv_freq``
    [vdim / 2] every pair (i, i + vdim / 2) of o is first turned by -positions[t] * inv_freq[i]. ``out``: where to write
    (o's shape, any row stride)."""
    T = o.shape[0]
    if out is None:
        out = torch.empty(T, heads * vdim, dtype=o.dtype, device=o.device)
    if o.is_cuda:
        _kern().rot_head_gate(out, o, g, heads, vdim, positions if inv_freq is not None else None, inv_freq, float(mult))
        return out
    x = o.float().view(T, heads, vdim)
    if inv_freq is not None:
        ang = positions.float()[:, None] * inv_freq[None, :]
        c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
        u, v = x[..., : vdim // 2], x[..., vdim // 2:]
        x = torch.cat([u * c + v * s, v * c - u * s], -1)
    out.copy_((x * (mult * torch.sigmoid(g.float()))[:, :, None]).reshape(T, heads * vdim))
    return out
