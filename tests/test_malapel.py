"""
Malapel on the serving engine against the plain float64 oracle (tests/malapel_oracle.py).

Every test makes its own small configuration and random weights, writes them as a checkpoint directory, loads it
through ``LLMEngine.from_pretrained`` (registry -> model class -> loader) and steps it with
``LLMEngine.replay_step`` (scheduler, block manager, runner, kernels). The CPU cases run the engine's control flow on the
plain-PyTorch op semantics; the ``gpu`` cases run the HIP kernels. Structural faults (a window or chunk one token off, a
pass that reads another pass's keys, a missing unit in a denominator, a wrong expert) are far above the fp32 tolerance, so
those cases run in fp32; bf16 cases check the served precision.
"""

import copy
import json
import math
import os
import subprocess
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import malapel_oracle as orc  # noqa: E402

F64 = torch.float64
CPU = pytest.param("cpu", id="cpu")
GPU = pytest.param("cuda:0", marks=pytest.mark.gpu, id="gpu")
DEVICES = [CPU, GPU]
TOL = {torch.float32: 2e-4, torch.bfloat16: 8e-2}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _need(device):
    if device != "cpu":
        if not torch.cuda.is_available():
            pytest.skip("no GPU")
        from src.ops import mix

        assert mix.mix_available(), "HIP extension src/_Cmix not loaded"


def save_checkpoint(path, config, weights):
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))


def make_engine(tmp_path, config, weights, device, dtype, max_tokens=512, max_seqs=4, block_size=16, name="ckpt",
                capture=False, **cfg_kw):
    from src.config import EngineConfig
    from src.engine import LLMEngine

    path = str(tmp_path / name)
    save_checkpoint(path, config, weights)
    nb = (max_tokens + block_size - 1) // block_size
    kw = dict(max_num_seqs=max_seqs, max_num_batched_tokens=nb * block_size, block_size=block_size, num_kv_blocks=nb,
              enable_prefix_caching=False, use_cuda_graph=False, preemption_mode="recompute", tuned_gemm_table=False,
              decode_window=1)
    kw.update(cfg_kw)
    return LLMEngine.from_pretrained(path, device=device, cfg=EngineConfig(**kw), max_model_len=nb * block_size,
                                     capture=capture, dtype=dtype)


def row_errs(got, want):
    """Per row: rms of the logit difference (mean taken off) over the rms of the wanted logits."""
    d = got.double() - want.double()
    d = d - d.mean(-1, keepdim=True)
    w = want.double() - want.double().mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt().clamp_min(1e-12)


def tokens_for(config, n, seed):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, config["vocab"], (n,), generator=g).tolist()


def replay(eng, steps):
    """steps: list of lists of (request id, tokens, wanted places[, ends]). Returns {rid: {position: logits row}}."""
    got, at = {}, {}
    for step in steps:
        entries, end = [], []
        for e in step:
            rid, toks, want = e[:3]
            entries.append((rid, toks, want))
            if len(e) > 3 and e[3]:
                end.append(rid)
        logits = eng.replay_step(entries, end)
        r = 0
        for rid, toks, want in entries:
            base = at.get(rid, 0)
            for w in want:
                got.setdefault(rid, {})[base + w] = logits[r]
                r += 1
            at[rid] = base + len(toks)
        for rid in end:
            at.pop(rid, None)
        assert r == logits.shape[0]
    return got


def cut(rid, toks, sizes, end=True):
    """One request alone, cut into portions of the given sizes (the rest one token at a time)."""
    steps, lo = [], 0
    sizes = list(sizes)
    while lo < len(toks):
        n = min(sizes.pop(0) if sizes else 1, len(toks) - lo)
        hi = lo + n
        steps.append([(rid, toks[lo:hi], list(range(n)), end and hi == len(toks))])
        lo = hi
    return steps


def check(got, want, tol):
    """got: {position: logits row}, want [T, vocab]. fp32: every row; bf16: the typical row is held to the tolerance and nine
    in ten to twice it (a router's close call that rounding turns the other way moves single rows by more)."""
    pos = sorted(got)
    g = torch.stack([got[p] for p in pos])
    assert torch.isfinite(g).all()
    e = row_errs(g, want[pos])
    if tol >= 1e-2:
        far = float(e.quantile(0.9))
        assert float(e.median()) < tol / 2 and (far < 2 * tol or len(pos) < 10), f"median {float(e.median()):.3e} 90% {far:.3e}"
    else:
        assert float(e.max()) < tol, f"relative error {float(e.max()):.3e} >= {tol} at {pos[int(e.argmax())]}"


CONFIGS = {
    # every mixer with every feed-forward or none, all sizes different, three passes over the middle layers
    "std": lambda: orc.make_config(
        [orc.window_layer(mlp=orc.dense_mlp()), orc.chunk_layer(mlp=orc.moe_mlp()), orc.full_layer(mlp=None),
         orc.window_layer(heads=2, kv_heads=1, dim=14, vdim=6, rot_dims=14, size=9, mlp=orc.moe_mlp(9, 2, 12, 3, 1, 0.7)),
         orc.chunk_layer(heads=3, kv_heads=1, dim=6, vdim=16, rot_dims=6, size=21, mlp=orc.dense_mlp(28, 0.6)),
         orc.full_layer(heads=4, kv_heads=1, dim=8, vdim=5, rot_dims=4, base=20.0, mlp=orc.dense_mlp(24, 2.5))], loop=(1, 4, 3)),
    # one head, no rotation, every expert group kept, one expert chosen of all; the loop over the whole stack, twice
    "odd": lambda: orc.make_config(
        [orc.chunk_layer(heads=1, kv_heads=1, dim=9, vdim=3, rot_dims=0, size=1, mlp=orc.moe_mlp(5, 1, 7, 1, 1, 1.0)),
         orc.window_layer(heads=3, kv_heads=3, dim=5, vdim=11, rot_dims=4, size=1, mlp=orc.moe_mlp(6, 6, 9, 3, 3, 1.0)),
         orc.full_layer(heads=2, kv_heads=1, dim=7, vdim=7, rot_dims=0, mlp=None)], vocab=53, width=30, eps=1e-6, loop=(0, 3, 2)),
    # no loop at all
    "flat": lambda: orc.make_config([orc.chunk_layer(mlp=orc.dense_mlp()), orc.window_layer(mlp=None)], width=20),
    # matrix-core shapes, head sizes of 32 .. 192 and values that are no multiple of 32; a single pass over the last layer
    "mc": lambda: orc.make_config(
        [orc.chunk_layer(heads=4, kv_heads=2, dim=64, vdim=64, rot_dims=32, base=10000.0, scale=0.15, size=40,
                         mlp=orc.moe_mlp(16, 4, 32, 4, 2, 2.5)),
         orc.window_layer(heads=4, kv_heads=1, dim=96, vdim=72, rot_dims=96, scale=0.1, size=50, mlp=orc.dense_mlp(96, 1.2)),
         orc.full_layer(heads=6, kv_heads=3, dim=32, vdim=40, rot_dims=16, scale=0.2, mlp=orc.dense_mlp(64)),
         orc.window_layer(heads=2, kv_heads=2, dim=176, vdim=192, rot_dims=64, scale=0.08, size=33, mlp=None)],
        vocab=128, width=64, loop=(3, 4, 1)),
}


def weights_for(config, seed=0):
    return orc.make_weights(config, seed)


# ---------------------------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W", [36, 64, 1032, 2100, 4200])
def test_residual_updates_and_norms(device, W):
    """conv_norm without a convolution in every combination: residual present or not, kept or not, normed or copied, into a
    slice of a wider buffer; the sublayer's output as rows or as partial sums. embed_norm with its strided copy."""
    _need(device)
    from src.ops import conv, mix

    g = torch.Generator().manual_seed(W)
    T, eps = 7, 3e-5
    for dt in (torch.float32, torch.bfloat16):
        tol = 2e-5 if dt == torch.float32 else 2e-2
        x0, w = torch.randn(T, W, generator=g), 1.0 + 0.2 * torch.randn(W, generator=g)
        ys = [None, torch.randn(T, W, generator=g).to(dt), torch.randn(3, T, W, generator=g)]
        for y in ys:
            for resid in (True, False):
                if y is None and not resid:
                    continue
                for normed in (True, False):
                    for keep in (True, False):
                        ref = x0.to(F64) * resid
                        if y is not None:
                            ref = ref + (y.to(F64).sum(0) if y.dim() == 3 else y.to(F64))
                        want = orc.rms(ref, eps) * w.to(F64) if normed else ref
                        wide = torch.full((T, 2 * W + 8), 3.0, dtype=dt, device=device)
                        x, h = conv.conv_norm(x0.to(device) if resid else None, None if y is None else y.to(device),
                                              w.to(device) if normed else None, eps, dt, out=wide[:, 4: 4 + W], keep=keep)
                        assert torch.allclose(h.cpu().double(), want, atol=tol, rtol=tol)
                        assert float((wide[:, :4] - 3).abs().max()) == 0 and float((wide[:, 4 + W:] - 3).abs().max()) == 0
                        if keep:
                            assert float((x.cpu().double() - ref).abs().max()) < 1e-5
                        else:
                            assert x is None
        table = torch.randn(11, W, generator=g).to(dt)
        ids = torch.randint(0, 11, (T,), generator=g)
        both = torch.zeros(T, 2 * W, dtype=dt, device=device)
        x = mix.embed_norm(ids.to(device), table.to(device), w.to(device), eps, copy=both[:, W:])
        want = orc.rms(table.to(F64)[ids], eps) * w.to(F64)
        assert x.dtype == torch.float32 and float((x.cpu().double() - want).abs().max()) < 1e-4
        assert torch.allclose(both[:, W:].cpu().double(), want, atol=tol, rtol=tol) and float(both[:, :W].abs().max()) == 0
        x = mix.embed_norm(ids.to(device), table.to(device), None, eps)
        assert float((x.cpu().double() - orc.rms(table.to(F64)[ids], eps)).abs().max()) < 1e-4
        for shape in ((5, 24), (3, 7), (300, 520)):
            z = (torch.randn(*shape, generator=g) * 2.0).to(dt)
            assert torch.allclose(mix.relu2_act(z.to(device)).cpu().double(), orc.relu_squared(z.to(F64)), atol=1e-6, rtol=tol)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("T", [1, 5, 300])
@pytest.mark.parametrize("E,K,count,keep,scale", [(12, 3, 4, 2, 1.5), (8, 8, 2, 2, 1.0), (6, 1, 6, 1, 0.5), (7, 2, 1, 1, 3.0),
                                                  (64, 8, 8, 4, 2.5), (130, 6, 10, 3, 1.0), (512, 9, 128, 5, 16.0)])
def test_group_limited_routing(device, T, E, K, count, keep, scale):
    """Decode-sized (logits and choice in one launch) and prompt-sized steps; strided inputs."""
    _need(device)
    from src.ops import mix

    g = torch.Generator().manual_seed(E * 7 + T)
    W = 40
    r = {"experts": E, "top": K, "groups": {"count": count, "keep": keep}, "scale": scale}
    for dt in (torch.float32, torch.bfloat16):
        x = torch.randn(T, W + 8, generator=g).to(dt)[:, :W]
        router = torch.randn(E, W, generator=g).to(dt) * 0.5
        z = x.to(F64) @ router.to(F64).T
        want = orc.route(z, r)
        w, ids = mix.route_grouped_topk(x.to(device), router.to(device), K, count, keep, scale)
        got = torch.zeros(T, E, dtype=F64).scatter_(1, ids.cpu().long(), w.cpu().double())
        assert ids.shape == (T, K) and all(len(set(row)) == K for row in ids.tolist())
        # the scores of a close call may swap; nothing here is that close except by chance in one row of hundreds
        bad = ((got - want).abs().amax(1) > 1e-4 * scale).sum()
        assert int(bad) <= (1 if T * E > 10000 else 0), int(bad)
    # the choice is limited to the groups: an expert that beats all but those of better groups is not taken
    z = torch.tensor([[5.0, 0.0, 4.9, 4.8, 4.7, 1.0]])
    x, router = torch.eye(6)[:1] * 1.0, torch.zeros(6, 6)
    router[:, 0] = z[0]
    w, ids = mix.route_grouped_topk(x.to(device), router.to(device), 3, 3, 2, 1.0)
    assert sorted(ids[0].tolist()) == [0, 2, 3]
    w, ids = mix.route_grouped_topk(x.to(device), router.to(device), 3, 1, 1, 1.0)
    assert sorted(ids[0].tolist()) == [0, 2, 3]
    w, ids = mix.route_grouped_topk(x.to(device), router.to(device), 2, 3, 1, 1.0)
    assert sorted(ids[0].tolist()) == [0, 1]
    assert torch.allclose(w.cpu().sum(), torch.softmax(z, -1)[0, [0, 1]].sum(), atol=1e-5)   # not renormalised
    # equal scores: the first groups and experts
    w, ids = mix.route_grouped_topk(torch.ones(T, 6, device=device), torch.ones(6, 6, device=device), 3, 3, 2, 1.0)
    assert all(row == [0, 1, 2] for row in ids.tolist())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("T", [1, 6, 40, 200])
def test_mixture_with_residual_and_next_norm(device, T):
    """moe_output_weighted with squared-ReLU experts on all its paths (decode-sized, gathered, per-expert products), its sum
    added into the residual with the next norm or a plain copy in the same launch."""
    _need(device)
    from src.ops import mix

    g = torch.Generator().manual_seed(T)
    for W, ff, E, K, count, keep in ((36, 20, 8, 3, 4, 2), (64, 32, 12, 4, 3, 2)):
        m = orc.moe_mlp(E, K, ff, count, keep, 1.5)
        for dt in (torch.float32, torch.bfloat16):
            tol = 1e-4 if dt == torch.float32 else 4e-2
            h = torch.randn(T, W, generator=g).to(dt)
            wt = {"router": (torch.randn(E, W, generator=g) * 0.4).to(dt)}
            for e in range(E):
                wt[f"e{e}.up"] = (torch.randn(ff, W, generator=g) / W ** 0.5).to(dt)
                wt[f"e{e}.down"] = (torch.randn(W, ff, generator=g) / ff ** 0.5).to(dt)
            w1 = torch.stack([wt[f"e{e}.up"] for e in range(E)]).to(device)
            w2 = torch.stack([wt[f"e{e}.down"] for e in range(E)]).to(device)
            want = orc.mixture(h.to(F64), {k: v.to(F64) for k, v in wt.items()}, m)
            p, ids = mix.route_grouped_topk(h.to(device), wt["router"].to(device), K, count, keep, 1.5)
            got = mix.moe_output_weighted(h.to(device), w1, w2, p, ids, mix.ACT_RELU2, 0.0, 0.0)
            scale = float(want.abs().max())
            assert float((got.cpu().double() - want).abs().max()) < tol * scale
            x0, nw = torch.randn(T, W, generator=g), 1.0 + 0.2 * torch.randn(W, generator=g)
            for gain in (nw, None):
                x, wide = x0.clone().to(device), torch.full((T, 2 * W), 3.0, dtype=dt, device=device)
                assert mix.moe_output_weighted(h.to(device), w1, w2, p, ids, mix.ACT_RELU2, 0.0, 0.0,
                                               pre_norm=(x, None if gain is None else gain.to(device), 1e-5, wide[:, :W])) is None
                ref = x0.to(F64) + want
                assert float((x.cpu().double() - ref).abs().max()) < tol * scale
                nref = ref if gain is None else orc.rms(ref, 1e-5) * nw.to(F64)
                assert float((wide[:, :W].cpu().double() - nref).abs().max()) < tol * max(scale, float(nref.abs().max()))
                assert float((wide[:, W:] - 3).abs().max()) == 0


def _attention_case(device, dt, kind, n_ctx, q_lo, standout, size, present=True, H=4, G=2, D=32, V=32, R=16, block=16, impl=0):
    """One sequence of n_ctx tokens whose queries q_lo .. n_ctx - 1 run as one step over scattered pages. The last query
    and the key at ``standout`` carry their weight on the unrotated dimensions and point the same way, so that key's score
    stands far above the others (and the unit in the denominator) when it is visible; its value is large. ``kind``: chunk,
    full, window. Returns (the ops' output, the oracle's) for the query rows."""
    from src.ops import mix, seq

    g = torch.Generator().manual_seed(n_ctx * 7 + standout)
    scale = 0.5
    C = (H + G) * D + G * V
    p = torch.randn(n_ctx, C, generator=g)
    p[-1, : H * D].view(H, D)[:, R:] = 12.0 / math.sqrt(D - R)
    if present:
        p[standout, H * D: (H + G) * D].view(G, D)[:, R:] = 12.0 / math.sqrt(D - R)
        p[standout, (H + G) * D:] = 9.0
    p = p.to(dt)
    pb = torch.randn(H, generator=g) - 2.0
    nb = (n_ctx + block - 1) // block
    perm = torch.randperm(nb + 3, generator=g)[:nb]
    cache = torch.zeros(nb + 3, block, G * (D + V), dtype=dt, device=device)
    pos = torch.arange(n_ctx)
    slots = perm[pos // block] * block + pos % block
    inv = mix.rope_inv_freq(100.0, R, device)
    pd = p.to(device)
    qr = seq.qkv_prep(pd[:, : H * D], pd[:, H * D: (H + G) * D], pd[:, (H + G) * D:], cache, H, G, D, V, pos.to(device),
                      slots.to(device), 1e-5, rot_dims=R, inv_freq=inv)
    nq = n_ctx - q_lo
    single = nq == 1
    kw = {"chunk": dict(seg=size), "full": {}, "window": dict(sigmoid=True, head_bias=pb.to(device))}[kind]
    out = seq.sink_attn(qr[q_lo:].contiguous(), cache, perm[None].to(torch.int32).to(device),
                        None if single else torch.tensor([0, nq], dtype=torch.int32, device=device),
                        torch.tensor([n_ctx], dtype=torch.int32, device=device), pos[q_lo:].to(device),
                        torch.zeros(H, device=device) if kind == "chunk" else None, None, nq, H, G, D, V,
                        size if kind == "window" else 0, scale, impl=impl, **kw)
    q, k, v = (x.to(F64) for x in (p[:, : H * D].view(-1, H, D), p[:, H * D: (H + G) * D].view(-1, G, D), p[:, (H + G) * D:].view(-1, G, V)))
    fr = orc.rotary_frequencies({"dims": R, "base": 100.0})
    of = torch.arange(H) // (H // G)
    s = torch.einsum("ihd,jhd->hij", orc.rotate(q, fr), orc.rotate(k, fr)[:, of]) * scale
    wts = {"chunk": lambda: orc.softmax_one_weights(s, orc.chunk_mask(n_ctx, size or n_ctx)),
           "full": lambda: orc.softmax_weights(s, orc.causal_mask(n_ctx)),
           "window": lambda: orc.sigmoid_weights(s, orc.window_mask(n_ctx, size or n_ctx), pb.to(F64))}[kind]()
    want = torch.einsum("hij,jhv->ihv", wts, v[:, of])[q_lo:]
    return out.cpu().double(), want.reshape(nq, H * V)


EDGES = [("chunk", "inside", 40, 120), ("chunk", "outside", 40, 119), ("chunk", "first", 0, 0), ("chunk", "page", 48, 144),
         ("window", "inside", 40, 110), ("window", "outside", 40, 109), ("window", "far", 0, 3), ("window", "first", 0, 0),
         ("window", "page", 60, 128), ("full", "far", 0, 3), ("full", "first", 0, 0), ("full", "page", 0, 128)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind,where,size,standout", EDGES)
@pytest.mark.parametrize("rows", ["portion", "decode"])
def test_attention_edges_and_far_keys(device, kind, where, size, standout, rows):
    """A key made to stand out just inside / just outside the last query's window or chunk, far back, on a page border and
    at position 0, for a prompt portion and for a decode row, over scattered pages. The key moves the last row by far more
    than the tolerance when visible, and not at all when not."""
    _need(device)
    n_ctx = 150
    q_lo = n_ctx - 1 if rows == "decode" else n_ctx - 37
    cases = [(torch.float32, {}), (torch.bfloat16, {})]
    if device != "cpu":   # the matrix-core form on prompt rows and on a decode row, wide keys and values
        cases += [(torch.bfloat16, {"impl": 2}), (torch.bfloat16, {"D": 96, "V": 160, "R": 24}),
                  (torch.bfloat16, {"D": 256, "V": 256, "R": 32}), (torch.bfloat16, {"D": 176, "V": 56, "R": 32, "H": 6, "G": 1}),
                  (torch.bfloat16, {"D": 64, "V": 200, "R": 48, "impl": 2}), (torch.float32, {"D": 200, "V": 136, "R": 8}),
                  (torch.bfloat16, {"D": 80, "V": 40, "R": 32, "H": 9, "G": 3, "impl": 2}),
                  (torch.bfloat16, {"D": 32, "V": 8, "R": 16, "H": 9, "G": 1}), (torch.bfloat16, {"D": 24, "V": 20, "R": 8, "H": 5, "G": 5})]
    for dt, kw in cases:
        got, want = _attention_case(device, dt, kind, n_ctx, q_lo, standout, size, **kw)
        scale = float(want.abs().max())
        tol = 2e-4 if dt == torch.float32 else 3e-2
        assert float((got - want).abs().max()) < tol * scale, (dt, kw)
        _, without = _attention_case(device, dt, kind, n_ctx, q_lo, standout, size, present=False, **kw)
        moved = float((want[-1] - without[-1]).abs().max())
        if where == "outside":
            assert moved < 1e-9
        else:
            assert moved > 1.0, (where, moved)


@pytest.mark.gpu
@pytest.mark.parametrize("size", [1, 31, 32, 33, 100, 128])
@pytest.mark.parametrize("kind", ["chunk", "window"])
def test_attention_across_row_tiles(kind, size):
    """Whole prompts over many windows or chunks on the matrix cores: sizes smaller, equal and larger than a key tile, one
    query head per key/value head and many; long contexts whose keys are split over workgroups, in decode rows and short
    portions."""
    _need("cuda:0")
    for kw in (dict(), dict(H=8, G=1, D=64, V=104, R=32), dict(H=2, G=2, D=16, V=24, R=12)):
        got, want = _attention_case("cuda:0", torch.bfloat16, kind, 333, 0, 5, size, impl=2, **kw)
        assert float((got - want).abs().max()) < 3e-2 * float(want.abs().max()), kw
    n = 20 * size + 470
    for lo in (n - 1, n - 3):
        for sz in (size, 0):
            got, want = _attention_case("cuda:0", torch.bfloat16, kind, n, lo, n - 1, sz)
            assert float((got - want).abs().max()) < 3e-2 * float(want.abs().max()), (lo, sz)


# ------------------------------------------------------------------------------------------- the model in the engine
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_and_layer_runs_match_the_oracle(tmp_path, device, name):
    _need(device)
    config = CONFIGS[name]()
    weights = weights_for(config, 1)
    toks = tokens_for(config, 90 if device != "cpu" else 50, 3)
    layers = []
    want = orc.forward(config, weights, toks, hook=lambda r, x: layers.append(x))
    eng = make_engine(tmp_path, config, weights, device, torch.float32)
    kept, fw = {}, eng.model.forward
    eng.model.forward = lambda i, p, m, k: fw(i, p, m, k, layer_hook=lambda r, x: kept.__setitem__(r, x.double().cpu().clone()))
    got = replay(eng, [[("a", toks, list(range(len(toks))), True)]])
    assert sorted(kept) == list(range(len(layers)))
    for r, x in enumerate(layers):
        assert float((kept[r] - x).abs().max()) < 1e-4 * float(x.abs().max()), r
    check(got["a"], want, TOL[torch.float32])
    eng.model.forward = fw
    again = replay(eng, [[("b", toks, list(range(len(toks))), True)]])   # without a hook: nothing kept that is not needed
    assert all(torch.equal(again["b"][p], got["a"][p]) for p in got["a"])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("sizes", [[1], [2, 2, 2, 2, 3, 2, 5], [16, 16, 16], [7, 4, 2, 13], [33]], ids=str)
def test_portions_match_the_oracle(tmp_path, device, name, sizes):
    """A prompt token by token, in portions down to two tokens, cut at page, window and chunk borders and elsewhere; the
    rest is decoded one by one."""
    _need(device)
    if device == "cpu" and name == "mc":
        pytest.skip("matrix-core shapes: GPU")
    config = CONFIGS[name]()
    weights = weights_for(config, 2)
    toks = tokens_for(config, 60, 4)
    eng = make_engine(tmp_path, config, weights, device, torch.float32)
    got = replay(eng, cut("a", toks, sizes))
    check(got["a"], orc.forward(config, weights, toks), TOL[torch.float32])


@pytest.mark.parametrize("device", DEVICES)
def test_long_decode_bf16_and_prefill_equals_decode(tmp_path, device):
    """A prompt then 100 single-token steps in bf16 (windows and chunk borders pass over decoded tokens), and the same
    positions from one whole-prompt step: both hold the oracle's logits."""
    _need(device)
    config = CONFIGS["mc" if device != "cpu" else "std"]()
    weights = weights_for(config, 4)
    toks = tokens_for(config, 130, 6)
    eng = make_engine(tmp_path, config, weights, device, torch.bfloat16)
    want = orc.forward(config, weights, toks)
    dec = replay(eng, cut("a", toks, [30]))
    check(dec["a"], want, TOL[torch.bfloat16])
    whole = replay(eng, [[("b", toks, list(range(len(toks))), True)]])
    check(whole["b"], want, TOL[torch.bfloat16])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])
def test_unequal_requests_share_steps_and_pages_are_reused(tmp_path, device, dtype):
    """Six unequal requests, at most four live, in a pool too small for all of them: portions beside single tokens,
    requests sitting out steps, finished requests' pages handed to later ones. Every request's logits equal those of the
    request alone (the oracle)."""
    _need(device)
    config = CONFIGS["std" if dtype == torch.float32 else "mc"]()
    weights = weights_for(config, 5)
    lens = {"a": 70, "b": 33, "c": 1, "d": 47, "e": 64, "f": 18}
    toks = {r: tokens_for(config, n, 10 + i) for i, (r, n) in enumerate(lens.items())}
    eng = make_engine(tmp_path, config, weights, device, dtype, max_tokens=208, max_seqs=4)

    def part(r, lo, hi):
        return (r, toks[r][lo:hi], list(range(hi - lo)), hi == lens[r])

    steps = [[part("a", 0, 17), part("b", 0, 2)], [part("a", 17, 18), part("b", 2, 33), part("c", 0, 1)],
             [part("a", 18, 50), part("d", 0, 16)], [part("d", 16, 17), part("a", 50, 51)],
             [part("a", 51, 52), part("d", 17, 18), part("e", 0, 3)], [part("e", 3, 40), part("d", 18, 47)],
             [part("a", 52, 70), part("e", 40, 41), part("f", 0, 2)], [part("f", 2, 3), part("e", 41, 42)],
             [part("f", 3, 18), part("e", 42, 64)]]
    used_blocks, got, at = {}, {}, {}
    for step in steps:
        logits = eng.replay_step([(r, t, w) for r, t, w, _ in step], [])
        k = 0
        for r, t, w, _ in step:
            used_blocks.setdefault(r, set()).update(eng.seqs[r].block_table)
            for x in w:
                got.setdefault(r, {})[at.get(r, 0) + x] = logits[k]
                k += 1
            at[r] = at.get(r, 0) + len(t)
        eng.replay_step([], [r for r, _, _, e in step if e])
    assert used_blocks["e"] & (used_blocks["b"] | used_blocks["c"] | used_blocks["a"])   # pages were handed on
    for r in lens:
        assert len(got[r]) == lens[r]
        check(got[r], orc.forward(config, weights, toks[r]), TOL[dtype])


def test_oracle_sensitivity():
    """What the engine is checked against moves by far more than the tolerance when a mechanism is altered: a window or
    chunk by one token, rotation, scales, norms, the sigmoid's numbers, the clamp, the groups, the passes."""
    config = CONFIGS["std"]()
    weights = weights_for(config, 1)
    toks = tokens_for(config, 40, 2)
    base = orc.forward(config, weights, toks)
    floor = 20 * TOL[torch.float32]

    def moved(cfg=None, w=None, t=None):
        return float(row_errs(orc.forward(cfg or config, w or weights, t or toks), base)[-20:].max())

    def with_entry(i, path, value):
        c = copy.deepcopy(config)
        node = c["layers"][i]
        for k in path[:-1]:
            node = node[k]
        node[path[-1]] = value
        return c

    for i in (0, 1, 3, 4):
        size = config["layers"][i]["mixer"]["mask"]["size"]
        assert moved(with_entry(i, ["mixer", "mask", "size"], size - 1)) > floor, i
        assert moved(with_entry(i, ["mixer", "mask", "size"], size + 1)) > floor, i
    for i in range(6):
        assert moved(with_entry(i, ["mixer", "rot", "base"], 60.0)) > floor, i
        assert moved(with_entry(i, ["mixer", "rot", "dims"], 0 if config["layers"][i]["mixer"]["rot"]["dims"] == 2 else 2)) > floor, i
        assert moved(with_entry(i, ["mixer", "scale"], 0.5)) > floor, i
    for i in (0, 4, 5):
        assert moved(with_entry(i, ["mlp", "limit"], 0.9)) > floor, i
    for i in (1, 3):
        assert moved(with_entry(i, ["mlp", "router", "scale"], 1.1)) > floor, i
        assert moved(with_entry(i, ["mlp", "router", "groups"], {"count": 1, "keep": 1})) > floor, i
    for loop in ((1, 4, 2), (1, 4, 4), (1, 3, 3), (2, 4, 3)):
        c = copy.deepcopy(config)
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
        assert moved(c) > floor, loop
    for name in ("embed.norm", "final.norm", "l0.norm1", "l3.norm2", "l1.mix.q.norm", "l1.mix.k.norm", "l0.mix.pb", "l3.mix.pb", "loop.in"):
        w = dict(weights)
        w[name] = torch.flip(weights[name], [-1])
        assert moved(w=w) > floor, name
    # the unit in the denominator
    s, ok = torch.randn(2, 9, 9, generator=torch.Generator().manual_seed(0)).to(F64), orc.chunk_mask(9, 4)
    assert float((orc.softmax_one_weights(s, ok) - orc.softmax_weights(s, ok)).abs().max()) > 0.05
    # the first token reaches the last rows through the causal layers
    assert moved(t=[(toks[0] + 1) % config["vocab"]] + toks[1:]) > floor


# ------------------------------------------------------------------------------------ generation, registry, CLI
@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_engine(tmp_path, device):
    """LLMEngine.generate (scheduler, continuous batching on three slots, sampling) continues five prompts as the oracle's
    greedy choice does: plainly, with cached prefixes (two prompts share one), from a pool so small that requests are
    preempted and recomputed, and on the GPU from captured decode graphs."""
    _need(device)
    from src.preproc import SamplingParams

    config = CONFIGS["mc" if device != "cpu" else "std"]()
    weights = weights_for(config, 7)
    prompts = [tokens_for(config, n, 20 + n) for n in (5, 1, 19, 33, 8)]
    prompts.append(prompts[3][:32] + tokens_for(config, 4, 77))
    n_new = 6

    def is_greedy(prompt, out):
        """Every generated token is the oracle's argmax given the tokens before it, or ties with it at the sampler's
        precision (the GPU sampling kernel reads the logits as bf16)."""
        lg = orc.forward(config, weights, list(prompt) + list(out))
        for i, tok in enumerate(out):
            row = lg[len(prompt) + i - 1]
            slack = 1e-3 * float(row.std()) if device == "cpu" else 2.0 ** -7 * float(row.abs().max())
            if float(row[tok]) < float(row.max()) - slack:
                return False
        return len(out) == n_new

    modes = [dict(capture=False), dict(capture=False, enable_prefix_caching=True), dict(capture=False, max_tokens=80)]
    if device != "cpu":
        modes.append(dict(capture=True, use_cuda_graph=True, graph_batch_sizes=[1, 2, 4], decode_window=4))
    for i, kw in enumerate(modes):
        eng = make_engine(tmp_path, config, weights, device, torch.float32, max_seqs=3, name=f"g{i}", **kw)
        eng.eos_token_id = None
        outs = eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.0))
        if kw.get("enable_prefix_caching"):
            outs = eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.0))   # now from the cache
        assert all(is_greedy(p, o) for p, o in zip(prompts, outs)), (kw, outs)


@pytest.mark.gpu
def test_decode_graph_replays_equal_eager_steps(tmp_path):
    """bf16 generation from captured decode graphs, replayed step after step with prompts in between, gives the tokens of
    eager steps (ties at the sampler's precision aside)."""
    _need("cuda:0")
    from src.preproc import SamplingParams

    config = CONFIGS["mc"]()
    weights = weights_for(config, 11)
    prompts = [tokens_for(config, n, 40 + n) for n in (40, 7, 21, 3)]
    eager = make_engine(tmp_path, config, weights, "cuda:0", torch.bfloat16, name="e")
    graph = make_engine(tmp_path, config, weights, "cuda:0", torch.bfloat16, name="g", capture=True, use_cuda_graph=True,
                        graph_batch_sizes=[1, 2, 4], decode_window=1)
    for eng in (eager, graph):
        eng.eos_token_id = None
    sp = SamplingParams(max_tokens=24, temperature=0.0)
    for _ in range(2):
        a, b = eager.generate(prompts, sp), graph.generate(prompts, sp)
        for p, x, y in zip(prompts, a, b):
            same = next((i for i in range(24) if x[i] != y[i]), 24)
            if same < 24:   # the first difference must be a tie
                row = orc.forward(config, weights, list(p) + list(x[:same]))[-1]
                assert abs(float(row[x[same]] - row[y[same]])) < 0.05 * float(row.std()), (same, x, y)


def test_registry_config_roundtrip(tmp_path):
    from safetensors.torch import load_file

    from src.models.malapel import MalapelArch, MalapelLM
    from src.models.registry import family_of, resolve

    config = CONFIGS["std"]()
    path = str(tmp_path / "ckpt")
    save_checkpoint(path, config, weights_for(config))
    assert family_of(path) == "malapel"
    _, arch, cls = resolve(path)
    assert cls is MalapelLM and arch.num_layers == len(orc.runs(config)) == 12
    assert [r.layer for r in arch.runs()] == [r["layer"] for r in orc.runs(config)]
    assert [r.enter for r in arch.runs()] == [r["enter"] for r in orc.runs(config)]
    assert arch.to_config() == json.loads(json.dumps(config))
    model = cls(arch, "cpu", dtype=torch.float32)
    widths = [2 * (8 + 9), 2 * (12 + 10), 3 * (10 + 14), 1 * (14 + 6), 1 * (6 + 16), 1 * (8 + 5)]
    assert arch.cache_widths() == [widths[r["layer"]] for r in orc.runs(config)]
    pool = model.make_kv_pool(3, 16)   # every pass has keys and values of its own
    assert len({t.data_ptr() for t in pool.layers}) == 12
    n = model.load_state_dict(load_file(os.path.join(path, "model.safetensors")))
    assert n == len(weights_for(config))
    again = weights_for(config, 3)   # loading again, in place
    assert model.load_state_dict(again) == len(again)
    model.save(str(tmp_path / "again"))
    back = load_file(str(tmp_path / "again" / "model.safetensors"))
    assert set(back) == set(again)
    for k, v in again.items():
        assert torch.equal(back[k].float(), v.float()), k
    assert MalapelArch.from_config(CONFIGS["flat"]()).runs() == [(0, False), (1, False)]
    bad_moe = orc.moe_mlp(9, 4, 12, 3, 1)
    for bad in (dict(type="lightning"), dict(mlp={"kind": "poly", "ff": 4}), dict(mlp=bad_moe), dict(mlp=orc.moe_mlp(8, 2, 4, 3, 2))):
        c = copy.deepcopy(config)
        c["layers"][0].update(bad)
        with pytest.raises(ValueError):
            MalapelArch.from_config(c)
    for loop in ((4, 4, 2), (-1, 2, 1), (0, 7, 2), (0, 2, 0)):
        c = copy.deepcopy(config)
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
        with pytest.raises(ValueError):
            MalapelArch.from_config(c)


@pytest.mark.parametrize("device", DEVICES)
def test_trace_runner_command_line(tmp_path, device):
    _need(device)
    import numpy as np

    config = CONFIGS["std"]()
    weights = weights_for(config, 9)
    path = str(tmp_path / "ckpt")
    save_checkpoint(path, config, weights)
    toks = tokens_for(config, 21, 1)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:12], "want": [0, 11]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[12:13], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[13:], "want": [7]}], "end": ["x"]}]
    out = str(tmp_path / "out")
    cmd = [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", out,
           "--max-tokens", "64", "--device", device]
    r = subprocess.run(cmd, input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True,
                       timeout=600, cwd=ROOT)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = orc.forward(config, weights, toks)
    a = torch.from_numpy(np.fromfile(os.path.join(out, "0.f32"), dtype="<f4").reshape(2, -1))
    b = torch.from_numpy(np.fromfile(os.path.join(out, "2.f32"), dtype="<f4").reshape(1, -1))
    assert not os.path.exists(os.path.join(out, "1.f32"))
    assert float(row_errs(torch.cat([a, b]), want[[0, 11, 20]]).max()) < TOL[torch.float32]
