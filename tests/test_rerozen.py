"""
Rerozen on the serving engine against the plain float64 oracle (tests/rerozen_oracle.py).

Every test makes its own small configuration and random weights, writes them as a checkpoint directory, loads it
through ``LLMEngine.from_pretrained`` (registry -> model class -> loader) and steps it with
``LLMEngine.replay_step`` (scheduler, block manager with state slots, runner, kernels). The CPU cases run the engine's
control flow on the plain-PyTorch op semantics; the ``gpu`` cases run the HIP kernels. Structural faults (a chunk one
token off, a lost state, a convolution that forgets the previous step) are far above the fp32 tolerance, so those cases
run in fp32; bf16 cases check the served precision.
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
import rerozen_oracle as orc  # noqa: E402

F64 = torch.float64
CPU = pytest.param("cpu", id="cpu")
GPU = pytest.param("cuda:0", marks=pytest.mark.gpu, id="gpu")
DEVICES = [CPU, GPU]
TOL = {torch.float32: 3e-4, torch.bfloat16: 8e-2}
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
    """got: {position: logits row}, want [T, vocab]. fp32: every row; bf16: the typical row is held to the tolerance and no
    row may be far off (a structural fault moves rows by O(1))."""
    pos = sorted(got)
    g = torch.stack([got[p] for p in pos])
    assert torch.isfinite(g).all()
    e = row_errs(g, want[pos])
    if tol >= 1e-2:
        assert float(e.median()) < tol / 2 and float(e.max()) < 4 * tol, f"median {float(e.median()):.3e} max {float(e.max()):.3e}"
    else:
        assert float(e.max()) < tol, f"relative error {float(e.max()):.3e} >= {tol} at {pos[int(e.argmax())]}"


CONFIGS = {
    # both layer types twice, every head count, size and chunk different; a layer without feed-forward
    "std": lambda: orc.make_config(
        [orc.delta_layer(), orc.gla_layer(),
         orc.delta_layer(heads=2, kv_heads=1, dim=14, vdim=6, chunk=19, rot_dims=14, scaling=(2.0, 4.0, 0.5, 90), conv=4,
                         r_heads=3, r_kv_heads=1, r_dim=5, r_vdim=9, r_conv=2, left_scale=1.1, right_scale=0.6, ff=None),
         orc.gla_layer(heads=3, kv_heads=3, dim=7, vdim=5, chunk=23, rot_dims=4, r_heads=2, r_dim=9, r_vdim=4, tau=16.0,
                       left_scale=0.4, right_scale=1.2, ff=24)]),
    # one head, one tap everywhere, whole heads rotated, no chunks, no scaling of positions, embedding or logits
    "odd": lambda: orc.make_config(
        [orc.gla_layer(heads=1, kv_heads=1, dim=10, vdim=3, chunk=0, rot_dims=10, r_heads=1, r_dim=3, r_vdim=7, tau=1.0,
                       left_scale=1.0, right_scale=1.0, ff=11),
         orc.delta_layer(heads=3, kv_heads=1, dim=9, vdim=10, chunk=0, rot_dims=4, scaling=None, conv=1, r_heads=1,
                         r_kv_heads=1, r_dim=7, r_vdim=3, r_conv=1, left_scale=1.0, right_scale=1.0, ff=None)],
        vocab=53, width=30, eps=1e-6, embed_scale=1.0, taps=1, logit_scale=1.0),
    # matrix-core shapes: attention heads of 32 .. 192, wider recurrent heads
    "mc": lambda: orc.make_config(
        [orc.delta_layer(heads=4, kv_heads=2, dim=64, vdim=64, chunk=40, rot_dims=32, rot_base=10000.0,
                         scaling=(8.0, 32.0, 1.0, 512), scale=0.2, conv=3, r_heads=4, r_kv_heads=2, r_dim=32, r_vdim=64,
                         r_conv=4, ff=96),
         orc.gla_layer(heads=4, kv_heads=1, dim=96, vdim=160, chunk=56, rot_dims=48, scale=0.15, r_heads=2, r_dim=64,
                       r_vdim=32, tau=8.0, ff=64),
         orc.delta_layer(heads=2, kv_heads=1, dim=176, vdim=192, chunk=72, rot_dims=64, scale=0.1, conv=2, r_heads=2,
                         r_kv_heads=2, r_dim=80, r_vdim=40, r_conv=3, ff=None)], vocab=128, width=64, taps=3),
}


def weights_for(config, seed=0, **kw):
    return orc.make_weights(config, seed, **kw)


def _rag(device, pos, cu, slots):
    from src.ops import seq

    return seq.Ragged(torch.tensor(pos, device=device), None if cu is None else torch.tensor(cu, dtype=torch.int32, device=device),
                      torch.tensor(slots, dtype=torch.int32, device=device))


def _steps(portions, slots, lens):
    """Shared steps of several sequences: per step (rows per sequence, positions, cu or None, slots, max rows)."""
    at = [0] * len(lens)
    for step in portions:
        rows, pos, cu, sl = [], [], [0], []
        for s, n in step:
            rows.append((s, at[s], n))
            pos += list(range(at[s], at[s] + n))
            cu.append(cu[-1] + n)
            sl.append(slots[s])
            at[s] += n
            assert at[s] <= lens[s]
        single = all(n == 1 for _, n in step)
        yield rows, pos, None if single else cu, sl, max(n for _, n in step)


PORTIONS = [[(0, 5), (1, 1)], [(0, 1)], [(0, 2), (1, 2)], [(1, 6)], [(0, 1), (1, 1)], [(0, 70)], [(1, 3), (0, 2)]]
LENS = (81, 14)


# ---------------------------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W,taps", [(48, 3), (30, 2), (1032, 4), (24, 1), (40, 7), (2100, 3), (4200, 2), (8200, 3), (1500, 5)])
def test_input_convolution_with_norm_and_residual(device, W, taps):
    """conv_norm: two sequences in shared steps (portions down to one token and longer than a workgroup's tile), in slots
    that hold stale rows; the residual takes the sublayer's output, the convolution runs over the normed rows of earlier
    steps."""
    _need(device)
    from src.ops import conv

    g = torch.Generator().manual_seed(W + taps)
    eps = 1e-5
    for dt in (torch.float32, torch.bfloat16):
        w = 1.0 + 0.2 * torch.randn(W, generator=g)
        cw = 0.5 * torch.randn(W, taps, generator=g)
        xs = [torch.randn(n, W, generator=g) for n in LENS]
        ys = [torch.randn(n, W, generator=g).to(dt) for n in LENS]
        sums = [x.to(F64) + y.to(F64) for x, y in zip(xs, ys)]
        want = [orc.input_conv(orc.rms(s, eps) * w.to(F64), cw.to(F64)) for s in sums]
        state = torch.full((4, taps - 1, W), 7.0, device=device)
        got = [[], []]
        for rows, pos, cu, sl, mq in _steps(PORTIONS, [2, 0], LENS):
            x = torch.cat([xs[s][a:a + n] for s, a, n in rows]).to(device)
            y = torch.cat([ys[s][a:a + n] for s, a, n in rows]).to(device)
            new, h = conv.conv_norm(x, y, w.to(device), eps, dt, cw.t().contiguous().to(device), state,
                                    _rag(device, pos, cu, sl), mq)
            ref = torch.cat([sums[s][a:a + n] for s, a, n in rows])
            assert float((new.cpu().double() - ref).abs().max()) < 1e-5
            i = 0
            for s, a, n in rows:
                got[s].append(h[i: i + n].cpu().double())
                i += n
        tol = 2e-5 if dt == torch.float32 else 2e-2
        for s in range(2):
            out = torch.cat(got[s])
            assert torch.allclose(out, want[s][: out.shape[0]], atol=tol, rtol=tol), (dt, s)
        if taps > 1:
            assert float(state[1].min()) == 7.0 and float(state[3].max()) == 7.0    # other slots untouched
            keep = (orc.rms(sums[0], eps) * w.to(F64))[-(taps - 1):]
            assert torch.allclose(state[2].cpu().double(), keep, atol=1e-5)
        # the sublayer's output as fp32 partial sums, as a split product leaves it; one row per sequence
        if dt == torch.float32:
            parts = torch.randn(3, 2, W, generator=g)
            x2 = torch.stack([xs[0][0], xs[1][0]])
            state.fill_(7.0)
            new, h = conv.conv_norm(x2.to(device), parts.to(device), w.to(device), eps, dt, cw.t().contiguous().to(device), state,
                                    _rag(device, [0, 0], None, [3, 1]), 1)
            ref = x2.to(F64) + parts.to(F64).sum(0)
            assert float((new.cpu().double() - ref).abs().max()) < 1e-5
            want2 = orc.rms(ref, eps) * w.to(F64) * (1.0 + cw[:, -1].to(F64))
            assert torch.allclose(h.cpu().double(), want2, atol=tol, rtol=tol)
        # no convolution, no sublayer output: the plain norm
        x = xs[0].to(device)
        same, h = conv.conv_norm(x, None, w.to(device), eps, dt)
        assert same is x and torch.allclose(h.cpu().double(), orc.rms(xs[0].to(F64), eps) * w.to(F64), atol=tol, rtol=tol)


@pytest.mark.gpu
def test_input_convolution_in_large_steps():
    """Thousands of rows per step (several rows per workgroup), unequal sequences beside single rows, cut at places that
    are no multiple of a workgroup's rows: equal to the convolution over whole sequences."""
    _need("cuda:0")
    from src.ops import conv

    g = torch.Generator().manual_seed(3)
    W, taps, eps = 64, 3, 1e-6
    lens = (7001, 1203, 2, 4099)
    w, cw = 1.0 + 0.1 * torch.randn(W, generator=g), 0.5 * torch.randn(W, taps, generator=g)
    xs = [torch.randn(n, W, generator=g) for n in lens]
    ys = [torch.randn(n, W, generator=g) for n in lens]
    norm = [orc.rms(x.to(F64) + y.to(F64), eps) * w.to(F64) for x, y in zip(xs, ys)]

    def ref(n):
        pad = torch.cat([torch.zeros(taps - 1, W, dtype=F64), n])
        return n + sum(pad[j: j + n.shape[0]] * cw[:, j].to(F64) for j in range(taps))

    state = torch.full((5, taps - 1, W), -3.0, device="cuda:0")
    portions = [[(0, 5002), (1, 1), (3, 97)], [(1, 1201), (0, 1), (2, 1), (3, 4001)], [(2, 1), (3, 1), (1, 1)], [(0, 1998)]]
    got = [[] for _ in lens]
    for rows, pos, cu, sl, mq in _steps(portions, [4, 1, 0, 3], lens):
        x = torch.cat([xs[s][a:a + n] for s, a, n in rows]).cuda()
        y = torch.cat([ys[s][a:a + n] for s, a, n in rows]).cuda()
        _, h = conv.conv_norm(x, y, w.cuda(), eps, torch.float32, cw.t().contiguous().cuda(), state, _rag("cuda:0", pos, cu, sl), mq)
        i = 0
        for s, a, n in rows:
            got[s].append(h[i: i + n].cpu().double())
            i += n
    for s in range(len(lens)):
        out = torch.cat(got[s])
        assert float((out - ref(norm[s])[: out.shape[0]]).abs().max()) < 3e-5, s


@pytest.mark.parametrize("device", DEVICES)
def test_gelu_and_head_gate_and_frequencies(device):
    _need(device)
    from src.ops import conv, mix

    g = torch.Generator().manual_seed(0)
    for dt in (torch.float32, torch.bfloat16):
        tol = 2e-6 if dt == torch.float32 else 2e-2
        for shape in ((5, 24), (3, 7), (300, 520)):
            z = (torch.randn(*shape, generator=g) * 2.5).to(dt)
            assert torch.allclose(mix.gelu_act(z.to(device)).cpu().double(), orc.gelu_erf(z.to(F64)), atol=tol, rtol=tol)
        for H, V in ((3, 10), (4, 16), (2, 24), (16, 128)):
            T = 9
            o = torch.randn(T, H * V, generator=g).to(dt)
            gt = torch.randn(T, H + 5, generator=g).to(dt)[:, 2: 2 + H]
            pos = torch.randint(0, 4000, (T,), generator=g)
            freq = orc.rotary_frequencies({"dims": V, "base": 500.0})
            for turned in (False, True):
                x = o.to(F64).view(T, H, V)
                if turned:
                    ang = pos.to(F64)[:, None] * freq.float().to(F64)
                    c, s = torch.cos(ang)[:, None], torch.sin(ang)[:, None]
                    u, v = x[..., : V // 2], x[..., V // 2:]
                    x = torch.cat([u * c + v * s, v * c - u * s], -1)
                want = (0.7 * x * orc.sigmoid(gt.to(F64))[:, :, None]).reshape(T, H * V)
                wide = torch.zeros(T, H * V + 12, dtype=dt, device=device)
                conv.rot_head_gate(o.to(device), gt.to(device), H, V, 0.7, pos.to(device) if turned else None,
                                   freq.float().to(device) if turned else None, out=wide[:, 8: 8 + H * V])
                # fp32 angles: up to 4000 radians, so about 1e-4 of rounding
                assert torch.allclose(wide[:, 8: 8 + H * V].cpu().double(), want, atol=max(tol, 6e-4), rtol=tol)
                assert float(wide[:, :8].abs().max()) == 0 and float(wide[:, 8 + H * V:].abs().max()) == 0
    for rot in ({"base": 50.0, "dims": 6, "scaling": {"factor": 4.0, "fast": 8.0, "slow": 1.0, "original": 60}},
                {"base": 10000.0, "dims": 64, "scaling": {"factor": 16.0, "fast": 32.0, "slow": 1.0, "original": 4096}},
                {"base": 10.0, "dims": 4, "scaling": {"factor": 2.0, "fast": 1.0, "slow": 1.0, "original": 6}}):
        sc = rot["scaling"]
        f, gain = mix.rope_inv_freq_yarn(rot["base"], rot["dims"], device, sc["factor"], sc["original"], sc["fast"], sc["slow"])
        assert torch.allclose(f.cpu().double(), orc.rotary_frequencies(rot), rtol=1e-6)
        assert abs(gain - orc.rotary_gain(rot)) < 1e-12


def _mixer_case(device, layer, dt=torch.float32, W=24, seed=0, **ranks):
    """A recurrent mixer alone (its projections by the oracle's matrices, no attention beside it): two sequences in shared
    steps, portions down to one token and longer than several staging trips, in slots with stale content, against the
    oracle's loop over each whole sequence. The output lands in a slice of a wider buffer."""
    from src.models import rerozen as rz
    from src.ops import mix

    config = orc.make_config([layer], width=W)
    weights = weights_for(config, seed, **ranks)
    spec_fn, cls = rz.REROZEN_MIXERS[layer["type"]]
    pair = cls(spec_fn(layer["mixer"]), W, device, dt, None, 0.0)
    w = {k[len("l0.mix."):]: v for k, v in weights.items() if k.startswith("l0.mix.")}
    for k, v in w.items():
        assert pair.load(k, v), k
    pair.finalize()
    g = torch.Generator().manual_seed(seed + 5)
    xs = [(torch.randn(n, W, generator=g) * 1.5).to(dt) for n in LENS]
    ofn = {"parallel": orc.gated_linear, "parallel_2": orc.channel_delta}[layer["type"]]
    wr = {k[6:]: v.to(F64) for k, v in w.items() if k.startswith("right.")}
    want = [ofn(x.to(F64), wr, layer["mixer"]["right"], 1e-5) for x in xs]
    r = pair.right
    state = {k: torch.full((4,) + tuple(shape), 7.0, dtype=sdt, device=device) for k, (shape, sdt) in r.spec.state_shapes().items()}
    got = [[], []]
    nv = r.spec.heads * r.spec.vdim
    for rows, pos, cu, sl, _ in _steps(PORTIONS, [2, 0], LENS):
        h = torch.cat([xs[s][a:a + n] for s, a, n in rows]).to(device)
        p = mix.linear(h, pair.w_in)
        low = mix.linear(p[:, pair.low_cols[0]: pair.low_cols[1]], pair.w_low)
        u = torch.zeros(h.shape[0], nv + 8, dtype=dt, device=device)
        r.recur(p, pair.at, low, 1e-5, state, _rag(device, pos, cu, sl), 2.0, u[:, 4: 4 + nv])
        assert float(u[:, :4].abs().max()) == 0 and float(u[:, 4 + nv:].abs().max()) == 0
        y = mix.linear(0.5 * u[:, 4: 4 + nv], r.o).cpu().double()
        i = 0
        for s, a, n in rows:
            got[s].append(y[i: i + n])
            i += n
    for s in range(2):
        out = torch.cat(got[s])
        ref = want[s][: out.shape[0]]
        if dt == torch.float32:
            assert float((out - ref).abs().max()) < 2e-4 * float(ref.abs().max()), s
        else:   # a norm over a narrow head magnifies single rounding errors; the whole is held
            assert float((out - ref).pow(2).mean().sqrt()) < 5e-2 * float(ref.pow(2).mean().sqrt()), s
    for t in state.values():
        if t.numel():
            assert float(t[1].min()) == 7.0 and float(t[3].max()) == 7.0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,D,V,tau,rank", [(2, 5, 7, 4.0, 3), (3, 16, 16, 1.0, 1), (2, 64, 136, 16.0, 12), (1, 128, 40, 8.0, 16), (2, 200, 24, 2.0, 9)])
def test_gated_linear_attention_in_portions(device, H, D, V, tau, rank):
    _need(device)
    layer = orc.gla_layer(r_heads=H, r_dim=D, r_vdim=V, tau=tau)
    _mixer_case(device, layer, seed=D, rank=rank)
    if device != "cpu":
        _mixer_case(device, layer, dt=torch.bfloat16, seed=D, rank=rank)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,V,K,rank", [(3, 1, 5, 7, 1, 3), (4, 2, 16, 8, 4, 5), (2, 2, 64, 128, 3, 16), (6, 3, 24, 20, 2, 8), (1, 1, 130, 36, 5, 4)])
def test_channel_delta_rule_in_portions(device, H, G, D, V, K, rank):
    _need(device)
    layer = orc.delta_layer(r_heads=H, r_kv_heads=G, r_dim=D, r_vdim=V, r_conv=K)
    _mixer_case(device, layer, seed=D, rank=rank, gate_rank=rank + 3)
    if device != "cpu":
        _mixer_case(device, layer, dt=torch.bfloat16, seed=D, rank=rank, gate_rank=rank + 3)


def _attention_case(device, dt, n_ctx, q_lo, standout, chunk, present=True, H=4, G=2, D=32, V=32, R=16, block=16, impl=0,
                    rotate_values=True):
    """One sequence of n_ctx tokens whose queries q_lo .. n_ctx - 1 run as one step over scattered pages. The last query
    and the key at ``standout`` carry their weight on the unrotated dimensions and point the same way, so that key's score
    stands far above the others (and the unit in the denominator) when it is visible; its value is large. Returns (ops'
    output, oracle output) for the query rows, with random head gates."""
    from src.ops import mix, seq

    g = torch.Generator().manual_seed(n_ctx * 7 + standout)
    scale = 0.5
    rot = {"base": 100.0, "dims": R, "scaling": {"factor": 8.0, "fast": 4.0, "slow": 1.0, "original": 40}}
    C = (H + G) * D + G * V
    p = torch.randn(n_ctx, C, generator=g)
    p[-1, : H * D].view(H, D)[:, R:] = 12.0 / math.sqrt(D - R)
    if present:
        p[standout, H * D: (H + G) * D].view(G, D)[:, R:] = 12.0 / math.sqrt(D - R)
        p[standout, (H + G) * D:] = 9.0
    p = p.to(dt)
    nb = (n_ctx + block - 1) // block
    perm = torch.randperm(nb + 3, generator=g)[:nb]
    cache = torch.zeros(nb + 3, block, G * (D + V), dtype=dt, device=device)
    pos = torch.arange(n_ctx)
    slots = perm[pos // block] * block + pos % block
    inv, gain = mix.rope_inv_freq_yarn(100.0, R, device, 8.0, 40, 4.0, 1.0)
    vf = mix.rope_inv_freq(100.0, V, device) if rotate_values else None
    pd = p.to(device)
    qr = seq.qkv_prep(pd[:, : H * D], pd[:, H * D: (H + G) * D], pd[:, (H + G) * D:], cache, H, G, D, V, pos.to(device),
                      slots.to(device), 1e-5, rot_dims=R, inv_freq=inv, rot_gain=gain, v_inv_freq=vf)
    nq = n_ctx - q_lo
    single = nq == 1
    sink = torch.zeros(H, device=device)
    gate = torch.randn(nq, H + 3, generator=g).to(dt)
    wide = torch.zeros(nq, H * V + 16, dtype=dt, device=device)
    seq.sink_attn(qr[q_lo:].contiguous(), cache, perm[None].to(torch.int32).to(device),
                  None if single else torch.tensor([0, nq], dtype=torch.int32, device=device),
                  torch.tensor([n_ctx], dtype=torch.int32, device=device), pos[q_lo:].to(device), sink, None,
                  nq, H, G, D, V, 0, scale, impl=impl, seg=chunk, gate=gate.to(device)[:, 2: 2 + H],
                  out_inv_freq=vf, gate_mult=0.8, out=wide[:, 8: 8 + H * V])
    assert float(wide[:, :8].abs().max()) == 0 and float(wide[:, 8 + H * V:].abs().max()) == 0
    out = wide[:, 8: 8 + H * V]
    q, k, v = (x.to(F64) for x in (p[:, : H * D].view(-1, H, D), p[:, H * D: (H + G) * D].view(-1, G, D), p[:, (H + G) * D:].view(-1, G, V)))
    fr, gn = orc.rotary_frequencies(rot), orc.rotary_gain(rot)
    vfr = orc.rotary_frequencies({"dims": V, "base": 100.0})
    if rotate_values:
        v = orc.rotate(v, vfr)
    want = orc.attend(orc.rotate(q, fr, gn), orc.rotate(k, fr, gn), v, scale, chunk, plus_one=True)
    if rotate_values:
        want = orc.rotate(want, vfr, sign=-1.0)
    want = want[q_lo:] * (0.8 * orc.sigmoid(gate.to(F64)[:, 2: 2 + H]))[:, :, None]
    return out.cpu().double(), want.reshape(nq, H * V)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("where", ["inside", "outside", "far", "page", "first"])
@pytest.mark.parametrize("rows", ["portion", "decode"])
def test_attention_chunk_edges_and_far_keys(device, where, rows):
    """A key made to stand out just inside / just outside the query's chunk, far back without chunks, on a page border and
    at position 0, for a prompt portion and for a decode row, over scattered pages. The key moves the last row by far more
    than the tolerance when visible, and not at all when not."""
    _need(device)
    n_ctx, chunk = 150, 40                       # the last row's chunk starts at position 120
    standout = {"inside": 120, "outside": 119, "far": 3, "page": 128, "first": 0}[where]
    if where in ("far", "first"):
        chunk = 0
    q_lo = n_ctx - 1 if rows == "decode" else n_ctx - 37
    cases = [(torch.float32, {}), (torch.bfloat16, {})]
    if device != "cpu":   # the matrix-core form on prompt rows and on a decode row, wide keys and values
        cases += [(torch.bfloat16, {"impl": 2}), (torch.bfloat16, {"D": 96, "V": 160, "R": 24}),
                  (torch.bfloat16, {"D": 256, "V": 256, "R": 32}), (torch.bfloat16, {"D": 176, "V": 64, "R": 32, "H": 6, "G": 1}),
                  (torch.bfloat16, {"D": 64, "V": 192, "R": 64 - 16, "impl": 2}), (torch.float32, {"D": 200, "V": 136, "R": 8}),
                  (torch.bfloat16, {"D": 24, "V": 20, "R": 8, "H": 5, "G": 5})]
    for dt, kw in cases:
        got, want = _attention_case(device, dt, n_ctx, q_lo, standout, chunk, **kw)
        scale = float(want.abs().max())
        tol = 2e-4 if dt == torch.float32 else 3e-2
        assert float((got - want).abs().max()) < tol * scale, (dt, kw)
        _, without = _attention_case(device, dt, n_ctx, q_lo, standout, chunk, present=False, **kw)
        moved = float((want[-1] - without[-1]).abs().max())
        if where == "outside":
            assert moved < 1e-9
        else:
            assert moved > 1.0, (where, moved)


@pytest.mark.gpu
@pytest.mark.parametrize("chunk", [31, 32, 33, 100, 128])
def test_attention_chunks_across_row_tiles(chunk):
    """Whole prompts over many chunks on the matrix cores: chunks smaller, equal and larger than a key tile, tiles whose
    rows belong to several chunks, single heads per key/value head and many; long contexts in split decode."""
    _need("cuda:0")
    for kw in (dict(), dict(H=8, G=1, D=64, V=96, R=32), dict(H=2, G=2, D=16, V=32, R=16 - 4)):
        got, want = _attention_case("cuda:0", torch.bfloat16, 333, 0, 5, chunk, impl=2, **kw)
        assert float((got - want).abs().max()) < 3e-2 * float(want.abs().max()), kw
    n = 20 * chunk + 7
    for lo in (n - 1, n - 3):
        got, want = _attention_case("cuda:0", torch.bfloat16, n, lo, 2, chunk if lo == n - 1 else 0)
        assert float((got - want).abs().max()) < 3e-2 * float(want.abs().max()), lo


# ------------------------------------------------------------------------------------------- the model in the engine
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_and_layers_match_the_oracle(tmp_path, device, name):
    _need(device)
    config = CONFIGS[name]()
    weights = weights_for(config, 1)
    toks = tokens_for(config, 90 if device != "cpu" else 50, 3)
    want, layers = orc.forward(config, weights, toks, keep_layers=True)
    eng = make_engine(tmp_path, config, weights, device, torch.float32)
    kept, fw = {}, eng.model.forward
    eng.model.forward = lambda i, p, m, k: fw(i, p, m, k, layer_hook=lambda li, x: kept.__setitem__(li, x.double().cpu().clone()))
    got = replay(eng, [[("a", toks, list(range(len(toks))), True)]])
    for li in range(len(config["layers"])):
        assert float((kept[li] - layers[li]).abs().max()) < 2e-4 * float(layers[li].abs().max()), li
    check(got["a"], want, TOL[torch.float32])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("sizes", [[1], [2, 2, 2, 2, 3, 2, 5], [16, 16, 16], [7, 4, 2, 13], [33]], ids=str)
def test_portions_match_the_oracle(tmp_path, device, name, sizes):
    """A prompt token by token, in portions down to two tokens, cut at page and chunk borders and elsewhere; the rest is
    decoded one by one."""
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
    """A prompt then 100 single-token steps in bf16 (chunk borders pass over decoded tokens, every state is carried 100
    times), and the same positions from one whole-prompt step: both hold the oracle's logits."""
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
def test_unequal_requests_share_steps_pages_and_slots_reused(tmp_path, device, dtype):
    """Six unequal requests, at most four live, in a pool too small for all of them: portions beside single tokens,
    requests sitting out steps, finished requests' pages and state slots handed to later ones. Every request's logits
    equal those of the request alone (the oracle)."""
    _need(device)
    config = CONFIGS["std"]()
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
    used_slots, used_blocks = {}, {}
    got, at = {}, {}
    for step in steps:
        entries = [(r, t, w) for r, t, w, _ in step]
        logits = eng.replay_step(entries, [])
        for r, _, _, _ in step:
            s = eng.seqs[r]
            used_slots[r] = s.state_slot
            used_blocks.setdefault(r, set()).update(s.block_table)
        k = 0
        for r, t, w, _ in step:
            for x in w:
                got.setdefault(r, {})[at.get(r, 0) + x] = logits[k]
                k += 1
            at[r] = at.get(r, 0) + len(t)
        eng.replay_step([], [r for r, _, _, e in step if e])
    assert len(set(used_slots.values())) <= 4 and len(used_slots) == 6      # slots were handed on
    assert used_blocks["e"] & (used_blocks["b"] | used_blocks["c"] | used_blocks["a"])   # and so were pages
    for r in lens:
        assert len(got[r]) == lens[r]
        check(got[r], orc.forward(config, weights, toks[r]), TOL[dtype])


def test_oracle_sensitivity():
    """What the engine is checked against moves by far more than the tolerance when a mechanism is altered: a chunk by one
    token, the position scaling, the turned values, scales, taps, decays, gates, biases, norms, the first tokens."""
    config = CONFIGS["std"]()
    weights = weights_for(config, 1)
    toks = tokens_for(config, 40, 2)
    base = orc.forward(config, weights, toks)
    floor = 30 * TOL[torch.float32]

    def moved(cfg=None, w=None, t=None):
        return float(row_errs(orc.forward(cfg or config, w or weights, t or toks), base)[-8:].max())

    def with_entry(i, path, value):
        c = copy.deepcopy(config)
        node = c["layers"][i]
        for k in path[:-1]:
            node = node[k]
        if value is None:
            node.pop(path[-1], None)
        else:
            node[path[-1]] = value
        return c

    for i, size in ((0, 6), (0, 8), (1, 10), (1, 12)):
        assert moved(with_entry(i, ["mixer", "left", "mask", "size"], size)) > floor, (i, size)
    assert moved(with_entry(0, ["mixer", "left", "rot", "scaling"], None)) > floor
    assert moved(with_entry(0, ["mixer", "left", "rot", "base"], 60.0)) > floor
    assert moved(with_entry(1, ["mixer", "left", "scale"], 0.5)) > floor
    assert moved(with_entry(1, ["mixer", "right", "tau"], 8.0)) > floor
    for i in (0, 1):
        assert moved(with_entry(i, ["mixer", "left_scale"], 0.6)) > floor
        assert moved(with_entry(i, ["mixer", "right_scale"], 0.55)) > floor
    for name in ("l0.canon1", "l1.canon2", "l0.mix.left.q.conv", "l0.mix.left.v.conv", "l0.mix.right.k.conv", "l1.mix.left.k.norm",
                 "l1.mix.right.norm", "l0.mix.right.norm"):
        w = dict(weights)
        w[name] = torch.flip(weights[name], [-1])
        assert moved(w=w) > floor, name
    for name in ("l0.mix.right.A_log", "l0.mix.right.dt_bias", "l1.mix.right.a2.b", "l1.mix.left.q.b", "l1.mix.left.v.b"):
        w = dict(weights)
        w[name] = weights[name] + torch.linspace(0.5, 1.5, weights[name].numel()).view(weights[name].shape)
        assert moved(w=w) > floor, name
    for name in ("l0.mix.left.g", "l0.mix.right.b", "l0.mix.right.g2", "l1.mix.left.g", "l1.mix.right.g"):
        w = dict(weights)
        w[name] = torch.zeros_like(weights[name])
        assert moved(w=w) > floor, name
    # the unit in the denominator and the turned values
    h = torch.randn(20, 3, 6, generator=torch.Generator().manual_seed(0)).to(F64)
    assert float((orc.attend(h, h, h, 0.4, 7, True) - orc.attend(h, h, h, 0.4, 7, False)).abs().max()) > 0.05
    vf = orc.rotary_frequencies({"dims": 6, "base": 50.0})
    turned = orc.rotate(orc.attend(h, h, orc.rotate(h, vf), 0.4, 7, True), vf, sign=-1.0)
    assert float((turned - orc.attend(h, h, h, 0.4, 7, True)).abs().max()) > 0.05
    # the first tokens reach the last rows through the recurrent states although every chunk is shorter
    assert moved(t=[(toks[0] + 1) % config["vocab"]] + toks[1:]) > floor


# ------------------------------------------------------------------------------------ generation, registry, CLI
@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_engine(tmp_path, device):
    """LLMEngine.generate (scheduler, continuous batching on three slots, sampling) continues five prompts as the
    oracle's greedy choice does; on the GPU also from captured decode graphs."""
    _need(device)
    from src.preproc import SamplingParams

    config = CONFIGS["mc" if device != "cpu" else "std"]()
    weights = weights_for(config, 7)
    prompts = [tokens_for(config, n, 20 + n) for n in (5, 1, 19, 33, 8)]
    n_new = 6

    def is_greedy(prompt, out):
        """Every generated token is the oracle's argmax given the tokens before it, or ties with it at the sampler's
        precision (the GPU sampling kernel reads the logits as bf16)."""
        seq_ = list(prompt) + list(out)
        lg = orc.forward(config, weights, seq_)
        for i, tok in enumerate(out):
            row = lg[len(prompt) + i - 1]
            slack = 1e-3 * float(row.std()) if device == "cpu" else 2.0 ** -7 * float(row.abs().max())
            if float(row[tok]) < float(row.max()) - slack:
                return False
        return len(out) == n_new

    modes = [dict(capture=False)]
    if device != "cpu":
        modes.append(dict(capture=True, use_cuda_graph=True, graph_batch_sizes=[1, 2, 4], decode_window=4))
    for i, kw in enumerate(modes):
        eng = make_engine(tmp_path, config, weights, device, torch.float32, max_seqs=3, name=f"g{i}", **kw)
        eng.eos_token_id = None
        outs = eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.0))
        assert all(is_greedy(p, o) for p, o in zip(prompts, outs)), (kw, outs)


def test_registry_config_roundtrip(tmp_path):
    from safetensors.torch import load_file

    from src.models.registry import family_of, resolve
    from src.models.rerozen import RerozenArch, RerozenLM

    config = CONFIGS["std"]()
    path = str(tmp_path / "ckpt")
    save_checkpoint(path, config, weights_for(config, rank=11, gate_rank=3))
    assert family_of(path) == "rerozen"
    _, arch, cls = resolve(path)
    assert cls is RerozenLM and arch.num_layers == len(config["layers"])
    assert arch.to_config() == json.loads(json.dumps(config))
    model = cls(arch, "cpu", dtype=torch.float32)
    assert model.needs_seq_state and not model.supports_prefix_cache
    assert [l.mixer.cache_width for l in arch.layers] == [2 * (8 + 12), 2 * (12 + 8), 1 * (14 + 6), 3 * (7 + 5)]
    assert set(arch.state_shapes(0)) == {"qkv_conv", "delta", "conv", "canon1", "canon2"}
    assert set(arch.state_shapes(1)) == {"linear", "canon1", "canon2"}
    assert set(arch.state_shapes(2)) == {"qkv_conv", "delta", "conv", "canon1"}       # no feed-forward
    n = model.load_state_dict(load_file(os.path.join(path, "model.safetensors")))
    assert n == len(orc.tensor_shapes(config))
    # loading again, in place, and with other low-rank widths
    for kw in (dict(rank=11, gate_rank=3), dict(rank=4, gate_rank=9)):
        again = weights_for(config, 3, **kw)
        assert model.load_state_dict(again) == len(again)
        model.save(str(tmp_path / "again"))
        back = load_file(str(tmp_path / "again" / "model.safetensors"))
        assert set(back) == set(again)
        for k, v in again.items():
            assert torch.equal(back[k].float(), v.float()), k
    for bad in (dict(type="lightning"), dict(mlp={"kind": "moe", "ff": 4})):
        c = copy.deepcopy(config)
        c["layers"][0].update(bad)
        with pytest.raises(ValueError):
            RerozenArch.from_config(c)


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
