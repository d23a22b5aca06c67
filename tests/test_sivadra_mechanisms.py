"""Each Sivadra mechanism alone -- norms, rotary positions, gated delta rule, latent
attention, feed-forward activation -- against its plain function, at sizes a served
model has as well as ragged ones.  CPU path and, marked gpu, the HIP kernels."""
import os
import sys
from types import SimpleNamespace

import pytest
import torch

sys.path.insert(0, os.path.dirname(__file__))
import plain_sivadra as plain  # noqa: E402
import sivadra_cases as sc  # noqa: E402

from omnia_amd.models.layers import (LatentAttentionSpec, RotarySpec, YarnSpec,  # noqa: E402
                                     _delta, _latent_attention)
from omnia_amd.models.llama import ForwardBatch  # noqa: E402
from omnia_amd.models.mixers import GatedDelta, LatentAttention, rotary_table  # noqa: E402
from omnia_amd.ops import mixers as mops  # noqa: E402

GPU = pytest.mark.gpu
RUNS = [pytest.param(("cpu", torch.float32), id="cpu"),
        pytest.param(("cuda", torch.float32), id="gpu32", marks=GPU),
        pytest.param(("cuda", torch.bfloat16), id="gpu16", marks=GPU)]
LIMIT = {torch.float32: 3e-5, torch.bfloat16: 0.02}


def rel(got, want):
    want = want.double()
    return float((got.double().cpu() - want.cpu()).norm() / want.norm().clamp(min=1e-30))


def gen(seed=0):
    return torch.Generator().manual_seed(seed)


def rnd(*shape, g, dtype=torch.float64, scale=1.0):
    return (torch.randn(*shape, generator=g, dtype=torch.float64) * scale).to(
        torch.bfloat16).to(dtype)


# ------------------------------------------------------------------- tanh norm
@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("d", [8, 48, 1000, 4096])
def test_tanh_norm_residual(d, run):
    dev, dt = run
    g = gen(d)
    M = 7
    n1 = (0.7, torch.rand(d, generator=g) + 0.5, torch.randn(d, generator=g) * 0.2)
    n2 = (1.6, torch.rand(d, generator=g) + 0.5, torch.randn(d, generator=g) * 0.2)
    bias = torch.randn(d, generator=g)
    x0 = torch.randn(M, d, generator=g) * 3
    kinds = [(dt, 1), (torch.float32, 3)] + ([(torch.float16, 5)] if dt == torch.bfloat16 else [])
    for pdt, S in kinds:
        m = rnd(S, M, d, g=g).to(pdt)
        for b in (None, bias):
            v = m.double().sum(0) + (0 if b is None else b.double())
            wx = x0.double() + plain.dyn_tanh(v, n1[1].double(), n1[2].double(), n1[0])
            wh = plain.dyn_tanh(wx, n2[1].double(), n2[2].double(), n2[0])
            x = x0.to(dev).clone()
            norms = [mops.TanhNorm(a, w.to(dev), bb.to(dev)) for a, w, bb in (n1, n2)]
            h = mops.tanh_norm_residual(x, (m if S > 1 else m[0]).to(dev), *norms, dt,
                                        None if b is None else b.to(dev))
            assert x.dtype == torch.float32 and h.dtype == dt
            assert rel(x, wx) < 1e-6 and rel(h, wh) < (1e-6 if dt == torch.float32 else 4e-3)
            if S > 1:  # the parts of a row side by side
                x = x0.to(dev).clone()
                h2 = mops.norm_residual(x, m.transpose(0, 1).contiguous().to(dev), *norms, dt,
                                        None if b is None else b.to(dev), slots=True)
                assert rel(x, wx) < 1e-6 and rel(h2, h.double()) < 4e-3


@pytest.mark.parametrize("run", RUNS)
def test_tanh_norm_embed(run):
    """Gather, fp32 residual and first norm; tokens still on the device."""
    dev, dt = run
    g = gen(3)
    table = rnd(50, 24, g=g).to(dt)
    w, b = torch.rand(24, generator=g), torch.randn(24, generator=g)
    ids = torch.tensor([3, 49, 0, 7], dtype=torch.int32)
    src = torch.tensor([-1, 2, -1, 0])
    slots = torch.tensor([11, 12, 13], dtype=torch.int32)
    x, h = mops.tanh_norm_embed(ids.to(dev), table.to(dev), 50,
                                mops.TanhNorm(0.8, w.to(dev), b.to(dev)), src.to(dev),
                                slots.to(dev))
    want = table[[3, 13, 0, 11]].float()
    assert torch.equal(x.cpu(), want)
    assert rel(h, plain.dyn_tanh(want.double(), w.double(), b.double(), 0.8)) < LIMIT[dt]


@pytest.mark.parametrize("run", RUNS)
def test_glu(run):
    dev, dt = run
    g = gen(4)
    for S, pdt in ((1, dt), (4, torch.float32)):
        m, b = rnd(S, 5, 2 * 88, g=g).to(pdt), torch.randn(2 * 88, generator=g)
        v = m.double().sum(0) + b.double()
        got = mops.glu((m if S > 1 else m[0]).to(dev), b.to(dev), dt)
        assert rel(got, plain.silu(v[:, :88]) * v[:, 88:]) < (2e-6 if dt == torch.float32 else 4e-3)


@GPU
def test_fused_gate_up_bias():
    """The prefill GEMM's biased SwiGLU epilogue."""
    from omnia_amd import ops

    g = gen(5)
    x, w = rnd(300, 256, g=g), rnd(2 * 384, 256, g=g, scale=0.1)
    b = torch.randn(2 * 384, generator=g)
    got = ops.pgemm(1, x.bfloat16().cuda(), w.bfloat16().cuda(), bias=b.cuda())
    v = x @ w.T + b.double()
    assert rel(got, plain.silu(v[:, :384]) * v[:, 384:]) < 6e-3


# ---------------------------------------------------------------------- rotary
@pytest.mark.parametrize("scaling", [None, (8.0, 4096, 32.0, 1.0), (2.5, 40, 9.0, 3.0),
                                     (4.0, 7, 30.0, 20.0)])
@pytest.mark.parametrize("dims,base", [(2, 10000.0), (12, 500.0), (64, 50000.0)])
def test_rotary_table(dims, base, scaling):
    y = None if scaling is None else YarnSpec(*scaling)
    rot = {"dims": dims, "base": base}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    cos, sin = plain.rotary_table(rot, torch.arange(3000), torch.float64)
    got = rotary_table(RotarySpec(dims, base, y), 3000, "cpu")
    assert (got.double() - torch.cat([cos, sin], 1)).abs().max() < 1e-6


# --------------------------------------------------------------- mixers, alone
class Stub(SimpleNamespace):
    """The parts of a model a mixer uses."""

    def __init__(self, dev, dt, eps, positions=4096):
        super().__init__(device=torch.device(dev), dtype=dt,
                         cfg=SimpleNamespace(rms_eps=eps, max_position=positions))

    def rotary(self, rot):
        return rotary_table(rot, self.cfg.max_position, self.device)

    def project(self, x, w, is_decode):
        return torch.nn.functional.linear(x, w)


def batch(dev, spans, bs, maxb, decode, window=0):
    """ForwardBatch of [(sequence, start, n)]; sequence s owns pages [s*maxb+1, ...) and
    state slot s + 1."""
    B = len(spans)
    pos = torch.cat([torch.arange(a, a + n) for _, a, n in spans])
    bt = torch.stack([torch.arange(maxb) + 1 + s * maxb for s, _, _ in spans])
    lens = torch.tensor([n for _, _, n in spans])
    row = torch.repeat_interleave(torch.arange(B), lens)
    slots = bt[row, pos // bs] * bs + pos % bs

    def i32(t):
        return torch.as_tensor(t).to(torch.int32).to(dev)

    fb = ForwardBatch(input_ids=None, positions=i32(pos), slots=slots.to(dev), block_tables=i32(bt),
                      seq_lens=i32([a + n for _, a, n in spans]), logits_indices=None,
                      is_decode=decode, num_seqs=B, state_slots=i32([s + 1 for s, _, _ in spans]))
    if not decode:
        from omnia_amd import ops

        fb.q_start_loc = i32(torch.cat([torch.zeros(1, dtype=torch.long), lens.cumsum(0)]))
        ts, tq = ops.prefill_tiles(lens.tolist(), 128)
        fb.tile_seq, fb.tile_q0 = i32(ts), i32(tq)
        first = [max(0, a - window + 1) if window else 0 for _, a, _ in spans]
        n = [(a + k - f + 63) // 64 * 64 for (_, a, k), f in zip(spans, first)]
        start = torch.cat([torch.zeros(1, dtype=torch.long), torch.tensor(n).cumsum(0)])
        fb.kv_start, fb.kv_first, fb.kv_rows = i32(start), i32(first), int(start[-1])
    return fb


def run_mixer(mixer, w, hs, steps, bs, maxb):
    """hs: per-sequence inputs [T, d]; steps: lists of (sequence, n); a step of single
    tokens past the start is a decode step.  Outputs per sequence (output projection's
    input)."""
    m = mixer.model
    cache = mixer.alloc(len(hs) * maxb + 1, bs, len(hs) + 1)
    at, out = [0] * len(hs), [[] for _ in hs]
    for step in steps:
        spans = [(s, at[s], n) for s, n in step]
        dec = all(n == 1 and a > 0 for _, a, n in spans)
        fb = batch(m.device, spans, bs, maxb, dec, getattr(mixer.spec, "window", 0))
        h = torch.cat([hs[s][a:a + n] for s, a, n in spans]).to(m.dtype).to(m.device)
        y, o = mixer.forward(w, h, fb, cache), 0
        for s, a, n in spans:
            out[s].append(y[o:o + n])
            at[s] += n
            o += n
    return [torch.cat(o) for o in out]


def mixer_case(kind, spec, d, run, seed=0, eps=1e-5):
    dev, dt = run
    g = gen(seed)
    parse = {"delta": _delta, "latent_attention": _latent_attention}[kind]
    from omnia_amd.models.layers import _mixer_shapes

    s = parse(spec)
    W = {}
    for n, shape in _mixer_shapes(s, d).items():
        t = rnd(*shape, g=g)
        if n.endswith("norm"):
            t = 1 + 0.2 * t
        elif n == "A_log":
            t = 0.7 * t
        elif n.endswith("conv"):
            t = t * shape[1] ** -0.5
        elif len(shape) == 2:
            t = t * 1.5 * shape[1] ** -0.5
        W[n] = t.bfloat16().double()
    cls = {"delta": GatedDelta, "latent_attention": LatentAttention}[kind]
    mixer = cls(s, Stub(dev, dt, eps))
    w = mixer.pack(lambda n: W[n].to(dt).to(dev), d)
    fn = {"delta": plain.delta_mixer, "latent_attention": plain.latent_attention}[kind]
    return mixer, w, W, (lambda h: fn(h, spec, W.__getitem__, eps))


def project_out(y, w):
    return y.double().cpu() @ w["o"].double().cpu().T


STEPS = {
    "whole": lambda n: [[(s, k)] for s, k in enumerate(n)],
    "together": lambda n: [[(s, k) for s, k in enumerate(n)]],
    "portions": lambda n: [[(s, 2) for s in range(len(n))]] + [
        [(s, min(33, k - 2)) for s, k in enumerate(n)]] + [
        [(s, k - 35) for s, k in enumerate(n) if k > 35]],
    "decode": lambda n: [[(s, 3) for s in range(len(n))]] + [
        [(s, 1) for s, k in enumerate(n) if k > t] for t in range(3, max(n))],
}

DELTAS = [dict(heads=3, kv_heads=1, dim=9, vdim=13, conv=2),
          dict(heads=2, kv_heads=2, dim=16, vdim=16, conv=1),
          dict(heads=4, kv_heads=2, dim=128, vdim=128, conv=4),
          dict(heads=2, kv_heads=1, dim=64, vdim=256, conv=3),
          dict(heads=2, kv_heads=2, dim=200, vdim=36, conv=4),
          dict(heads=1, kv_heads=1, dim=260, vdim=24, conv=6)]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("how", sorted(STEPS))
@pytest.mark.parametrize("spec", DELTAS, ids=lambda s: f"{s['dim']}x{s['vdim']}c{s['conv']}")
def test_delta_rule(spec, how, run):
    d, lens = 40, [70, 36, 41]
    mixer, w, W, want = mixer_case("delta", spec, d, run, 7)
    g = gen(8)
    hs = [rnd(n, d, g=g) for n in lens]
    steps = [s for s in STEPS[how](lens) if s]
    for h, y in zip(hs, run_mixer(mixer, w, hs, steps, 16, 8)):
        # the recurrence amplifies the bf16 rounding of its inputs
        assert rel(project_out(y, w), want(h)) < (LIMIT[run[1]] if run[1] == torch.float32
                                                  else 0.04)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("a_log,bias", [(4.0, 6.0), (-8.0, -4.0), (0.0, 0.0)])
def test_delta_rule_extreme_decay(a_log, bias, run):
    """Decays that wipe the state every token, and ones that never forget."""
    spec = dict(heads=2, kv_heads=1, dim=32, vdim=32, conv=4)
    mixer, w, W, want = mixer_case("delta", spec, 32, run, 9)
    W["A_log"].fill_(a_log)
    W["dt_bias"].fill_(bias)
    w["a_log"].fill_(a_log)
    w["dt_bias"].fill_(bias)
    h = rnd(400, 32, g=gen(10))
    y = run_mixer(mixer, w, [h], [[(0, 200)], [(0, 199)], [(0, 1)]], 64, 8)[0]
    assert torch.isfinite(y).all()
    assert rel(project_out(y, w), want(h)) < (1e-4 if run[1] == torch.float32 else 0.06)


LATENTS = [dict(heads=1, dim=11, rot=6, vdim=9, q_rank=13, kv_rank=17, window=33),
           dict(heads=5, dim=24, rot=8, vdim=40, q_rank=20, kv_rank=48, window=16),
           dict(heads=18, dim=32, rot=2, vdim=16, q_rank=40, kv_rank=96),
           dict(heads=4, dim=128, rot=64, vdim=128, q_rank=96, kv_rank=512, window=50,
                scaling=(8.0, 64, 32.0, 1.0)),
           dict(heads=20, dim=64, rot=32, vdim=64, q_rank=64, kv_rank=256, window=1),
           dict(heads=2, dim=200, rot=80, vdim=160, q_rank=32, kv_rank=560, window=64)]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("how", sorted(STEPS))
@pytest.mark.parametrize("size", LATENTS, ids=lambda s: f"h{s['heads']}c{s['kv_rank']}w{s.get('window')}")
def test_latent_attention(size, how, run):
    d, lens = 40, [150, 36, 67]
    spec = sc.latent(**size)["mixer"]
    mixer, w, W, want = mixer_case("latent_attention", spec, d, run, 11)
    g = gen(12)
    hs = [rnd(n, d, g=g) for n in lens]
    steps = [s for s in STEPS[how](lens) if s]
    for h, y in zip(hs, run_mixer(mixer, w, hs, steps, 32, 5)):
        assert rel(project_out(y, w), want(h)) < LIMIT[run[1]]


# ------------------------------------------------- one key that stands out
def attended(q, c, kr, W_uk, W_uv, spec, gate, visible):
    """Plain attention of one query over the keys `visible`."""
    H, D, R = spec.heads, spec.dim, spec.rot_dim
    out = []
    for h in range(H):
        k = c[visible] @ W_uk[h].T
        s = (q[h, :D] @ k.T + q[h, D:] @ kr[visible].T) * spec.scale
        p = torch.softmax(s, -1)
        out.append((p @ (c[visible] @ W_uv[h].T)) * torch.sigmoid(gate[h]))
    return torch.stack(out)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("mode", ["prefill", "decode"])
@pytest.mark.parametrize("page", [16, 32, 64])
def test_spiked_key_at_window_and_page_edges(mode, page, run):
    """One cached key whose score dominates, placed just inside and just outside the
    window, at page borders, far away and at position 0: seen exactly when it should."""
    dev, dt = run
    W0, n = 70, 300
    spec = LatentAttentionSpec(heads=3, dim=16, rot_dim=4, vdim=16, q_rank=8, kv_rank=32,
                               scale=0.25, rotary=RotarySpec(4, 1000.0), window=W0)
    m = LatentAttention(spec, Stub(dev, dt, 1e-5))
    g = gen(13)
    uk, uv = rnd(3, 16, 32, g=g, scale=0.3), rnd(3, 16, 32, g=g, scale=0.3)
    W = {"uk": uk.reshape(48, 32), "uv": uv.reshape(48, 32), "uq": rnd(60, 8, g=g),
         "dq": rnd(8, 24, g=g), "dkv": rnd(36, 24, g=g), "g": rnd(3, 24, g=g),
         "dq.norm": torch.ones(8), "kv_norm": None, "dkv.norm": torch.ones(32),
         "o": rnd(24, 48, g=g)}
    w = m.pack(lambda k: W[k].to(dt).to(dev), 24)
    c0, kr0 = rnd(n, 32, g=g, scale=0.5), rnd(n, 4, g=g, scale=0.5)
    gate = rnd(1, 3, g=g)
    maxb = -(-n // page)
    for pos in (n - 1, 255, 256, 69, 70, 71):
        lo = pos - W0 + 1
        marks = {lo, lo - 1, lo + 1, pos, pos - 1, 0, (lo // page) * page,
                 (lo // page) * page - 1, (pos // page) * page, (pos // page) * page - 1}
        for j in sorted(x for x in marks if 0 <= x <= pos):
            q = rnd(3, 20, g=gen(100 + j))
            c = c0.clone()
            # aligned with every head's absorbed query: the score stands far out
            a = torch.stack([uk[h].T @ q[h, :16] for h in range(3)])
            t = torch.linalg.lstsq(a, torch.full((3, 1), 60.0, dtype=torch.float64)).solution
            c[j] = t[:, 0].bfloat16().double()
            pages = torch.zeros(maxb + 1, page, spec.padded_cache_width, dtype=dt)
            flat = pages[1:].view(-1, spec.padded_cache_width)
            flat[:n, :32] = c.to(dt)
            flat[:n, spec.latent_pad:spec.latent_pad + 4] = kr0.to(dt)
            pages = pages.to(dev)
            qp = torch.zeros(1, 3, spec.qk_pad, dtype=dt)
            # the kernels rotate q: hand them the vector turned back
            cs = rotary_table(spec.rotary, n, "cpu")[pos].double()
            u, v = q[:, 16:18], q[:, 18:20]
            back = torch.cat([u * cs[:2] + v * cs[2:], v * cs[:2] - u * cs[2:]], 1)
            qp[0, :, :16], qp[0, :, 16:20] = q[:, :16].to(dt), back.to(dt)
            qp = qp.view(1, -1).to(dev)
            fb = batch(dev, [(0, pos, 1)], page, maxb, mode == "decode", W0)
            gt = gate.to(dt).to(dev)
            if mode == "decode":
                y = m._decode(w, qp, gt, pages, fb.block_tables, fb.positions, None)
            else:
                y = m._prefill(w, qp, gt, pages, fb, fb.positions, None)
            y = y.view(3, spec.v_pad)[:, :16]
            vis = torch.arange(max(0, lo), pos + 1)
            want = attended(q, c, kr0, uk, uv, spec, gate[0], vis)
            assert rel(y, want) < (1e-4 if dt == torch.float32 else 0.03), (pos, j)
            alone = (uv @ c[j]) * torch.sigmoid(gate[0])[:, None]
            if j >= lo:
                assert rel(want, alone) < 0.05  # the case really is one key against the rest
            else:
                assert rel(want, alone) > 0.5


@GPU
@pytest.mark.parametrize("splits", [1, 2, 5, 32])
def test_decode_splits_agree(splits):
    """Rows of very different lengths, their keys in any number of parts."""
    spec = LatentAttentionSpec(heads=20, dim=64, rot_dim=32, vdim=64, q_rank=64, kv_rank=480,
                               scale=0.1, rotary=RotarySpec(32, 1e4), window=700)
    g = gen(14)
    pos = [0, 1, 63, 64, 65, 699, 700, 701, 1500, 2047]
    pages = rnd(64, 32, spec.padded_cache_width, g=g).bfloat16().cuda()
    bt = torch.stack([torch.randperm(64, generator=g) for _ in pos]).to(torch.int32).cuda()
    q = rnd(len(pos), 20 * spec.padded_cache_width, g=g, scale=0.5).bfloat16().cuda()
    p = torch.tensor(pos, dtype=torch.int32).cuda()
    got = mops.latent_decode(q, pages, bt, p, spec, splits)
    ref = mops.latent_attend(q.float(), pages.float(), bt, None, p, spec)
    assert rel(got, ref.cpu()) < 0.01
