"""Each Bisuzen mechanism alone -- pre-norms around a plain residual, joined branches,
neighbour rotation and biases, windows with kept first tokens, chunks, unit queries and keys,
fixed-decay linear attention, gelu feed-forwards, grouped routing with identity experts --
against its plain function, at sizes a served model has as well as ragged ones.  CPU path and,
marked gpu, the HIP kernels."""
import math
import os
import sys

import pytest
import torch
import torch.nn.functional as F

sys.path.insert(0, os.path.dirname(__file__))
import plain_bisuzen as plain  # noqa: E402
from test_sekazen_mechanisms import Paged, gen, rel, rnd  # noqa: E402
from test_sivadra_mechanisms import Stub, batch  # noqa: E402

from omnia_amd.models.feedforward import DenseGLU, Experts  # noqa: E402
from omnia_amd.models.layers import (DESIGNS, AttentionSpec, DenseMLPSpec,  # noqa: E402
                                     ExpertsSpec, LightningSpec, RotarySpec, parse_layers)
from omnia_amd.models.mixers import GroupedQueryAttention, Lightning  # noqa: E402
from omnia_amd.ops import mixers as mops  # noqa: E402

GPU = pytest.mark.gpu
RUNS = [pytest.param(("cpu", torch.float32), id="cpu"),
        pytest.param(("cuda", torch.float32), id="gpu32", marks=GPU),
        pytest.param(("cuda", torch.bfloat16), id="gpu16", marks=GPU)]
LIMIT = {torch.float32: 3e-5, torch.bfloat16: 0.012}


def pad(t, d):
    return F.pad(t, (0, d - t.shape[-1]))


# ------------------------------------------------------------- around a sublayer
def tanh_params(n, d, g, dev):
    a, w, b = 0.8, 1.0 + 0.3 * rnd(n, g=g), 0.2 * rnd(n, g=g)
    return (a, w, b), mops.TanhNorm(a, pad(w, d).float().to(dev), pad(b, d).float().to(dev))


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("n,d", [(5, 8), (72, 72), (1000, 1024), (4096, 4096)])
def test_pre_norm_residual(n, d, run):
    """The sublayer's output joins the residual as it is; the next norm reads the sum."""
    dev, dt = run
    g = gen(n)
    M = 5
    p, norm = tanh_params(n, d, g, dev)
    x0, bias = rnd(M, n, g=g, scale=2.0), rnd(n, g=g)
    kinds = [(dt, 1, False), (torch.float32, 3, False), (dt, 4, True)]
    if dt == torch.bfloat16:
        kinds.append((torch.float16, 5, False))
    for pdt, S, slots in kinds:
        parts = rnd(S, M, n, g=g)
        m = pad(parts.transpose(0, 1) if slots else parts, d)
        m = (m[0] if S == 1 else m).contiguous().to(dev, pdt)
        for b in (None, bias):
            want = x0 + parts.sum(0) + (0 if b is None else b)
            x = pad(x0, d).float().to(dev)
            h = mops.norm_residual(x, m, None, norm, dt,
                                   None if b is None else pad(b, d).float().to(dev), slots)
            assert rel(x[:, :n], want) < 1e-6 and float(x[:, n:].abs().sum()) == 0
            assert rel(h[:, :n], plain.tanh_norm(want, *p)) < (2e-6 if dt == torch.float32
                                                               else 4e-3)


@pytest.mark.parametrize("run", RUNS)
def test_identity_parts(run):
    """Slots of identity experts hold garbage: their weight times the input stands there."""
    dev, dt = run
    g = gen(2)
    M, S, n, first = 6, 3, 48, 4
    p, norm = tanh_params(n, n, g, dev)
    x0, hin, parts = rnd(M, n, g=g), rnd(M, n, g=g), rnd(M, S, n, g=g)
    ids = torch.tensor([[0, 3, 1], [4, 5, 6], [6, 0, 2], [3, 4, 3], [1, 2, 5], [7, 4, 5]])
    wts = torch.rand(M, S, generator=g)
    idn = ids >= first
    want = x0 + torch.where(idn[..., None], wts.double()[..., None] * hin[:, None], parts).sum(1)
    m = parts.masked_fill(idn[..., None], float("nan")).to(dev, dt).contiguous()
    x = x0.float().to(dev)
    h = mops.norm_residual(x, m, None, norm, dt, None, True,
                           (ids.int().to(dev), wts.to(dev), hin.to(dev, dt), first))
    assert rel(x, want) < 1e-6
    assert rel(h, plain.tanh_norm(want, *p)) < (2e-6 if dt == torch.float32 else 4e-3)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("M,n,d", [(1, 5, 8), (7, 72, 128), (600, 1000, 1024), (3, 2048, 2048),
                                   (520, 2000, 2048), (520, 3000, 3008), (4, 4096, 4096),
                                   (513, 5000, 5056), (2, 9000, 9024)])
def test_joined_branches(M, n, d, run):
    """Two outputs, each with its own statistic, weight, bias and storage; every next norm."""
    dev, dt = run
    g = gen(n)
    eps = 3e-3
    p, tanh = tanh_params(n, d, g, dev)
    x0 = rnd(M, n, g=g, scale=2.0)
    wa, wb, wn, bias = (rnd(n, g=g) for _ in range(4))

    def norm(w):
        return mops.RMSNorm(pad(w, d).float().to(dev), n, eps)

    half = torch.float16 if dt == torch.bfloat16 else torch.float32
    for Sa, ta, Sb, tb in ((1, dt, 1, dt), (3, torch.float32, 6, half), (1, dt, 2, half)):
        a = rnd(Sa, M, n, g=g, scale=0.05)  # small: eps inside the root matters
        b = rnd(Sb, M, n, g=g, scale=3.0)
        am = pad(a if Sa > 1 else a[0], d).to(dev, ta).contiguous()
        bm = pad(b if Sb > 1 else b[0], d).to(dev, tb).contiguous()
        want = x0 + plain.branches(a.sum(0) + bias, b.sum(0), wa, wb, eps)
        for pre, wh in ((tanh, plain.tanh_norm(want, *p)), (None, want),
                        (norm(wn), plain.rms(want, eps) * wn)):
            x = pad(x0, d).float().to(dev)
            h = mops.norm_residual(x, pre=pre, dtype=dt, branches=[
                (am, pad(bias, d).float().to(dev), norm(0.5 * wa)), (bm, None, norm(0.5 * wb))])
            assert rel(x[:, :n], want) < 2e-6
            assert rel(h[:, :n], wh) < (2e-6 if dt == torch.float32 else 4e-3)
            assert float(x[:, n:].abs().sum()) == 0


def test_residual_kinds_that_do_not_exist():
    w = mops.RMSNorm(torch.ones(8), 8, 1e-5)
    x = torch.zeros(1, 8)
    with pytest.raises(ValueError, match="post-norm"):
        mops.norm_residual(x, x, None, w, torch.float32)
    with pytest.raises(ValueError, match="own norms"):
        mops.norm_residual(x, post=w, pre=w, dtype=torch.float32, branches=[(x, None, w)] * 2)


# ------------------------------------------------------- queries, keys, values
@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("shape", [(8, 2, 128, 128, 64), (3, 1, 22, 13, 6), (4, 4, 64, 32, 64),
                                   (6, 2, 96, 192, 2), (2, 2, 300, 264, 300), (5, 5, 40, 24, 20)])
@pytest.mark.parametrize("kind", ["rotated", "unit", "plain"])
def test_projection_to_queries_and_pages(kind, shape, run):
    """Bias, neighbour rotation and no norm; unit norm and no rotation; nothing at all.  From
    rows, slabs, and columns of a wider projection."""
    dev, dt = run
    g = gen(3)
    H, G, D, V, R = shape
    rot = {"dims": R, "base": 500.0}
    spec = AttentionSpec(H, G, D, V, 1.0, RotarySpec(R, 500.0, interleaved=True)
                         if kind == "rotated" else None, sink=None,
                         qk_norm="unit" if kind == "unit" else None,
                         bias="qkvo" if kind == "rotated" else "")
    eps, d, T, page = 1e-2, 40, 21, 16
    mod = GroupedQueryAttention(spec, Stub(dev, dt, eps))
    W = {"q": rnd(H * D, d, g=g), "k": rnd(G * D, d, g=g), "v": rnd(G * V, d, g=g),
         "o": rnd(d, H * V, g=g)}
    for n in "qkvo":
        W[n + ".b"] = rnd(W[n].shape[0], g=g) * (kind == "rotated")
    w = mod.pack(lambda k: W[k].to(dev, dt), d)
    assert ("in_b" in w) == (kind == "rotated") and ("q_norm" in w) == (kind == "unit")
    h = rnd(T, d, g=g)
    at = 1000  # a position whose angles are far apart
    pos = torch.arange(at, at + T, dtype=torch.int32, device=dev)
    slots = torch.arange(T, device=dev) + 3 * page
    slots[4] = -1  # a padded row writes nothing

    def heads(n, count, width, turn):
        z = (h @ W[n].T + W[n + ".b"]).view(T, count, width)
        if not turn or kind == "plain":
            return z
        if kind == "unit":
            return plain.rms(z, eps)
        return plain.rotate(torch.cat([z.new_zeros(at, count, width), z]), rot)[at:]

    q, k, v = heads("q", H, D, True), heads("k", G, D, True), heads("v", G, V, False)
    xr = F.linear(h.to(dev, dt).float(), w["in"].float())
    wide = torch.cat([xr.new_full((T, 16), 7.0), xr, xr.new_full((T, 8), 7.0)], 1)
    inputs = [xr.to(dt), wide.to(dt)[:, 16:16 + xr.shape[1]]]
    if dt == torch.bfloat16 or dev == "cpu":
        cuts = torch.rand(3, 1, 1, generator=g).to(dev)
        s = xr * cuts / cuts.sum()
        inputs += [s.contiguous(), F.pad(s, (8, 24)).contiguous()[..., 8:8 + xr.shape[1]]]
    for x in inputs:
        pages, _ = mod.alloc(6, page, 1)
        got = mops.gqa_prep(x, w, spec, pages, pos, slots, mod.table, dt, eps).view(T, H, -1)
        assert rel(got[..., :D], q) < LIMIT[dt]
        assert float(got[..., D:].float().abs().sum()) == 0
        kc = pages[0].cpu().double()[3:5].transpose(1, 2).reshape(2 * page, G, -1)[:T]
        vc = pages[1].cpu().double()[3:5].transpose(1, 2).reshape(2 * page, G, -1)[:T]
        keep = [t for t in range(T) if t != 4]
        assert rel(kc[keep][..., :D], k[keep]) < LIMIT[dt]
        assert rel(vc[keep][..., :V], v[keep]) < LIMIT[dt]
        assert float(kc[4].abs().sum() + vc[4].abs().sum()) == 0


# ------------------------------------------------------------------ attention
MASKS = [("window", 1, 0), ("window", 1, 1), ("window", 33, 4), ("window", 64, 64),
         ("window", 20, 100), ("window", 100, 17), ("window", 65, 130), ("window", 40, 1000),
         ("chunk", 1, 0), ("chunk", 17, 0), ("chunk", 32, 0), ("chunk", 64, 0), ("chunk", 100, 0),
         ("chunk", 129, 0), ("chunk", 1000, 0)]


def masked(kind, size, keep, n):
    return plain.sees_chunk(n, size) if kind == "chunk" else plain.sees_window(n, size, keep)


def attn_spec(kind, size, keep, shape, scale=None, sink=True):
    H, G, D, V = shape
    mask = {"chunk": size} if kind == "chunk" else {"window": size, "keep_first": keep}
    return AttentionSpec(H, G, D, V, scale or 1.5 * D ** -0.5, None,
                         sink="learned" if sink else None, qk_norm=None, **mask)


def attended(q, k, v, seen, scale, sinks):
    """Queries of the last positions of k, v."""
    T, n, H, G = q.shape[0], k.shape[0], q.shape[1], k.shape[1]
    out = []
    for h in range(H):
        s = (q[:, h] @ k[:, h // (H // G)].T * scale).masked_fill(~seen[n - T:], float("-inf"))
        out.append(plain.softmax(s, None if sinks is None else sinks[h]) @ v[:, h // (H // G)])
    return torch.stack(out, 1)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("kind,size,keep", MASKS)
@pytest.mark.parametrize("shape,page", [((8, 2, 64, 64), 16), ((3, 1, 22, 13), 64),
                                        ((4, 4, 128, 96), 32), ((2, 1, 280, 40), 16)])
def test_masked_attention(shape, page, kind, size, keep, run):
    """Unequal portions over shuffled pages that hold leftovers; the same rows decoded, in any
    number of parts."""
    g = gen(4)
    spec = attn_spec(kind, size, keep, shape, sink=kind == "window")
    P = Paged(run, spec, g, page=page)
    sinks = rnd(spec.heads, g=g, scale=2.0) if spec.sink else None
    sdev = None if sinks is None else sinks.float().to(P.dev)
    lens, nq = [1, 17, 150, 300, 64, 129, 131], [1, 2, 131, 45, 64, 129, 3]
    ks = [rnd(n, spec.kv_heads, spec.dim, g=g) for n in lens]
    vs = [rnd(n, spec.kv_heads, spec.vdim, g=g) for n in lens]
    qs = [rnd(m, spec.heads, spec.dim, g=g) for m in nq]
    bts = [P.put(k, v) for k, v in zip(ks, vs)]
    want = [attended(q, k, v, masked(kind, size, keep, n), spec.scale, sinks)
            for q, k, v, n in zip(qs, ks, vs, lens)]
    got, o = P.prefill(qs, bts, lens, sdev), 0
    for i, w in enumerate(want):
        assert rel(got[o:o + nq[i]], w) < LIMIT[P.dt], (i, lens[i])
        o += nq[i]
    last = torch.stack([q[-1] for q in qs])
    for splits in (None, 1, 2, 5):
        got = P.decode(last, bts, lens, sdev, splits)
        for i in range(len(lens)):
            assert rel(got[i], want[i][-1]) < LIMIT[P.dt], (splits, lens[i])


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("kind,size,keep", [
    ("window", 16, 4), ("window", 33, 16), ("window", 40, 17), ("window", 64, 1),
    ("window", 31, 70), ("chunk", 16, 0), ("chunk", 33, 0), ("chunk", 64, 0)])
def test_one_key_that_stands_out(kind, size, keep, run):
    """One key far above all others, around the kept first ones, at page borders, in every
    chunk's ends and around the window's: seen, the output is its value; else nothing of it
    is left."""
    g = gen(5)
    H, G, D, V, n = 2, 1, 32, 32, 140
    spec = attn_spec(kind, size, keep, (H, G, D, V), 1.0)
    P = Paged(run, spec, g, page=16, blocks=600)
    seen = masked(kind, size, keep, n)
    ends = {c * size + e for c in range(n // size + 1) for e in (-1, 0)} if kind == "chunk" \
        else {n - 1 - size + e for e in (-1, 0, 1, 2)}
    spots = sorted(x for x in ends | {0, 1, keep - 1, keep, keep + 1, 15, 16, 63, 64, 128, n - 1}
                   if 0 <= x < n)
    sinks = torch.zeros(H, dtype=torch.float64)
    sdev = sinks.float().to(P.dev)
    lim = 1e-4 if P.dt == torch.float32 else 0.06
    for spot in spots:
        k, v = rnd(n, G, D, g=g, scale=0.01), rnd(n, G, V, g=g)
        q = torch.zeros(n, H, D, dtype=torch.float64)
        q[..., 3] = 8.0
        k[spot, :, 3] = 8.0  # its score is 64
        v[spot] += 5.0
        bt = P.put(k, v)
        want = attended(q, k, v, seen, 1.0, sinks)
        got = P.prefill([q], [bt], [n], sdev)
        part = P.prefill([q[77:]], [bt], [n], sdev)  # the same rows from a later portion
        for i in range(n):
            assert float((got[i] - want[i]).abs().max()) < lim, (spot, i)
            if i >= 77:
                assert float((part[i - 77] - want[i]).abs().max()) < lim, (spot, i)
            if seen[i, spot]:
                assert float((want[i] - v[spot]).abs().max()) < 1e-6
        edge = {n, spot + 1, spot + size, spot + size + 1, (spot // size + 1) * size,
                (spot // size + 1) * size + 1}
        for m in sorted(x for x in edge if 1 <= x <= n):
            for splits in (1, 3):
                d = P.decode(q[m - 1:m], [bt], [m], sdev, splits)
                assert float((d[0] - want[m - 1]).abs().max()) < lim, (spot, m, splits)
        P.free = bt + P.free


@GPU
@pytest.mark.parametrize("page", [8, 64])
@pytest.mark.parametrize("kind,size,keep", [("window", 700, 300), ("window", 1500, 5000),
                                            ("chunk", 1100, 0)])
def test_long_contexts(kind, size, keep, page):
    """Thousands of keys: parts longer than one score tile, kept keys of many pages."""
    g = gen(7)
    spec = attn_spec(kind, size, keep, (8, 2, 64, 64), 0.2)
    P = Paged(("cuda", torch.bfloat16), spec, g, page=page, blocks=6000 // page * 2)
    lens = [5000, 1101, 3]
    ks, vs = [rnd(n, 2, 64, g=g) for n in lens], [rnd(n, 2, 64, g=g) for n in lens]
    qs = [rnd(min(n, 200), 8, 64, g=g) for n in lens]
    bts = [P.put(k, v) for k, v in zip(ks, vs)]
    sinks = rnd(8, g=g)
    sdev = sinks.float().cuda()
    want = [attended(q, k, v, masked(kind, size, keep, n), 0.2, sinks)
            for q, k, v, n in zip(qs, ks, vs, lens)]
    assert rel(P.prefill(qs, bts, lens, sdev), torch.cat(want)) < 0.012
    for splits in (None, 1, 7):
        d = P.decode(torch.stack([q[-1] for q in qs]), bts, lens, sdev, splits)
        for i in range(3):
            assert rel(d[i], want[i][-1]) < 0.012, (splits, i)


# ------------------------------------------------ fixed-decay linear attention
def lightning_case(dim, vdim, decay, d, run, seed=0, eps=1e-4):
    dev, dt = run
    g = gen(seed)
    spec = LightningSpec(len(decay), dim, vdim, tuple(decay))
    mod = Lightning(spec, Stub(dev, dt, eps))
    mod.model._slabs = lambda tag, x, w, dec: F.linear(x, w)
    H = len(decay)
    W = {n: rnd(H * (vdim if n in "vg" else dim), d, g=g, scale=1.5 * d ** -0.5) for n in "qkvg"}
    W["norm"], W["o"] = 1.0 + 0.2 * rnd(H * vdim, g=g), rnd(d, H * vdim, g=g)
    w = mod.pack(lambda n: W[n].to(dev, dt), d)
    m = {"heads": H, "dim": dim, "vdim": vdim, "decay": list(decay)}
    return mod, w, lambda h: plain.lightning(h, m, W.__getitem__, eps)


def run_lightning(mod, w, hs, steps):
    """hs: per-sequence inputs; steps: lists of (sequence, n).  Single tokens past the start
    that come first in a step are decode rows, as in the engine's mixed steps."""
    m = mod.model
    cache = mod.alloc(1, 16, len(hs) + 2)
    cache[1][0].fill_(1e3)  # what other sequences left
    at, out = [0] * len(hs), [[] for _ in hs]
    for step in steps:
        spans = [(s, at[s], n) for s, n in step]
        nd = 0
        while nd < len(spans) and spans[nd][2] == 1 and spans[nd][1] > 0:
            nd += 1
        fb = batch(m.device, spans, 16, 40, nd == len(spans))
        if nd < len(spans):
            rest = batch(m.device, spans[nd:], 16, 40, False)
            fb.q_start_loc, fb.num_decode = rest.q_start_loc, nd
        h = torch.cat([hs[s][a:a + n] for s, a, n in spans]).to(m.dtype).to(m.device)
        y, o = mod.forward(w, h, fb, cache), 0
        for s, a, n in spans:
            out[s].append(y[o:o + n])
            at[s] += n
            o += n
    assert float(cache[1][0][0].min()) == 1e3  # nobody's slot is left alone
    return [(torch.cat(o).double().cpu() @ w["o"].double().cpu().T) for o in out]


LIGHTNINGS = [(9, 13, (0.9, 0.5)), (16, 16, (0.999,)), (128, 128, (0.6, 0.99, 0.9999)),
              (64, 200, (0.9, 0.995)), (200, 36, (0.95, 0.7)), (264, 24, (0.9,)),
              (24, 300, (0.97,)), (8, 1040, (0.9,))]
LSTEPS = {
    "whole": lambda n: [[(s, k)] for s, k in enumerate(n)],
    "together": lambda n: [list(enumerate(n))],
    "portions": lambda n: [[(s, 2) for s in range(len(n))], [(s, 33) for s in range(len(n))],
                           [(s, k - 35) for s, k in enumerate(n)]],
    "decode": lambda n: [[(s, 3) for s in range(len(n))]] + [
        [(s, 1) for s, k in enumerate(n) if k > t] for t in range(3, max(n))],
    "mixed": lambda n: [[(0, n[0] - 2)], [(0, 1), (1, 17)], [(0, 1), (2, n[2])],
                        [(1, 1), (3, 40)], [(3, n[3] - 40), (1, n[1] - 18)]],
}


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("how", sorted(LSTEPS))
@pytest.mark.parametrize("dim,vdim,decay", LIGHTNINGS, ids=lambda x: str(x))
def test_linear_attention(dim, vdim, decay, how, run):
    d, lens = 40, [70, 36, 41, 48]
    mod, w, want = lightning_case(dim, vdim, decay, d, run, 7)
    g = gen(8)
    hs = [rnd(n, d, g=g) for n in lens]
    for h, y in zip(hs, run_lightning(mod, w, hs, LSTEPS[how](lens))):
        assert rel(y, want(h)) < LIMIT[run[1]]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("decay", [(0.0, 1.0), (1.0, 1e-3), (0.9999, 0.3)])
def test_extreme_decays(decay, run):
    """Decays that keep one token, and ones that never forget."""
    mod, w, want = lightning_case(32, 24, decay, 32, run, 9)
    h = rnd(300, 32, g=gen(10))
    y = run_lightning(mod, w, [h], [[(0, 150)], [(0, 149)], [(0, 1)]])[0]
    assert torch.isfinite(y).all() and rel(y, want(h)) < 2 * LIMIT[run[1]]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("gap", [1, 15, 16, 17, 31, 32, 33, 127, 128, 129, 256, 400])
def test_one_token_remembered(gap, run):
    """A state holds one strong key and value, read back ``gap`` tokens later: exactly
    decay^gap of it is left, whatever blocks and segments lie between."""
    dev, dt = run
    D = V = 16
    n, at, lam = 420, 11, 0.99
    spec = LightningSpec(1, D, V, (lam,))
    x = torch.full((n, spec.in_cols), -60.0)  # silu: nothing
    x[at, D + 3] = 20.0  # key 3
    x[at, 2 * D:2 * D + V] = torch.arange(1.0, V + 1)
    x[at + gap, 3] = 10.0  # query 3
    x[:, 2 * D + V:] = 100.0  # open gate
    w = {"norm": torch.ones(V, device=dev), "pow": mops.decay_powers((lam,), dev)}
    for cut in ((n,), (at + 1, n - at - 1), (200, 100, 120)):
        state = torch.full((2, 1, D, V), 9.0, device=dev)
        o, p = [], 0
        for m in cut:
            pos = torch.arange(p, p + m, dtype=torch.int32, device=dev)
            o.append(mops.lightning(x[p:p + m].to(dev, dt), w, spec, state,
                                    torch.tensor([0, m], dtype=torch.int32, device=dev), pos,
                                    torch.tensor([1], dtype=torch.int32, device=dev), 1e6, dt))
            p += m
        o = torch.cat(o).double().cpu() * 1e3  # eps swamps the norm: y = o / 1000
        v = torch.arange(1.0, V + 1).double()
        want = plain.silu(v) * 200.0 * lam ** gap
        lim = 1e-4 if dt == torch.float32 else 6e-3
        # the norm's own mean square is a small part of eps
        scale = math.sqrt(1e6 / (float((want ** 2).mean()) + 1e6))
        assert rel(o[at + gap], want * scale) < lim, cut
        rest = o.clone()
        rest[at + gap] = 0
        assert float(rest.abs().max()) < 1e-3 * float(want.max())
        left = float(state[1, 0, 3, 4])
        assert left == pytest.approx(float(plain.silu(v)[4]) * 20.0 * lam ** (n - 1 - at), rel=1e-3)


@GPU
@pytest.mark.parametrize("run", RUNS[1:])
@pytest.mark.parametrize("lens", [(3000,), (1500, 100, 129, 2, 700), (128, 128, 129, 1)])
def test_long_scans(lens, run):
    """Portions of many segments beside short ones, fresh and continued; padded rows."""
    dev, dt = run
    H, D, V = 3, 64, 72
    spec = LightningSpec(H, D, V, (0.7, 0.99, 0.9995))
    g = gen(11)
    x = rnd(sum(lens), spec.in_cols, g=g)
    w = {"norm": torch.ones(H * V, device=dev), "pow": mops.decay_powers(spec.decay, dev)}
    state = rnd(len(lens) + 1, H, D, V, g=g).float()
    start = [0 if i % 2 == 0 else 50 for i in range(len(lens))]
    slots = [i + 1 for i in range(len(lens))]
    if len(lens) == 4:
        slots[2] = -1

    def i32(v):
        return torch.tensor(v, dtype=torch.int32, device=dev)

    qs = [0]
    for n in lens:
        qs.append(qs[-1] + n)
    got_state = state.to(dev)
    pos = [p for s, n in zip(start, lens) for p in range(s, s + n)]
    y = mops.lightning(x.to(dev, dt), w, spec, got_state, i32(qs), i32(pos), i32(slots), 1e-5, dt)
    for i, n in enumerate(lens):
        if slots[i] < 0:
            continue
        xs = x[qs[i]:qs[i + 1]]
        q, k, v, gate = xs.split([H * D, H * D, H * V, H * V], 1)
        # activations may be 16-bit; the state and what it meets are not: it is as exact
        q, k, v = (plain.silu(z).to(dt).double().view(n, H, -1) for z in (q, k, v))
        o, S = plain.recurrence(q, k, v, spec.decay,
                                state[slots[i]].double() if start[i] else None)
        want = plain.gated_out(o.reshape(n, -1), gate, 1.0, 1e-5)
        assert rel(y[qs[i]:qs[i + 1]], want) < (1e-5 if dt == torch.float32 else 4e-3)
        assert rel(got_state[slots[i]], S) < (1e-5 if dt == torch.float32 else 1e-4)
    assert torch.equal(got_state[0].cpu(), state[0])


@GPU
def test_decode_reads_slabs():
    """A decode step's split-K slabs, columns of a wider projection."""
    H, D, V, T, S = 2, 128, 64, 5, 4
    spec = LightningSpec(H, D, V, (0.9, 0.99))
    g = gen(12)
    x = rnd(S, T, spec.in_cols, g=g)
    w = {"norm": torch.ones(H * V, device="cuda"), "pow": mops.decay_powers(spec.decay, "cuda")}
    state = rnd(T + 1, H, D, V, g=g).float()
    pos = torch.tensor([0, 5, 9, 1, 70], dtype=torch.int32, device="cuda")
    slots = torch.tensor([3, 1, -1, 5, 2], dtype=torch.int32, device="cuda")
    for pdt in (torch.float32, torch.float16):
        st = state.cuda()
        y = mops.lightning(F.pad(x, (8, 16)).to("cuda", pdt)[..., 8:8 + spec.in_cols], w, spec, st,
                           None, pos, slots, 1e-5, torch.bfloat16)
        for t in range(T):
            if slots[t] < 0:
                assert float(y[t].float().abs().sum()) == 0
                continue
            xs = x.to(pdt).double().sum(0)[t:t + 1]
            q, k, v, gate = xs.split([H * D, H * D, H * V, H * V], 1)
            o, Sn = plain.recurrence(plain.silu(q).view(1, H, D), plain.silu(k).view(1, H, D),
                                     plain.silu(v).view(1, H, V), spec.decay,
                                     state[slots[t]].double() if pos[t] else None)
            assert rel(y[t:t + 1], plain.gated_out(o.reshape(1, -1), gate, 1.0, 1e-5)) < 4e-3
            assert rel(st[slots[t]], Sn) < 1e-6
        assert torch.equal(st[0].cpu(), state[0]) and torch.equal(st[4].cpu(), state[4])


# -------------------------------------------------------------- feed-forwards
@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("d,ff,T", [(40, 56, 9), (45, 35, 3), (128, 256, 70)])
def test_dense_gelu(d, ff, T, run):
    dev, dt = run
    g = gen(ff)
    W = {"gate": rnd(ff, d, g=g, scale=2 * d ** -0.5), "up": rnd(ff, d, g=g, scale=d ** -0.5),
         "down": rnd(d, ff, g=g, scale=ff ** -0.5)}
    model = Stub(dev, dt, 1e-5)
    model._pgemm_ok = lambda *a: False
    model._wcfg = lambda *a: None
    model._slabs = lambda tag, x, w, dec: F.linear(x, w)
    mod = DenseGLU(DenseMLPSpec(ff, "gelu_tanh", False), model)
    dp = -(-d // 8) * 8
    w = mod.pack(lambda n: W[n].to(dev, dt), dp)
    h = rnd(T, d, g=g, scale=2.0)
    out = mod.forward(w, pad(h, dp).to(dev, dt), False)
    assert out["bias"] is None
    assert rel(out["m"][:, :d], plain.dense(h, W.__getitem__)) < LIMIT[dt]


@pytest.mark.parametrize("run", RUNS)
def test_gelu_glu_over_its_range(run):
    dev, dt = run
    g = gen(4)
    z = torch.linspace(-12, 12, 88, dtype=torch.float64).to(torch.bfloat16).double()
    u = rnd(3, 88, g=g)
    m = torch.cat([z.expand(3, 88), u], 1).to(dt)
    got = mops.glu(m.to(dev), None, dt, "gelu_tanh")
    assert rel(got, plain.gelu_tanh(z) * u) < (1e-6 if dt == torch.float32 else 3e-3)
    if dt == torch.float32:
        parts = torch.stack([0.25 * m, 0.75 * m])
        b = torch.randn(176, generator=g)
        want = plain.gelu_tanh(z + b[:88]) * (u + b[88:])
        assert rel(mops.glu(parts.to(dev), b.to(dev), dt, "gelu_tanh"), want) < 1e-6


@pytest.mark.parametrize("run", RUNS)
def test_expert_gelu_over_its_range(run):
    """The erf form, through an expert whose down projection picks its hidden units."""
    dev, dt = run
    z = torch.linspace(-6, 6, 64, dtype=torch.float64).to(torch.bfloat16).double()
    spec = ExpertsSpec(ff=64, experts=1, top=1, score="softmax", renorm=True, expert="gelu")
    eye = torch.eye(64, dtype=torch.float64)
    w = {"router": torch.zeros(1, 64), "up": torch.diag(z)[None], "down": eye[None]}
    h = torch.ones(3, 64, dtype=torch.float64)
    y, _, _ = mops.experts(h.to(dev, dt), {k: t.to(dev, dt) for k, t in w.items()}, spec)
    want = plain.gelu_erf(z)
    err = (y[:, 0].double().cpu() - want).abs()
    tol = 1e-6 if dt == torch.float32 else 0.0
    assert bool((err <= tol + want.abs() * (1e-5 if dt == torch.float32 else 5e-3) + 1e-6).all())


@GPU
def test_fused_gate_up_gelu():
    """The prefill GEMM's gelu epilogue."""
    from omnia_amd import ops

    g = gen(5)
    x, w = rnd(300, 256, g=g), rnd(2 * 384, 256, g=g, scale=0.1)
    got = ops.pgemm(1, x.bfloat16().cuda(), w.bfloat16().cuda(), gelu=True)
    v = x @ w.T
    assert rel(got, plain.gelu_tanh(v[:, :384]) * v[:, 384:]) < 6e-3


# -------------------------------------------------------------------- routing
ROUTES = [(8, 2, 1, 1, 0), (6, 2, 4, 2, 2), (5, 3, 3, 2, 1), (1, 1, 1, 1, 0), (1, 2, 1, 1, 1),
          (12, 4, 8, 3, 4), (63, 5, 10, 4, 7), (20, 9, 12, 6, 4), (200, 6, 8, 2, 56),
          (128, 64, 128, 128, 0), (17, 3, 1, 1, 0)]


def routed(run, h, router, corr, top, groups, keep):
    """(ids, weights) of the framework."""
    dev, dt = run
    spec = ExpertsSpec(ff=64, experts=router.shape[0], top=top, score="softmax", renorm=True,
                       expert="gelu", correction=True, groups=groups, keep=keep)
    x, r, c = h.to(dev, dt), router.to(dev, dt), corr.float().to(dev)
    if dev == "cpu":
        from omnia_amd.ops import reference_mixers as ref

        ids, wts = ref.route(x, r, spec, c)
    else:
        from omnia_amd.ops import kernels

        ids = torch.empty(h.shape[0], top, dtype=torch.int32, device=dev)
        wts = torch.empty(h.shape[0], top, device=dev)
        kernels().moe_route(ids, wts, x, r, top, False, True, c, groups, keep)
    return ids.cpu().long(), wts.cpu().double()


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("E,top,groups,keep,identity", ROUTES)
@pytest.mark.parametrize("shift", [0.0, -3.0])
def test_grouped_routing(E, top, groups, keep, identity, shift, run):
    """Choice by corrected scores of both signs (all negative with the shift: a masked expert
    is minus infinity, not 0) within the best groups; weights by plain scores."""
    g = gen(E + top)
    n, d, T = E + identity, 96, 61
    router, corr = rnd(n, d, g=g, scale=0.3), 0.5 * rnd(n, g=g) + shift
    h = rnd(400, d, g=g)
    ids, wts = plain.route(h, router, corr, top, groups, keep)
    # no close calls: neighbours in the choice and at the edge of the groups well apart
    s = torch.softmax(h @ router.T, -1) + corr
    best = s.view(400, groups, -1).max(-1).values
    gs = best.sort(-1, descending=True).values
    c = s.masked_fill((best < gs[:, keep - 1:keep]).repeat_interleave(n // groups, 1),
                      float("-inf")).sort(-1, descending=True).values
    gap = (c[:, :-1] - c[:, 1:])[:, :top].min(-1).values if n > 1 else torch.ones(400)
    if keep < groups:
        gap = torch.minimum(gap, gs[:, keep - 1] - gs[:, keep])
    pick = gap.nan_to_num(1.0).sort(descending=True).indices[:T]
    assert float(gap[pick].min()) > 1e-5
    got, w = routed(run, h[pick], router, corr, top, groups, keep)
    assert torch.equal(got, ids[pick]) and rel(w, wts[pick]) < 1e-5


@pytest.mark.parametrize("run", RUNS)
def test_routing_by_hand(run):
    """Two groups: the one with the single best expert wins, not the one with more; the
    correction chooses but does not weigh."""
    d = 32
    router = torch.zeros(6, d, dtype=torch.float64)
    router[:, 0] = torch.tensor([1.0, 1.0, 1.0, 1.5, -2.0, -2.0])
    h = torch.zeros(1, d, dtype=torch.float64)
    h[0, 0] = 1.0
    s = torch.softmax(router[:, 0], 0)
    ids, w = routed(run, h, router, torch.zeros(6), 2, 2, 1)
    assert ids.tolist() == [[3, 4]]  # ties by number
    assert rel(w[0], s[[3, 4]] / s[[3, 4]].sum()) < 1e-6
    corr = torch.tensor([0.0, 0.0, 0.5, 0.0, 0.0, 0.4])
    ids, w = routed(run, h, router, corr, 3, 2, 1)
    assert ids.tolist() == [[2, 0, 1]] and rel(w[0], torch.full((3,), 1 / 3)) < 1e-6
    ids, w = routed(run, h, router, corr, 3, 2, 2)
    assert ids.tolist() == [[2, 5, 3]]
    assert rel(w[0], s[[2, 5, 3]] / s[[2, 5, 3]].sum()) < 1e-6


@pytest.mark.parametrize("run", RUNS)
def test_router_logits_stay_exact(run):
    """Neighbours that 16 bits would merge are told apart."""
    E, d = 12, 64
    router = torch.zeros(E, d, dtype=torch.float64)
    router[:, 0] = 8.0
    router[:, 1] = 2.0 ** -9 * torch.arange(E)  # 8 + e / 512: below bf16's spacing at 8
    h = torch.zeros(17, d, dtype=torch.float64)
    h[:, 0], h[:, 1] = torch.linspace(-1, 1, 17), 1.0
    ids, w = routed(run, h, router, torch.zeros(E), 3, 1, 1)
    assert ids.tolist() == [[11, 10, 9]] * 17
    _, want = plain.route(h.to(torch.bfloat16).double(), router, torch.zeros(E).double(), 3, 1, 1)
    assert rel(w, want) < 1e-6


def run_experts(run, E, top, d, ff, T, groups=1, keep=1, identity=0, seed=8):
    """(framework [T, d] added to a residual of zeros, plain)."""
    dev, dt = run
    g = gen(seed)
    n = E + identity
    spec = ExpertsSpec(ff=ff, experts=E, top=top, score="softmax", renorm=True, expert="gelu",
                       correction=True, groups=groups, keep=keep, identity=identity)
    W = {"router": torch.zeros(n, d, dtype=torch.float64), "correction": 0.05 * rnd(n, g=g)}
    W["router"][:, :8] = rnd(n, 8, g=g)
    for e in range(E):
        W[f"e{e}.up"] = rnd(ff, d, g=g, scale=1.5 * d ** -0.5)
        W[f"e{e}.down"] = rnd(d, ff, g=g, scale=ff ** -0.5)
    h = rnd(T, d, g=g, scale=2.0)
    if T > 1:  # rows the router is sure of, repeated codes with fresh features
        codes = rnd(256, 8, g=g, scale=2.0)
        x = torch.zeros(256, d, dtype=torch.float64)
        x[:, :8] = codes
        a, _ = plain.route(x, W["router"], W["correction"], top, groups, keep)
        noisy = torch.stack([plain.route(x * (1 + 0.02 * (2 * torch.rand(
            x.shape, generator=g, dtype=torch.float64) - 1)), W["router"], W["correction"], top,
            groups, keep)[0] for _ in range(3)])
        sure = codes[(noisy.sort(-1).values == a.sort(-1).values).all(-1).all(0)]
        h[:, :8] = sure[torch.arange(T) % sure.shape[0]]
    model = Stub(dev, dt, 1e-5)
    mod = Experts(spec, model)
    dp = -(-d // 64) * 64
    w = mod.pack(lambda k: W[k].to(dev, dt), dp)
    out = mod.forward(w, pad(h, dp).to(dev, dt), False)
    assert ("identity" in out) == (identity > 0)
    x = torch.zeros(T, dp, device=dev)
    one = torch.ones(dp, device=dev)
    mops.norm_residual(x, post=None, pre=mops.TanhNorm(1.0, one, one), dtype=dt, **out)
    mlp = {"router": {"experts": E, "top": top, "groups": {"count": groups, "keep": keep}}}
    return x[:, :d], plain.experts(h, mlp, W.__getitem__)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("E,top,d,ff,T,groups,keep,identity", [
    (8, 2, 128, 64, 40, 1, 1, 0), (6, 3, 72, 27, 33, 2, 1, 2), (1, 1, 64, 64, 3, 1, 1, 0),
    (1, 3, 64, 40, 9, 1, 1, 2), (63, 5, 48, 16, 50, 10, 4, 7), (16, 1, 256, 192, 65, 4, 1, 0),
    (3, 2, 100, 130, 1, 2, 2, 1)])
def test_gelu_experts(E, top, d, ff, T, groups, keep, identity, run):
    got, want = run_experts(run, E, top, d, ff, T, groups, keep, identity)
    assert rel(got, want) < LIMIT[run[1]]


@GPU
@pytest.mark.parametrize("d", [256, 512])
def test_gelu_experts_on_the_prefill_tile(d):
    """Enough rows per expert for the 256x256 tile (bf16); a ragged last segment."""
    run = ("cuda", torch.bfloat16)
    got, want = run_experts(run, 2, 1, d, 256, 1100)
    assert rel(got, want) < 0.012
    got, want = run_experts(run, 3, 2, d, 512, 900, 2, 2, 1)
    assert rel(got, want) < 0.012


# ----------------------------------------------------------------------- loops
def test_loops_and_names():
    """Passes of a looped layer share tensors under the checkpoint's numbers; every pass has
    a cache of its own."""
    import bisuzen_cases as sc

    d = DESIGNS["bisuzen"]
    entries = [sc.chunked(size=s) for s in (5, 6, 7, 8)]
    ls = parse_layers(entries, d, {"start": 1, "stop": 3, "times": 3})
    assert [l.mixer.chunk for l in ls] == [5, 6, 7, 6, 7, 6, 7, 8]
    assert [l.weights_of for l in ls] == [None, None, None, 1, 2, 1, 2, None]
    assert [l.index for l in ls] == [0, 1, 2, 1, 2, 1, 2, 3]
    assert plain.order({"layers": entries, "loop": {"start": 1, "stop": 3, "times": 3}}) == [
        l.index for l in ls]
    for loop in (None, {"start": 0, "stop": 4, "times": 1}, {"start": 2, "stop": 2, "times": 5}):
        assert [l.mixer.chunk for l in parse_layers(entries, d, loop)] == [5, 6, 7, 8]
    for loop in ({"start": 2, "stop": 5, "times": 1}, {"start": 0, "stop": 1, "times": 0}):
        with pytest.raises(ValueError, match="loop"):
            parse_layers(entries, d, loop)
    # a borrowing layer inside a loop borrows from its own pass, one behind it from the last
    kv = [{"type": "attention", "mixer": {
        "heads": 2, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 1.0,
        "rot": {"base": 1e4, "dims": 8}, **({"kv_from": 0} if i else {})}} for i in range(3)]
    ls = parse_layers(kv, DESIGNS["sekazen"], {"start": 0, "stop": 2, "times": 2})
    assert [l.mixer.kv_from for l in ls] == [None, 0, None, 2, 2]


def test_plain_pieces():
    """The oracle's own arithmetic on numbers worked out by hand."""
    assert plain.softmax(torch.zeros(1, 3), torch.tensor(0.0))[0].tolist() == [0.25] * 3
    assert plain.sees_window(5, 2, 1).int().tolist() == [
        [1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [1, 1, 1, 0, 0], [1, 0, 1, 1, 0], [1, 0, 0, 1, 1]]
    assert plain.sees_chunk(5, 2).int().tolist() == [
        [1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [0, 0, 1, 0, 0], [0, 0, 1, 1, 0], [0, 0, 0, 0, 1]]
    one = torch.ones(3, 1, 1, dtype=torch.float64)
    o, S = plain.recurrence(one, one, 2 * one, [0.5])
    assert o.flatten().tolist() == [2.0, 3.0, 3.5] and float(S) == 3.5
    x = torch.tensor([[[1.0, 2.0, 3.0]], [[1.0, 2.0, 3.0]]], dtype=torch.float64)
    r = plain.rotate(x, {"dims": 2, "base": 7.0})
    c, s = math.cos(1.0), math.sin(1.0)
    assert torch.equal(r[0], x[0])
    assert r[1, 0].tolist() == pytest.approx([c - 2 * s, 2 * c + s, 3.0])
    z = torch.tensor([1.0, -2.0], dtype=torch.float64)
    assert torch.allclose(plain.gelu_erf(z), F.gelu(z))
    assert torch.allclose(plain.gelu_tanh(z), F.gelu(z, approximate="tanh"))
    assert torch.allclose(plain.silu(z), F.silu(z))
