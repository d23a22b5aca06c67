"""Each Sekazen mechanism alone -- norms around the residual, frequency bands and partial
rotation, query/key norms, windows, sinks, expert routing and the clamped GLU, the logit
cap -- against its plain function, at sizes a served model has as well as ragged ones.
CPU path and, marked gpu, the HIP kernels."""
import math
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(__file__))
import plain_sekazen as plain  # noqa: E402

from omnia_amd.models.layers import (AttentionSpec, BandSpec, ExpertsSpec,  # noqa: E402
                                     RotarySpec)
from omnia_amd.models.llama import ForwardBatch  # noqa: E402
from omnia_amd.models.mixers import GroupedQueryAttention, rotary_table  # noqa: E402
from omnia_amd.ops import mixers as mops  # noqa: E402
from omnia_amd.ops import prefill_tiles  # noqa: E402

GPU = pytest.mark.gpu
RUNS = [pytest.param(("cpu", torch.float32), id="cpu"),
        pytest.param(("cuda", torch.float32), id="gpu32", marks=GPU),
        pytest.param(("cuda", torch.bfloat16), id="gpu16", marks=GPU)]
LIMIT = {torch.float32: 3e-5, torch.bfloat16: 0.012}


def rel(got, want):
    want = want.double()
    return float((got.double().cpu() - want.cpu()).norm() / want.norm().clamp(min=1e-30))


def gen(seed=0):
    return torch.Generator().manual_seed(seed)


def rnd(*shape, g, scale=1.0):
    """float64, bf16-representable."""
    return (torch.randn(*shape, generator=g, dtype=torch.float64) * scale).to(
        torch.bfloat16).double()


# ------------------------------------------------------------------- RMS norms
@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("n,d", [(5, 8), (72, 128), (1000, 1024), (1100, 1152), (2048, 2048),
                                 (4096, 4096), (5000, 5056), (9000, 9024)])
def test_rms_residual(n, d, run):
    """Plain rows, split-K slabs and expert slots; identity and a pre-norm after; zero
    padding columns do not enter the mean."""
    dev, dt = run
    g = gen(n)
    M, eps = 5, 3e-3
    w1, w2 = 0.3 * rnd(n, g=g), 0.3 * rnd(n, g=g)

    def pad(t):
        return torch.nn.functional.pad(t, (0, d - n))

    def norm(w):
        return mops.RMSNorm(pad(1.0 + w).float().to(dev), n, eps)

    x0 = rnd(M, n, g=g, scale=2.0)
    kinds = [(dt, 1, False), (torch.float32, 3, False), (dt, 2, True)]
    if dt == torch.bfloat16:
        kinds.append((torch.float16, 5, False))
    for pdt, S, slots in kinds:
        parts = rnd(S, M, n, g=g, scale=0.05)  # small: eps inside the root matters
        m = pad(parts.transpose(0, 1) if slots else parts)
        m = (m[0] if S == 1 else m).contiguous().to(dev, pdt)
        for pre, bias in ((None, None), (w2, None), (None, 0.1 * w2)):
            wx = x0 + plain.norm_one_plus(parts.sum(0) + (0 if bias is None else bias), w1, eps)
            x = pad(x0).float().to(dev)
            h = mops.norm_residual(x, m, norm(w1), None if pre is None else norm(pre), dt,
                                   None if bias is None else pad(bias).float().to(dev), slots)
            wh = wx if pre is None else plain.norm_one_plus(wx, pre, eps)
            assert rel(x[:, :n], wx) < 2e-6 and rel(h[:, :n], wh) < (
                2e-6 if dt == torch.float32 else 3e-3)
            assert float(x[:, n:].abs().sum()) == 0 and float(h[:, n:].float().abs().sum()) == 0


@pytest.mark.parametrize("run", RUNS)
def test_rms_embed(run):
    dev, dt = run
    g = gen(1)
    n, d, V, eps = 45, 64, 33, 1e-3
    table, w1, w2 = rnd(V, n, g=g), 0.3 * rnd(n, g=g), 0.3 * rnd(n, g=g)

    def norm(w):
        return mops.RMSNorm(torch.nn.functional.pad(1.0 + w, (0, d - n)).float().to(dev), n, eps)

    tab = torch.nn.functional.pad(table, (0, d - n)).to(dev, dt)
    ids = torch.tensor([0, 32, 7, 7, 5], dtype=torch.int32, device=dev)
    # two tokens still on the device
    src = torch.tensor([-1, 2, -1, 1, -1], device=dev)
    slots = torch.tensor([9, 11, 30], dtype=torch.int32, device=dev)
    real = [0, 30, 7, 11, 5]
    want = plain.norm_one_plus(table[real], w1, eps)
    for pre in (None, w2):
        x, h = mops.norm_embed(ids, tab, V, norm(w1), None if pre is None else norm(pre), src,
                               slots)
        assert rel(x[:, :n], want) < 1e-6 and float(x[:, n:].abs().sum()) == 0
        assert rel(h[:, :n], want if pre is None else plain.norm_one_plus(want, pre, eps)) < (
            1e-6 if dt == torch.float32 else 3e-3)


@pytest.mark.parametrize("run", RUNS)
def test_softcap(run):
    dev, dt = run
    for shape in ((1, 1), (3, 71), (5, 4096)):
        z = rnd(*shape, g=gen(2), scale=30.0)
        want = plain.softcap(z, 9.0)
        got = mops.softcap_(z.to(dev, dt), 9.0)
        assert rel(got, want) < (1e-6 if dt == torch.float32 else 3e-3)
        assert float(got.float().abs().max()) <= 9.0


# -------------------------------------------------------------------- rotation
@pytest.mark.parametrize("dims,base,bands", [
    (12, 1e4, None), (2, 1e4, (8.0, 1.0, 4.0, 64)), (64, 5e5, (8.0, 1.0, 4.0, 8192)),
    (128, 1e4, (32.0, 1.0, 4.0, 8192)), (48, 700.0, (4.0, 2.0, 2.0, 128)),
    (32, 1e4, (3.0, 0.5, 16.0, 2048))])
def test_frequency_bands(dims, base, bands):
    rot = {"dims": dims, "base": base}
    if bands:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), bands))
    spec = RotarySpec(dims, base, bands=BandSpec(*bands) if bands else None)
    f, want = spec.frequencies(), plain.frequencies(rot)
    assert f == pytest.approx(want, rel=1e-12)
    raw = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if bands and dims >= 32:  # a kept, a blended (unless the band is empty) and a slowed pair
        ratio = [a / b for a, b in zip(f, raw)]
        assert max(ratio) == 1.0 and min(ratio) == pytest.approx(1.0 / bands[0])
        assert bands[1] == bands[2] or any(1.01 / bands[0] < r < 0.99 for r in ratio)
    far = rotary_table(spec, 120001, "cpu")[120000]
    a = torch.tensor(want, dtype=torch.float64) * 120000
    assert torch.allclose(far.double(), torch.cat([a.cos(), a.sin()]), atol=1e-7)


def make(dev, dt, spec, g, page=16, blocks=24):
    """(module, packed weights, fp64 tensors): one attention layer of width 40 outside any
    model."""
    class M:
        device, dtype = torch.device(dev), dt

        @staticmethod
        def rotary(rot):
            return rotary_table(rot, 4096, dev)

    mod = GroupedQueryAttention(spec, M)
    d, n = 40, spec
    W = {"q": rnd(n.heads * n.dim, d, g=g), "k": rnd(n.kv_heads * n.dim, d, g=g),
         "v": rnd(n.kv_heads * n.vdim, d, g=g), "q.norm": 1 + 0.3 * rnd(n.dim, g=g),
         "k.norm": 1 + 0.3 * rnd(n.dim, g=g), "o": rnd(d, n.heads * n.vdim, g=g),
         "sink": rnd(n.heads, g=g)}
    W = {k: v.to(torch.bfloat16).double() for k, v in W.items()}
    return mod, mod.pack(lambda k: W[k].to(dev, dt), d), W


SHAPES = {  # heads, kv heads, dim, vdim, rotated dims
    "served": (8, 2, 128, 128, 64), "ragged": (3, 1, 22, 13, 6), "whole": (4, 4, 64, 32, 64),
    "pair": (6, 2, 96, 192, 2), "group10": (20, 2, 32, 64, 8), "big": (2, 1, 256, 256, 96),
    "past": (2, 2, 300, 264, 300), "mixed": (5, 5, 192, 96, 24)}


def spec_of(shape, window=0, scale=None, sink=True):
    H, G, D, V, R = SHAPES[shape]
    return AttentionSpec(H, G, D, V, scale or D ** -0.5, RotarySpec(R, 1e4), window,
                         "learned" if sink else None)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("shape", sorted(SHAPES))
def test_query_key_norm_rotation_and_pages(shape, run):
    dev, dt = run
    g = gen(3)
    spec = spec_of(shape)
    H, G, D, V = spec.heads, spec.kv_heads, spec.dim, spec.vdim
    mod, w, W = make(dev, dt, spec, g)
    T, page, eps = 21, 16, 1e-2
    h = rnd(T, 40, g=g)
    pos = torch.arange(T, dtype=torch.int32, device=dev)
    slots = torch.arange(T, device=dev) + 3 * page
    slots[4] = -1  # a padded row writes nothing
    rot = {"dims": spec.rotary.dims, "base": 1e4}
    q = plain.rotate(plain.rms((h @ W["q"].T).view(T, H, D), eps) * W["q.norm"], rot)
    k, v = plain.keys_values(h, {"kv_heads": G, "dim": D, "vdim": V, "rot": rot}, W.get, eps)
    xr = torch.nn.functional.linear(h.to(dev, dt).float(), w["in"].float())
    S = 3
    inputs = [xr.to(dt)]
    if dt == torch.bfloat16 or dev == "cpu":
        cuts = torch.rand(S, 1, 1, generator=g).to(dev)
        inputs.append((xr * cuts / cuts.sum()).contiguous())  # slabs
        if dt == torch.bfloat16:
            inputs.append((xr * cuts / cuts.sum()).half().contiguous())
    for x in inputs:
        pages, _ = mod_alloc(mod, 6, page)
        got = mops.gqa_prep(x, w, spec, pages, pos, slots, mod.table, dt, eps)
        assert rel(got.view(T, H, -1)[..., :D], q) < LIMIT[dt]
        assert float(got.view(T, H, -1)[..., D:].float().abs().sum()) == 0
        kc = pages[0].cpu().double()[3:5].transpose(1, 2).reshape(2 * page, G, -1)[:T]
        vc = pages[1].cpu().double()[3:5].transpose(1, 2).reshape(2 * page, G, -1)[:T]
        keep = [t for t in range(T) if t != 4]
        assert rel(kc[keep][..., :D], k[keep]) < LIMIT[dt]
        assert rel(vc[keep][..., :V], v[keep]) < LIMIT[dt]
        assert float(kc[4].abs().sum() + vc[4].abs().sum()) == 0
        # a borrowing layer: queries alone, pages untouched
        before = pages[0].clone()
        qo = mops.gqa_prep(x, {"q_norm": w["q_norm"]}, spec, None, pos, slots, mod.table, dt, eps)
        assert torch.equal(qo, got) and torch.equal(before, pages[0])


def mod_alloc(mod, blocks, page):
    return mod.alloc(blocks, page, 1)


# -------------------------------------------------------------- attention
def dense(q, k, v, scale, window, sinks):
    """q [T, H, D] at the last T of the n positions of k, v [n, G, .] -> [T, H, V]."""
    T, H = q.shape[:2]
    n, G = k.shape[:2]
    seen = plain.visible(n, {"mask": {"size": window}} if window else {})[n - T:]
    out = []
    for h in range(H):
        s = (q[:, h] @ k[:, h // (H // G)].T * scale).masked_fill(~seen, float("-inf"))
        sink = torch.tensor(-float("inf"), dtype=s.dtype) if sinks is None else sinks[h]
        out.append(plain.sink_softmax(s, sink) @ v[:, h // (H // G)])
    return torch.stack(out, 1)


class Paged:
    """Sequences laid out in shuffled pages, and the three attention entry points."""

    def __init__(self, run, spec, g, page=16, blocks=200):
        self.dev, self.dt = run
        self.spec, self.page = spec, page
        self.mod, self.w, _ = make(self.dev, self.dt, spec, g)
        self.pages, _ = self.mod.alloc(blocks, page, 1)
        for p in self.pages:  # what other sequences left
            p.copy_(torch.randn(p.shape, generator=g) * 3)
        self.free = (1 + torch.randperm(blocks - 1, generator=g)).tolist()

    def put(self, k, v):
        """Store keys / values; the sequence's pages."""
        n = k.shape[0]
        bt = [self.free.pop() for _ in range(-(-n // self.page))]
        for t, (pg, z) in ((0, (self.pages[0], k)), (1, (self.pages[1], v))):
            z = torch.nn.functional.pad(z, (0, pg.shape[3] - z.shape[2])).to(self.dev, self.dt)
            for b, blk in enumerate(bt):
                rows = z[b * self.page:(b + 1) * self.page]
                pg[blk, :, :rows.shape[0]] = rows.transpose(0, 1)
        return bt

    def table(self, bts):
        n = max(len(b) for b in bts)
        return torch.tensor([b + [0] * (n - len(b)) for b in bts], dtype=torch.int32,
                            device=self.dev)

    def q(self, q):
        q = torch.nn.functional.pad(q, (0, self.spec.dim_pad - self.spec.dim))
        return q.reshape(q.shape[0], -1).to(self.dev, self.dt)

    def heads(self, o):
        s = self.spec
        return o.view(o.shape[0], s.heads, s.v_pad)[..., :s.vdim].double().cpu()

    def prefill(self, qs, bts, lens, sinks):
        """Portions ``qs[i]`` = the last queries of a sequence of ``lens[i]`` keys."""
        nq = [q.shape[0] for q in qs]
        start = torch.tensor([0] + nq).cumsum(0).to(torch.int32).to(self.dev)
        ts, t0 = prefill_tiles(nq, 128)
        pos = torch.cat([torch.arange(n - m, n) for n, m in zip(lens, nq)])
        pos = pos.to(torch.int32).to(self.dev)

        def ints(x):
            return torch.tensor(x, dtype=torch.int32, device=self.dev)

        fb = ForwardBatch(None, pos, None, self.table(bts), ints(lens), None, is_decode=False,
                          q_start_loc=start, tile_seq=ints(ts), tile_q0=ints(t0))
        w = dict(self.w, sink=sinks)
        return self.heads(self.mod._prefill(w, self.q(torch.cat(qs)), self.pages, fb, pos, None))

    def decode(self, q, bts, lens, sinks, splits=None):
        pos = torch.tensor([n - 1 for n in lens], dtype=torch.int32, device=self.dev)
        bt, qq = self.table(bts), self.q(q)
        if splits is not None and self.mod.mfma:
            return self.heads(mops.gqa_decode(qq, self.pages, bt, pos, self.spec, sinks, splits))
        return self.heads(self.mod._decode(dict(self.w, sink=sinks), qq, self.pages, bt, pos,
                                           None))


def sink_pair(spec, g, dev):
    s = rnd(spec.heads, g=g, scale=2.0)
    return s, s.float().to(dev)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("shape,window,sink", [
    ("served", 0, True), ("served", 100, True), ("served", 1, True), ("served", 64, False),
    ("ragged", 33, True), ("whole", 0, False), ("pair", 70, True), ("group10", 48, True),
    ("big", 90, True), ("past", 40, True), ("mixed", 129, True)])
def test_attention_prefill_and_decode(shape, window, sink, run):
    """Unequal portions over shuffled pages; the same rows decoded, in any number of parts."""
    g = gen(4)
    spec = spec_of(shape, window, scale=1.5 * SHAPES[shape][2] ** -0.5, sink=sink)
    P = Paged(run, spec, g)
    sinks = sink_pair(spec, g, P.dev) if sink else (None, None)
    lens, nq = [1, 17, 150, 300, 64, 129], [1, 2, 131, 45, 64, 129]
    ks = [rnd(n, spec.kv_heads, spec.dim, g=g) for n in lens]
    vs = [rnd(n, spec.kv_heads, spec.vdim, g=g) for n in lens]
    qs = [rnd(m, spec.heads, spec.dim, g=g) for m in nq]
    bts = [P.put(k, v) for k, v in zip(ks, vs)]
    want = [dense(q, k, v, spec.scale, window, sinks[0]) for q, k, v in zip(qs, ks, vs)]
    got = P.prefill(qs, bts, lens, sinks[1])
    o = 0
    for i, w in enumerate(want):
        assert rel(got[o:o + nq[i]], w) < LIMIT[P.dt], (i, lens[i])
        o += nq[i]
    last = torch.stack([q[-1] for q in qs])
    ends = torch.stack([w[-1] for w in want])
    for splits in (None, 1, 2, 5, 16):
        got = P.decode(last, bts, lens, sinks[1], splits)
        for i in range(len(lens)):
            assert rel(got[i], ends[i]) < LIMIT[P.dt], (splits, lens[i])


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("window", [0, 1, 2, 16, 17, 31, 32, 33, 64, 65, 100])
def test_one_key_that_stands_out(window, run):
    """One key far above all others, at every page edge and around the window's: seen, the
    output is its value; outside, nothing of it is left."""
    g = gen(5)
    H, G, D, V = 2, 1, 32, 32
    spec = AttentionSpec(H, G, D, V, 1.0, RotarySpec(8, 1e4), window)
    P = Paged(run, spec, g, page=16, blocks=600)
    n = 130
    spots = sorted({0, 1, 15, 16, 17, 31, 32, 63, 64, 65, 127, 128, n - 1} |
                   {min(n - 1, max(0, n - 1 - window + e)) for e in (-1, 0, 1, 2)})
    sinks = torch.zeros(H, dtype=torch.float64)
    for spot in spots:
        k, v = rnd(n, G, D, g=g, scale=0.01), rnd(n, G, V, g=g)
        q = torch.zeros(n, H, D, dtype=torch.float64)
        q[..., 3] = 8.0
        k[spot, :, 3] = 8.0  # its score is 64
        v[spot] += 5.0
        bt = P.put(k, v)
        want = dense(q, k, v, 1.0, window, sinks)
        got = P.prefill([q], [bt], [n], sinks.float().to(P.dev))
        for i in range(n):
            e = float((got[i] - want[i]).abs().max())
            assert e < (1e-4 if P.dt == torch.float32 else 0.06), (spot, i, e)
            if i >= spot and (window == 0 or i - spot < window):
                assert float((want[i] - v[spot]).abs().max()) < 1e-6
        for m in (n, max(1, spot + 1), min(n, spot + max(1, window)),
                  min(n, spot + window + 1)):  # decoded just inside and just outside
            for splits in (1, 3):
                got1 = P.decode(q[m - 1:m], [bt], [m], sinks.float().to(P.dev), splits)
                e = float((got1[0] - want[m - 1]).abs().max())
                assert e < (1e-4 if P.dt == torch.float32 else 0.06), (spot, m, splits, e)
        P.free = bt + P.free


@pytest.mark.parametrize("run", RUNS)
def test_sinks(run):
    """A sink takes its share of the softmax once, whatever the split; far below the scores
    it vanishes, far above it leaves nothing; heads do not share it."""
    g = gen(6)
    spec = AttentionSpec(4, 2, 64, 64, 0.125, RotarySpec(8, 1e4), 90)
    P = Paged(run, spec, g)
    n = 200
    k, v, q = (rnd(n, 2, 64, g=g), rnd(n, 2, 64, g=g), rnd(n, 4, 64, g=g))
    bt = P.put(k, v)
    for sinks in ([-300.0, 0.0, 5.0, 30.0], [200.0, -1.0, 4.0, 90.0]):
        s = torch.tensor(sinks, dtype=torch.float64)
        want = dense(q, k, v, 0.125, 90, s)
        dev = s.float().to(P.dev)
        got = P.prefill([q], [bt], [n], dev)
        for h in range(4):
            assert rel(got[:, h], want[:, h]) < LIMIT[P.dt] or \
                float(got[:, h].abs().max()) < 1e-10, (sinks, h)
        for splits in (1, 2, 7):
            d = P.decode(q[-1:], [bt], [n], dev, splits)[0]
            for h in range(4):
                assert rel(d[h], want[-1, h]) < LIMIT[P.dt] or float(d[h].abs().max()) < 1e-10
    free = dense(q, k, v, 0.125, 90, None)
    low = P.prefill([q], [bt], [n], torch.full((4,), -1e4, device=P.dev))
    assert rel(low, free) < LIMIT[P.dt] and rel(P.prefill([q], [bt], [n], None), free) < LIMIT[P.dt]


@pytest.mark.gpu
@pytest.mark.parametrize("page", [8, 16, 64])
def test_long_contexts(page):
    """Thousands of keys and pages: parts longer than one score tile, contexts that differ."""
    g = gen(7)
    for window in (0, 1500):
        spec = AttentionSpec(8, 2, 64, 64, 0.2, RotarySpec(8, 1e4), window)
        P = Paged(("cuda", torch.bfloat16), spec, g, page=page, blocks=6000 // page * 2)
        lens = [5000, 1025, 3]
        ks = [rnd(n, 2, 64, g=g) for n in lens]
        vs = [rnd(n, 2, 64, g=g) for n in lens]
        qs = [rnd(min(n, 40), 8, 64, g=g) for n in lens]
        bts = [P.put(k, v) for k, v in zip(ks, vs)]
        sinks, dev = sink_pair(spec, g, "cuda")
        want = [dense(q, k, v, 0.2, window, sinks) for q, k, v in zip(qs, ks, vs)]
        got = P.prefill(qs, bts, lens, dev)
        assert rel(got, torch.cat(want)) < 0.012
        d = P.decode(torch.stack([q[-1] for q in qs]), bts, lens, dev)
        for i in range(3):
            assert rel(d[i], want[i][-1]) < 0.012


# ---------------------------------------------------------------- experts
def expert_weights(E, d, ff, g, scale=1.0):
    W = {"router": rnd(E, d, g=g, scale=d ** -0.5)}
    for e in range(E):
        W.update({f"e{e}.gate": rnd(ff, d, g=g, scale=scale * d ** -0.5),
                  f"e{e}.up": rnd(ff, d, g=g, scale=scale * d ** -0.5),
                  f"e{e}.down": rnd(d, ff, g=g, scale=ff ** -0.5)})
    return W


def run_experts(run, E, top, d, ff, T, limit, scale=1.0, seed=8):
    """(framework [T, d], plain [T, d]): inputs without a close call at the cut."""
    from omnia_amd.models.feedforward import Experts

    dev, dt = run
    g = gen(seed)
    spec = ExpertsSpec(ff=ff, experts=E, top=top, limit=limit)
    W = expert_weights(E, d, ff, g, scale)
    h = rnd(4 * T + 64, d, g=g, scale=2.0)
    z = (h @ W["router"].T).sort(-1, descending=True).values
    if top < E:
        h = h[z[:, top - 1] - z[:, top] > 1e-3]
    assert h.shape[0] >= T
    h = h[:T].contiguous()

    class M:
        device, dtype = torch.device(dev), dt

    dp = -(-d // 64) * 64
    mod = Experts(spec, M)
    w = mod.pack(lambda n: W[n].to(dev, dt), dp)
    x = torch.nn.functional.pad(h, (0, dp - d)).to(dev, dt)
    out = mod.forward(w, x, False)
    assert out["slots"] and out["m"].shape == (T, top, dp)
    assert float(out["m"][..., d:].float().abs().sum()) == 0
    mlp = {"router": {"experts": E, "top": top}, "expert": {"ff": ff, "limit": limit}}
    return out["m"][..., :d].double().cpu().sum(1), plain.experts(h, mlp, W.get)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("E,top,d,ff,T", [
    (8, 2, 128, 64, 40), (5, 5, 72, 27, 33), (1, 1, 64, 64, 3), (70, 6, 48, 16, 50),
    (200, 3, 64, 8, 9), (16, 1, 256, 192, 65), (3, 2, 100, 130, 1)])
def test_experts(E, top, d, ff, T, run):
    got, want = run_experts(run, E, top, d, ff, T, limit=1.1)
    assert rel(got, want) < LIMIT[run[1]]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("limit", [0.05, 0.5, 100.0])
def test_clamps_and_weighted_input(limit, run):
    """Both clamps bite after the weight: weighting the output instead would be seen."""
    got, want = run_experts(run, 4, 2, 64, 64, 24, limit, scale=3.0)
    assert rel(got, want) < LIMIT[run[1]]
    g = gen(9)
    W = expert_weights(4, 64, 64, g, 3.0)
    h = rnd(24, 64, g=g, scale=2.0)
    ids, wt = plain.route(h, W["router"], 2)
    after = sum(wt[:, j, None] * torch.stack([plain.expert(
        h[t:t + 1], lambda n, t=t: W[f"e{int(ids[t, j])}.{n}"], limit)[0] for t in range(24)])
        for j in range(2))
    mlp = {"router": {"top": 2}, "expert": {"limit": limit}}
    assert rel(after, plain.experts(h, mlp, W.get)) > 0.05


@pytest.mark.parametrize("run", RUNS)
def test_router_scores(run):
    """Scores stay fp32: neighbours that 16 bits would merge are told apart, and the score is
    a sigmoid that the others do not renormalise."""
    dev, dt = run
    E, d = 12, 64
    router = torch.zeros(E, d)
    router[:, 0] = 8.0  # exact in bf16
    router[:, 1] = 2.0 ** -9 * torch.arange(E)  # 8 + e / 512: below bf16's spacing at 8
    h = torch.zeros(3, d)
    h[:, 0] = torch.tensor([1.0, 0.5, -0.25])
    h[:, 1] = 1.0
    spec = ExpertsSpec(ff=64, experts=E, top=3, limit=1.0)
    if dev == "cpu":
        # the reference chooses inside `experts`; its choice shows in which down rows answer
        gu = torch.zeros(E, 128, d)
        gu[:, :64, 0] = 1.0
        down = torch.zeros(E, d, 64)
        for e in range(E):
            down[e, e] = 1.0
        y, _, _ = mops.experts(h, {"router": router, "up": gu, "down": down}, spec)
        assert [int(v) for v in y[0].abs().argmax(-1)] == [11, 10, 9]
        return
    from omnia_amd.ops import kernels

    for score, renorm in ((True, False), (True, True), (False, False), (False, True)):
        ids = torch.empty(3, 3, dtype=torch.int32, device=dev)
        wts = torch.empty(3, 3, device=dev)
        kernels().moe_route(ids, wts, h.to(dev, dt), router.to(dev, dt), 3, score, renorm)
        z = (h.double() @ router.double().T)
        s = torch.sigmoid(z) if score else torch.softmax(z, -1)
        want = s[:, [11, 10, 9]]
        if renorm:
            want = want / want.sum(-1, keepdim=True)
        assert ids.tolist() == [[11, 10, 9]] * 3 and rel(wts, want) < 1e-6


@pytest.mark.gpu
@pytest.mark.parametrize("d", [256, 512])
def test_experts_on_the_prefill_tile(d):
    """Enough rows per expert for the 256x256 tile (bf16); a ragged last segment."""
    run = ("cuda", torch.bfloat16)
    got, want = run_experts(run, 2, 1, d, 128, 1100, limit=0.7)
    assert rel(got, want) < 0.012
    got, want = run_experts(run, 3, 2, d, 256, 900, limit=0.7)
    assert rel(got, want) < 0.012


def test_plain_pieces():
    """The oracle's own arithmetic on numbers worked out by hand."""
    assert plain.sink_softmax(torch.zeros(1, 3), torch.tensor(0.0))[0].tolist() == [0.25] * 3
    one = torch.ones(1, 1, dtype=torch.float64)
    get = {"gate": 3 * one, "up": -5 * one, "down": 2 * one}.get
    g, u = 2.0, -2.0  # both clamped
    assert float(plain.expert(one, get, 2.0)) == pytest.approx(
        2 * g / (1 + math.exp(-1.702 * g)) * (u + 1))
    assert plain.visible(4, {"mask": {"size": 2}}).int().tolist() == [
        [1, 0, 0, 0], [1, 1, 0, 0], [0, 1, 1, 0], [0, 0, 1, 1]]
