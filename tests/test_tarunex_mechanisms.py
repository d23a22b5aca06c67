"""Each Tarunex mechanism alone -- the residual step of joined sublayers and what a loop's pass
enters with, biased projections with a query temperature and gates, capped scores with a
distance bias and one added to the denominator, latent attention that turns neighbours, biased
routing, experts beside a shared one -- against its plain function, at sizes a served model has
as well as ragged ones.  CPU path and, marked gpu, the HIP kernels."""
import math
import os
import sys

import pytest
import torch
import torch.nn.functional as F

sys.path.insert(0, os.path.dirname(__file__))
import plain_tarunex as plain  # noqa: E402
from test_sekazen_mechanisms import Paged, gen, rel, rnd  # noqa: E402
from test_sivadra_mechanisms import Stub, run_mixer  # noqa: E402

from omnia_amd.models.feedforward import Experts  # noqa: E402
from omnia_amd.models.layers import (DESIGNS, AttentionSpec, DenseMLPSpec,  # noqa: E402
                                     ExpertsSpec, LatentAttentionSpec, RotarySpec,
                                     TemperatureSpec, parse_layers)
from omnia_amd.models.mixers import GroupedQueryAttention, LatentAttention  # noqa: E402
from omnia_amd.ops import mixers as mops  # noqa: E402

GPU = pytest.mark.gpu
RUNS = [pytest.param(("cpu", torch.float32), id="cpu"),
        pytest.param(("cuda", torch.float32), id="gpu32", marks=GPU),
        pytest.param(("cuda", torch.bfloat16), id="gpu16", marks=GPU)]
LIMIT = {torch.float32: 3e-5, torch.bfloat16: 0.012}


def pad(t, d):
    return F.pad(t, (0, d - t.shape[-1]))


# -------------------------------------------------------- residual of joined sublayers
@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("M,n,d", [(5, 5, 8), (3, 72, 128), (600, 1000, 1024), (4, 2048, 2048),
                                   (600, 1500, 1536), (4, 4096, 4096), (600, 4000, 4096),
                                   (2, 6000, 6016), (3, 9000, 9024)])
def test_joined_residual(M, n, d, run):
    """Projections, slabs of either width and expert slots in every place; one norm or two of
    one mean, by a number and by a vector; padding columns stay zero."""
    dev, dt = run
    g = gen(n)
    eps = 3e-3
    x0 = rnd(M, n, g=g, scale=0.1)  # small: eps inside the root matters
    vec = 1.0 + 0.3 * rnd(n, g=g)

    def part(pdt, S, slots):
        p = rnd(S, M, n, g=g, scale=0.05)
        m = pad(p.transpose(0, 1) if slots else p, d)
        return p.sum(0), ((m if slots or S > 1 else m[0]).contiguous().to(dev, pdt), slots)

    def norm(w, gain):
        return mops.RMSNorm(None if w is None else pad(w, d).float().to(dev), n, eps, gain)

    half = torch.float16 if dt == torch.bfloat16 else dt
    kinds = [[], [(dt, 1, False)], [(torch.float32, 3, False), (dt, 2, True)],
             [(dt, 1, False), (dt, 3, True), (dt, 1, False)],
             [(half, 4, False), (dt, 1, True), (torch.float32, 6, False)],
             [(torch.float32, 1, False), (dt, 7, True), (half, 2, False)],
             [(dt, 1, False), (dt, 1, False)], [(half, 3, False), (half, 2, False)]]
    for kind in kinds if M < 100 else kinds[2:5]:
        made = [part(*k) for k in kind]
        want = x0 + sum((p for p, _ in made), torch.zeros(M, n, dtype=torch.float64))
        for pres in ([(None, 0.7)], [(None, 1.3), (None, 0.25)], [(vec, 1.0), (None, 0.5)],
                     [(None, 2.0), (vec, 0.3)]):
            x = pad(x0, d).float().to(dev)
            hs = mops.joined_residual(x, [m for _, m in made], [norm(*p) for p in pres], dt)
            assert len(hs) == len(pres) and rel(x[:, :n], want) < 2e-6
            assert float(x[:, n:].abs().sum()) == 0
            for h, (w, gain) in zip(hs, pres):
                wh = plain.rms(want, eps) * gain * (1.0 if w is None else w)
                assert h.dtype == dt and rel(h[:, :n], wh) < (2e-6 if dt == torch.float32 else 3e-3)
                assert float(h[:, n:].float().abs().sum()) == 0


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("n,d", [(45, 64), (2000, 2048)])
def test_entering_a_pass(n, d, run):
    """The embedding (of tokens some of which are still on the device; a padded row has none)
    and the pass's vector join the residual before the norms; the first step starts from
    them."""
    dev, dt = run
    g = gen(1)
    V, eps, scale = 33, 1e-3, 2.5
    table, step = rnd(V, n, g=g), rnd(n, g=g)
    tab, sdev = pad(table, d).to(dev, dt), pad(step, d).float().to(dev)
    ids = torch.tensor([0, 32, 7, 7, 5, -1], dtype=torch.int32, device=dev)
    src = torch.tensor([-1, 2, -1, 1, -1, -1], device=dev)
    slots = torch.tensor([9, 11, 30], dtype=torch.int32, device=dev)
    emb = table[[0, 30, 7, 11, 5, 0]] * scale
    emb[5] = 0.0
    x0, p = rnd(6, n, g=g), rnd(2, 6, n, g=g)
    m = pad(p, d).contiguous().to(dev, torch.float32)
    norms = [mops.RMSNorm(None, n, eps, 0.5), mops.RMSNorm(None, n, eps, 1.5)]
    for fresh in (True, False):
        for sc, st in ((scale, sdev), (scale, None), (0.0, sdev)):
            for parts in ([], [(m, False)]):
                e = mops.PassInput(ids, tab, V, sc, st, src, slots)
                x = pad(x0, d).float().to(dev)
                hs = mops.joined_residual(x, parts, norms, dt, e, fresh)
                want = (0.0 if fresh else x0) + (emb if sc else 0.0 * emb) + \
                    (0.0 if st is None else step) + (p.sum(0) if parts else 0.0)
                assert rel(x[:, :n], want) < 1e-6 and float(x[:, n:].abs().sum()) == 0
                for h, gain in zip(hs, (0.5, 1.5)):
                    assert rel(h[:, :n], plain.rms(want, eps) * gain) < (
                        2e-6 if dt == torch.float32 else 3e-3)


def test_passes_of_a_loop():
    """Where passes start, which tensors and names they use, and what the reader refuses."""
    import tarunex_cases as sc

    d = DESIGNS["tarunex"]
    entries = [sc.attention(cap=c) for c in (1.0, 2.0, 3.0, 4.0)]
    ls = parse_layers(entries, d, {"start": 1, "stop": 3, "times": 3})
    assert [l.mixer.softcap for l in ls] == [1, 2, 3, 2, 3, 2, 3, 4]
    assert [l.starts for l in ls] == [None, 0, None, 1, None, 2, None, None]
    assert [l.weights_of for l in ls] == [None, None, None, 1, 2, 1, 2, None]
    for loop in ({"start": 1, "stop": 3, "times": 3}, {"start": 0, "stop": 4, "times": 2},
                 {"start": 3, "stop": 4, "times": 1}, None, {"start": 2, "stop": 2, "times": 5}):
        ls = parse_layers(entries, d, loop)
        assert plain.passes({"layers": entries, "loop": loop}) == [
            (i if l.index is None else l.index, l.starts) for i, l in enumerate(ls)]


# ------------------------------------------------------ projection, temperature, gates
@pytest.mark.parametrize("coef,every", [(0.3, 16), (0.9, 1), (-0.2, 7), (0.0, 5), (0.5, 1000)])
def test_temperature(coef, every):
    got = mops.temperature_table(TemperatureSpec(coef, every), 5000, "cpu")
    want = plain.temperature(5000, {"coef": coef, "every": every}, torch.float64)
    assert float((got - want).abs().max()) < 1e-6 * (1 + abs(coef) * 9)
    t = TemperatureSpec(coef, every)
    for p in (0, every - 2, every - 1, every, 2 * every - 1, 4999):  # its steps
        if 0 <= p < 5000:
            assert float(want[p]) == pytest.approx(t.factor(p), rel=1e-12)


SHAPES = {"served": (8, 2, 128, 128), "ragged": (3, 1, 22, 13), "whole": (4, 4, 64, 32),
          "group10": (20, 2, 32, 64), "past": (2, 2, 300, 264), "mixed": (5, 5, 192, 96)}


def spec_of(shape, cap=6.0, dist=True, gate=True, temp=(0.5, 8), scale=None, **mask):
    H, G, D, V = SHAPES[shape] if isinstance(shape, str) else shape
    return AttentionSpec(H, G, D, V, scale or 1.5 * D ** -0.5, None, sink="zero", qk_norm=None,
                         bias="qkv", softcap=cap, distance_bias=dist, gate=gate,
                         temperature=TemperatureSpec(*temp) if temp else None, **mask)


class Model(Stub):
    def temperature(self, t):
        return mops.temperature_table(t, self.cfg.max_position, self.device)

    def _slabs(self, tag, x, w, is_decode):
        return F.linear(x, w)


def attention_weights(spec, d, g):
    H, G = spec.heads, spec.kv_heads
    W = {"q": rnd(H * spec.dim, d, g=g, scale=d ** -0.5),
         "k": rnd(G * spec.dim, d, g=g, scale=d ** -0.5),
         "v": rnd(G * spec.vdim, d, g=g, scale=d ** -0.5), "g": rnd(H, d, g=g, scale=d ** -0.5),
         "o": rnd(d, H * spec.vdim, g=g), "r1": 0.2 + rnd(H, g=g).abs(),
         "r2": 0.1 + rnd(H, g=g).abs()}
    W.update({n + ".b": rnd(W[n].shape[0], g=g) for n in "qkv"})
    return {k: v.to(torch.bfloat16).double() for k, v in W.items()}


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("shape", sorted(SHAPES))
def test_projection_to_queries_pages_and_gates(shape, run):
    """Biases, the temperature on queries alone, gates, from rows and from slabs."""
    dev, dt = run
    g = gen(3)
    spec = spec_of(shape)
    H, G, D, V = SHAPES[shape]
    d, T, page = 40, 21, 16
    mod = GroupedQueryAttention(spec, Model(dev, dt, 1e-5))
    W = attention_weights(spec, d, g)
    w = mod.pack(lambda n: W[n].to(dev, dt), d)
    h = rnd(T, d, g=g)
    pos = torch.arange(T, dtype=torch.int32, device=dev)
    slots = torch.arange(T, device=dev) + 3 * page
    slots[4] = -1  # a padded row writes nothing

    def lin(n, heads):
        return (h @ W[n].T + W[n + ".b"]).view(T, heads, -1)

    t = plain.temperature(T, {"coef": 0.5, "every": 8}, torch.float64)
    q, k, v = lin("q", H) * t[:, None, None], lin("k", G), lin("v", G)
    gates = plain.sigmoid(h @ W["g"].T)
    xr = F.linear(h.to(dev, dt).float(), w["in"].float())
    inputs = [xr.to(dt)]
    if dt == torch.bfloat16 or dev == "cpu":
        cuts = torch.rand(3, 1, 1, generator=g).to(dev)
        inputs.append((xr * cuts / cuts.sum()).contiguous())  # slabs
        if dt == torch.bfloat16:
            inputs.append((xr * cuts / cuts.sum()).half().contiguous())
    for x in inputs:
        pages, _ = mod.alloc(6, page, 1)
        gate = torch.full((T, H), float("nan"), device=dev)
        got = mops.gqa_prep(x, w, spec, pages, pos, slots, None, dt, 1e-5, mod.temp, gate)
        assert rel(got.view(T, H, -1)[..., :D], q) < LIMIT[dt]
        assert float(got.view(T, H, -1)[..., D:].float().abs().sum()) == 0
        assert rel(gate, gates) < LIMIT[dt]
        kc = pages[0].cpu().double()[3:5].transpose(1, 2).reshape(2 * page, G, -1)[:T]
        vc = pages[1].cpu().double()[3:5].transpose(1, 2).reshape(2 * page, G, -1)[:T]
        keep = [i for i in range(T) if i != 4]
        assert rel(kc[keep][..., :D], k[keep]) < LIMIT[dt]
        assert rel(vc[keep][..., :V], v[keep]) < LIMIT[dt]
        assert float(kc[4].abs().sum() + vc[4].abs().sum()) == 0


# ------------------------------------------------------------------- scores
class Shaped(Paged):
    """Paged sequences whose scores are capped and biased, heads gated."""

    def __init__(self, run, spec, g, r=None, **kw):
        super().__init__(run, spec, g, **kw)
        self.r = r
        if r is not None:
            self.w["dist"] = r.float().to(self.dev).contiguous()

    def prefill_gated(self, qs, bts, lens, sinks, gates):
        """With a running maximum, and without where scores are bounded."""
        if mops.scores_bounded(self.spec, self.w.get("dist")):
            self.w["bounded"] = True
            a = self._prefill_gated(qs, bts, lens, sinks, gates)
            self.w["bounded"] = False
            b = self._prefill_gated(qs, bts, lens, sinks, gates)
            assert rel(a, b) < (1e-6 if self.dt == torch.float32 else 6e-3)
            return a
        return self._prefill_gated(qs, bts, lens, sinks, gates)

    def _prefill_gated(self, qs, bts, lens, sinks, gates):
        dev = gates.float().to(self.dev).contiguous()
        call = self.mod._prefill
        self.mod._prefill = lambda *a: call(*a, gate=dev)
        try:
            return self.prefill(qs, bts, lens, sinks)
        finally:
            self.mod._prefill = call

    def decode_gated(self, q, bts, lens, sinks, gates, splits=None):
        pos = torch.tensor([n - 1 for n in lens], dtype=torch.int32, device=self.dev)
        bt, qq, dev = self.table(bts), self.q(q), gates.float().to(self.dev).contiguous()
        if splits is not None and self.mod.mfma:
            return self.heads(mops.gqa_decode(qq, self.pages, bt, pos, self.spec, sinks, splits,
                                              dist=self.w.get("dist"), gate=dev))
        return self.heads(self.mod._decode(dict(self.w, sink=sinks), qq, self.pages, bt, pos, None,
                                           dev))


def make_paged(run, spec, g, **kw):
    """Paged with plain tensors only: no projection is used."""
    plain_spec = AttentionSpec(spec.heads, spec.kv_heads, spec.dim, spec.vdim, spec.scale,
                               RotarySpec(2, 1e4), sink="learned")
    r = kw.pop("r", None)
    P = Shaped(run, plain_spec, g, r, **kw)
    P.spec = P.mod.spec = spec
    return P


def dense(q, k, v, spec, r, gates, window=0, keep=0):
    """q [T, H, D] at the last T of the n positions of k, v -> [T, H, V]."""
    T, H = q.shape[:2]
    n, G = k.shape[:2]
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    seen = plain.causal(n) & ((i - j < window) | (j < keep) if window else True)
    out = []
    for h in range(H):
        s = plain.capped(q[:, h] @ k[:, h // (H // G)].T * spec.scale, spec.softcap)
        if r is not None:
            s = s - plain.distance_bias(n, r[0, h], r[1, h])[n - T:]
        p = plain.softmax_one(s.masked_fill(~seen[n - T:], float("-inf")))
        out.append(p @ v[:, h // (H // G)] * gates[:, h:h + 1])
    return torch.stack(out, 1)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("shape,page,cap,dist,window,keep", [
    ("served", 16, 6.0, True, 0, 0), ("served", 32, 2.0, False, 0, 0),
    ("served", 16, 0.0, True, 0, 0), ("ragged", 64, 4.0, True, 0, 0),
    ("whole", 16, 50.0, True, 0, 0), ("group10", 32, 6.0, True, 0, 0),
    ("past", 16, 3.0, True, 0, 0), ("mixed", 8, 5.0, True, 0, 0),
    ("served", 16, 5.0, True, 70, 0), ("whole", 16, 5.0, True, 40, 19)])
def test_shaped_scores(shape, page, cap, dist, window, keep, run):
    """Unequal portions over shuffled pages that hold leftovers; the same rows decoded, in any
    number of parts; caps and biases each alone, together, and under a window."""
    g = gen(4)
    spec = spec_of(shape, cap, dist, temp=None, scale=2.5 * SHAPES[shape][2] ** -0.5,
                   window=window, keep_first=keep)
    H, G, D, V = SHAPES[shape]
    r = torch.stack([0.3 + rnd(H, g=g).abs(), 0.05 + rnd(H, g=g).abs()]) if dist else None
    P = make_paged(run, spec, g, r=r, page=page)
    sinks = torch.zeros(H, device=P.dev)
    lens, nq = [1, 17, 150, 300, 64, 129, 131], [1, 2, 131, 45, 64, 129, 3]
    ks, vs = [rnd(n, G, D, g=g) for n in lens], [rnd(n, G, V, g=g) for n in lens]
    qs = [rnd(m, H, D, g=g) for m in nq]
    gates = [torch.rand(m, H, generator=g, dtype=torch.float64) for m in nq]
    bts = [P.put(k, v) for k, v in zip(ks, vs)]
    want = [dense(*x, window, keep) for x in zip(qs, ks, vs, [spec] * 7, [r] * 7, gates)]
    got, o = P.prefill_gated(qs, bts, lens, sinks, torch.cat(gates)), 0
    for i, w in enumerate(want):
        assert rel(got[o:o + nq[i]], w) < LIMIT[P.dt], (i, lens[i])
        o += nq[i]
    last, ends = torch.stack([q[-1] for q in qs]), torch.stack([x[-1] for x in gates])
    for splits in (None, 1, 2, 5):
        got = P.decode_gated(last, bts, lens, sinks, ends, splits)
        for i in range(len(lens)):
            assert rel(got[i], want[i][-1]) < LIMIT[P.dt], (splits, lens[i])


@pytest.mark.parametrize("run", RUNS)
def test_distance_that_raises_scores(run):
    """Negative biases, and caps past what fp32 exponentials hold, keep the running maximum."""
    g = gen(14)
    r = torch.tensor([[-3.0, 0.5, -0.7, 0.0], [2.0, 0.1, 5.0, 1.0]], dtype=torch.float64)
    for cap, low in ((8.0, False), (300.0, True), (41.0, True), (40.0, True)):
        spec = spec_of((4, 2, 64, 64), cap=cap, scale=2.0, temp=None)
        rr = r.abs() if low else r
        assert mops.scores_bounded(spec, rr) == (low and cap == 40.0)
        P = make_paged(run, spec, g, r=rr)
        n, gates = 200, torch.ones(200, 4, dtype=torch.float64)
        q, k, v = rnd(n, 4, 64, g=g), rnd(n, 2, 64, g=g), rnd(n, 2, 64, g=g)
        if P.dt == torch.bfloat16 and cap > 100:  # sharp scores of rounded products
            q = 0.25 * q
        bt, sinks = P.put(k, v), torch.zeros(4, device=P.dev)
        want = dense(q, k, v, spec, rr, gates)
        lim = {torch.float32: 2e-4, torch.bfloat16: 0.03}[P.dt]
        assert rel(P.prefill_gated([q], [bt], [n], sinks, gates), want) < lim, cap
        d = P.decode_gated(q[-1:], [bt], [n], sinks, gates[:1], 3)
        assert rel(d[0], want[-1]) < lim, cap


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("n", [140, 700])
def test_one_key_that_stands_out(n, run):
    """One key far above all others, near and far away, at page borders and ends of tiles: its
    value is what is left, less what the cap and its distance take."""
    g = gen(5)
    H, G, D, V = 2, 1, 32, 32
    spec = spec_of((H, G, D, V), cap=20.0, scale=1.0, temp=None)
    r = torch.tensor([[0.0, 1.5], [0.3, 0.05]], dtype=torch.float64)
    P = make_paged(run, spec, g, r=r, page=16, blocks=800)
    sinks = torch.zeros(H, device=P.dev)
    gates = torch.ones(n, H, dtype=torch.float64)
    lim = 1e-4 if P.dt == torch.float32 else 0.06
    spots = [0, 1, 15, 16, 17, 31, 32, 63, 64, 65, 127, 128, n - 1]
    for spot in spots if n < 200 else [0, 3, 300]:
        k, v = rnd(n, G, D, g=g, scale=0.01), rnd(n, G, V, g=g)
        q = torch.zeros(n, H, D, dtype=torch.float64)
        q[..., 3] = 8.0
        k[spot, :, 3] = 8.0  # its score is 64, capped close to 20
        v[spot] += 5.0
        bt = P.put(k, v)
        want = dense(q, k, v, spec, r, gates)
        assert n < 200 or float((want[n - 1] - v[spot]).abs().max()) < 0.01  # seen from afar
        at = 77 if n < 200 else 600
        got = P.prefill_gated([q], [bt], [n], sinks, gates)
        part = P.prefill_gated([q[at:]], [bt], [n], sinks, gates[at:])
        assert float((got - want).abs().max()) < lim, spot
        assert float((part - want[at:]).abs().max()) < lim, spot
        for m in sorted({n, spot + 1, min(n, spot + 2), min(n, 129), min(n, 65)}):
            for splits in (1, 3):
                d = P.decode_gated(q[m - 1:m], [bt], [m], sinks, gates[:1], splits)
                assert float((d[0] - want[m - 1]).abs().max()) < lim, (spot, m, splits)
        P.free = bt + P.free


@pytest.mark.parametrize("run", RUNS)
def test_one_in_the_denominator(run):
    """Scores far below zero leave next to nothing of the values, not their mean; the one is
    added once however the keys are split; far above zero it does not show."""
    g = gen(6)
    shape = (4, 2, 64, 64)
    spec = spec_of(shape, cap=25.0, scale=1.0, temp=None)
    r = torch.tensor([[0.0] * 4, [1.0] * 4], dtype=torch.float64)
    P = make_paged(run, spec, g, r=r)
    n, sinks = 200, torch.zeros(4, device=P.dev)
    q, k, v = torch.zeros(n, 4, 64).double(), torch.zeros(n, 2, 64).double(), rnd(n, 2, 64, g=g)
    k[..., 0] = 1.0
    q[..., 0] = torch.tensor([-12.0, -5.0, 0.0, 12.0], dtype=torch.float64)
    gates = torch.ones(n, 4, dtype=torch.float64)
    bt = P.put(k, v)
    want = dense(q, k, v, spec, r, gates)
    assert rel(want[-1, 2], v.mean(0)[1] * n / (n + 1)) < 1e-9
    got = P.prefill_gated([q], [bt], [n], sinks, gates)
    for h in range(4):
        assert rel(got[:, h], want[:, h]) < LIMIT[P.dt], h
        for splits in (1, 2, 7):
            d = P.decode_gated(q[-1:], [bt], [n], sinks, gates[:1], splits)
            assert rel(d[0, h], want[-1, h]) < LIMIT[P.dt], (h, splits)


@GPU
@pytest.mark.parametrize("page", [8, 64])
def test_long_contexts(page):
    """Thousands of keys: parts longer than one score tile, large distances."""
    g = gen(7)
    spec = spec_of((8, 2, 64, 64), cap=8.0, scale=0.3, temp=None)
    r = torch.stack([0.2 * rnd(8, g=g).abs(), rnd(8, g=g).abs()])
    P = make_paged(("cuda", torch.bfloat16), spec, g, r=r, page=page, blocks=6000 // page * 2)
    lens = [5000, 1101, 3]
    ks, vs = [rnd(n, 2, 64, g=g) for n in lens], [rnd(n, 2, 64, g=g) for n in lens]
    qs = [rnd(min(n, 200), 8, 64, g=g) for n in lens]
    gates = [torch.rand(q.shape[0], 8, generator=g, dtype=torch.float64) for q in qs]
    bts = [P.put(k, v) for k, v in zip(ks, vs)]
    sinks = torch.zeros(8, device="cuda")
    want = [dense(*x) for x in zip(qs, ks, vs, [spec] * 3, [r] * 3, gates)]
    assert rel(P.prefill_gated(qs, bts, lens, sinks, torch.cat(gates)), torch.cat(want)) < 0.012
    ends = torch.stack([x[-1] for x in gates])
    for splits in (None, 1, 7):
        d = P.decode_gated(torch.stack([q[-1] for q in qs]), bts, lens, sinks, ends, splits)
        for i in range(3):
            assert rel(d[i], want[i][-1]) < 0.012, (splits, i)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("how", ["whole", "portions", "tokens", "batch"])
@pytest.mark.parametrize("shape", ["served", "ragged", "group10", "past"])
def test_attention_mixer(shape, how, run):
    """The whole mixer: projection, pages, attention, gates, output."""
    dev, dt = run
    g = gen(8)
    spec = spec_of(shape, cap=5.0)
    d = 64
    mod = GroupedQueryAttention(spec, Model(dev, dt, 1e-5))
    W = attention_weights(spec, d, g)
    w = mod.pack(lambda n: W[n].to(dev, dt), d)
    hs = [rnd(n, d, g=g) for n in (70, 41, 33)]
    steps = {"whole": [[(0, 70)], [(1, 41)], [(2, 33)]],
             "portions": [[(s, n)] for s, k in ((0, (2, 31, 37)), (1, (16, 25)), (2, (3, 30)))
                          for n in k],
             "tokens": [[(0, 40), (1, 11), (2, 3)]] + [[(0, 1), (1, 1), (2, 1)]] * 30,
             "batch": [[(0, 70), (1, 20)], [(1, 21), (2, 33)]]}[how]
    m = {"heads": spec.heads, "kv_heads": spec.kv_heads, "dim": spec.dim, "vdim": spec.vdim,
         "scale": spec.scale, "softcap": 5.0, "q_temp": {"coef": 0.5, "every": 8}}
    got = run_mixer(mod, w, hs, steps, 16, 6)
    for h, y in zip(hs, got):
        want = plain.attention(h, m, W.__getitem__)[:y.shape[0]]
        out = F.linear(y.double().cpu(), w["o"].double().cpu())
        assert rel(out, want) < LIMIT[dt]


# ----------------------------------------------------------- latent attention
LATENT = {"served": (8, 128, 64, 128, 96, 256), "ragged": (3, 11, 6, 9, 13, 17),
          "one": (1, 16, 2, 16, 16, 16), "wide": (2, 200, 40, 140, 150, 300),
          "many": (20, 24, 10, 48, 40, 70)}


def latent_case(size, run, g, scale=None, d=64, base=500.0):
    dev, dt = run
    H, D, R, V, Q, C = LATENT[size]
    spec = LatentAttentionSpec(H, D, R, V, Q, C, scale or 1.3 * (D + R) ** -0.5,
                               RotarySpec(R, base, interleaved=True))
    W = {"dq": rnd(Q, d, g=g, scale=d ** -0.5), "dq.norm": 1 + 0.2 * rnd(Q, g=g),
         "uq": rnd(H * (D + R), Q, g=g, scale=1.5 * Q ** -0.5),
         "dkv": rnd(C + R, d, g=g, scale=1.5 * d ** -0.5), "dkv.norm": 1 + 0.2 * rnd(C, g=g),
         "uk": rnd(H * D, C, g=g, scale=C ** -0.5), "uv": rnd(H * V, C, g=g, scale=C ** -0.5),
         "g": rnd(H, d, g=g, scale=d ** -0.5), "o": rnd(d, H * V, g=g)}
    W = {k: v.to(torch.bfloat16).double() for k, v in W.items()}
    mod = LatentAttention(spec, Model(dev, dt, 1e-4))
    w = mod.pack(lambda n: W[n].to(dev, dt), d)
    m = {"heads": H, "dim": D, "rot_dim": R, "vdim": V, "kv_rank": C, "scale": spec.scale,
         "rot": {"base": base, "dims": R}}
    return mod, w, W, m


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("how", ["whole", "portions", "tokens"])
@pytest.mark.parametrize("size", sorted(LATENT))
def test_latent_attention(size, how, run):
    """Neighbours turn together in queries and the shared key part, in both forms of the
    attention (expanded keys, absorbed queries)."""
    g = gen(9)
    mod, w, W, m = latent_case(size, run, g)
    hs = [rnd(n, 64, g=g) for n in (90, 35)]
    steps = {"whole": [[(0, 90)], [(1, 35)]],
             "portions": [[(0, 2)], [(0, 61), (1, 17)], [(0, 27), (1, 18)]],
             "tokens": [[(0, 60), (1, 5)]] + [[(0, 1), (1, 1)]] * 30}[how]
    got = run_mixer(mod, w, hs, steps, 16, 6)
    for h, y in zip(hs, got):
        want = plain.latent_attention(h, m, W.__getitem__, 1e-4)[:y.shape[0]]
        out = F.linear(y.double().cpu(), w["o"].double().cpu())
        assert rel(out, want) < {torch.float32: 3e-5, torch.bfloat16: 0.02}[run[1]]


@pytest.mark.parametrize("run", RUNS)
def test_rotated_parts_alone(run):
    """Scores from the rotated parts only, sharp enough that a pair turned by a neighbour's
    angle, or the wrong way, picks other keys."""
    g = gen(10)
    mod, w, W, m = latent_case("many", run, g, scale=4.0, base=50.0)
    H, D, R, V, Q, C = LATENT["many"]
    W["uq"] = W["uq"].view(H, D + R, Q) * torch.cat([torch.zeros(D), torch.ones(R)])[None, :, None]
    W["uq"] = W["uq"].reshape(H * (D + R), Q)
    w = mod.pack(lambda n: W[n].to(*run), 64)
    h = rnd(80, 64, g=g)
    for steps in ([[(0, 80)]], [[(0, 50)]] + [[(0, 1)]] * 30):
        got = run_mixer(mod, w, [h], steps, 16, 6)[0]
        want = plain.latent_attention(h, m, W.__getitem__, 1e-4)
        halves = dict(W, uq=W["uq"], dkv=torch.cat([W["dkv"][:C], W["dkv"][C:].flip(0)]))
        assert rel(plain.latent_attention(h, m, halves.__getitem__, 1e-4), want) > 0.2
        assert rel(F.linear(got.double().cpu(), w["o"].double().cpu()), want) < {
            torch.float32: 1e-4, torch.bfloat16: 0.08}[run[1]]


# ---------------------------------------------------------------- experts
def routed(run, h, router, bias, top):
    dev, dt = run
    spec = ExpertsSpec(ff=64, experts=router.shape[0], top=top, score="softmax", renorm=True,
                       expert="glu", router_bias=True)
    if dev == "cpu":
        from omnia_amd.ops import reference_mixers as ref

        return ref.route(h.to(dt), router.to(dt), spec, None, bias.float())
    from omnia_amd.ops import kernels

    T = h.shape[0]
    ids = torch.empty(T, top, dtype=torch.int32, device=dev)
    wts = torch.empty(T, top, device=dev)
    kernels().moe_route(ids, wts, h.to(dev, dt), router.to(dev, dt), top, False, True, None, 1, 1,
                        bias.float().to(dev))
    return ids.cpu(), wts.cpu()


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("E,top,shift", [(8, 2, 0.0), (5, 5, -3.0), (1, 1, 2.0), (70, 6, 50.0),
                                         (200, 3, -80.0), (16, 1, 0.0), (64, 8, 0.0)])
def test_biased_routing(E, top, shift, run):
    """The bias is part of the logits: it chooses and weighs; weights are a softmax over the
    chosen logits alone, whatever all of them have in common."""
    g = gen(E + top)
    d = 96
    router, bias = rnd(E, d, g=g, scale=0.3), 1.5 * rnd(E, g=g) + shift
    h = rnd(300, d, g=g)
    z = (h @ router.T + bias).sort(-1, descending=True).values
    if E > 1:
        h = h[(z[:, :-1] - z[:, 1:])[:, :top].min(-1).values > 2e-4][:61]
    ids, wts = plain.route(h, router, bias, top)
    got, w = routed(run, h, router, bias, top)
    assert torch.equal(got.long(), ids) and rel(w, wts) < 1e-5
    if 1 < top < E:
        plain_ids, _ = plain.route(h, router, torch.zeros(E).double(), top)
        assert not torch.equal(plain_ids.sort(-1).values, ids.sort(-1).values)


def run_experts(run, E, top, d, ff, shared, T, seed=8, decode=False):
    """(framework's parts summed [T, d], plain): inputs without a close call."""
    dev, dt = run
    g = gen(seed)
    spec = ExpertsSpec(ff=ff, experts=E, top=top, score="softmax", renorm=True, expert="glu",
                       router_bias=True, shared=DenseMLPSpec(shared, bias=False))
    W = {"router": rnd(E, d, g=g, scale=d ** -0.5), "router.b": rnd(E, g=g)}
    for n, f in [(f"e{e}", ff) for e in range(E)] + [("shared", shared)]:
        W.update({n + ".gate": rnd(f, d, g=g, scale=2 * d ** -0.5),
                  n + ".up": rnd(f, d, g=g, scale=d ** -0.5),
                  n + ".down": rnd(d, f, g=g, scale=f ** -0.5)})
    h = rnd(4 * T + 64, d, g=g)
    z = (h @ W["router"].T + W["router.b"]).sort(-1, descending=True).values
    if top < E:
        h = h[z[:, top - 1] - z[:, top] > 1e-3]
    h = h[:T].contiguous()
    assert h.shape[0] == T

    class M(Model):
        tp, tpr, use_pgemm, splitk_half = 1, 0, False, True

        def _pgemm_ok(self, *a):
            return False

        def _wcfg(self, *a):
            return None

    mod = Experts(spec, M(dev, dt, 1e-5))
    dp = -(-d // 64) * 64
    w = mod.pack(lambda n: W[n].to(dev, dt), dp)
    out = mod.forward(w, pad(h, dp).to(dev, dt), decode)
    assert out["slots"] and out["m"].shape == (T, top, dp)
    got = out["m"].double().cpu().sum(1) + out["shared"].double().cpu()
    assert float(got[:, d:].abs().sum()) == 0
    mlp = {"router": {"top": top}, "shared": {"ff": shared}}
    return got[:, :d], plain.experts(h, mlp, W.__getitem__)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("E,top,d,ff,shared,T", [
    (8, 2, 128, 64, 128, 40), (5, 5, 72, 27, 21, 33), (1, 1, 64, 64, 64, 3),
    (70, 6, 48, 16, 200, 50), (200, 3, 64, 8, 8, 9), (16, 1, 256, 192, 64, 65),
    (3, 2, 100, 130, 5, 1)])
def test_experts_beside_a_shared_one(E, top, d, ff, shared, T, run):
    got, want = run_experts(run, E, top, d, ff, shared, T)
    assert rel(got, want) < LIMIT[run[1]]


@GPU
@pytest.mark.parametrize("d", [256, 512])
def test_experts_on_the_prefill_tile(d):
    """Enough rows per expert for the 256x256 tile (bf16); a ragged last segment."""
    run = ("cuda", torch.bfloat16)
    got, want = run_experts(run, 2, 1, d, 128, 256, 1100)
    assert rel(got, want) < 0.012
    got, want = run_experts(run, 3, 2, d, 256, 128, 900)
    assert rel(got, want) < 0.012


def test_plain_pieces():
    """The oracle's own arithmetic on numbers worked out by hand."""
    assert plain.softmax_one(torch.zeros(1, 3))[0].tolist() == [0.25] * 3
    assert float(plain.capped(torch.tensor(3.0), 2.0)) == pytest.approx(2 * math.tanh(1.5))
    one = torch.tensor(1.0, dtype=torch.float64)
    assert plain.distance_bias(3, 2 * one, 3 * one)[2].tolist() == pytest.approx(
        [2 * math.log(7), 2 * math.log(4), 0.0])
    assert plain.temperature(5, {"coef": 2.0, "every": 2}, torch.float64).tolist() == \
        pytest.approx([1.0] + [1 + 2 * math.log(2)] * 2 + [1 + 2 * math.log(3)] * 2)
    ids, w = plain.route(torch.zeros(1, 2), torch.zeros(3, 2), torch.tensor([0.0, 1.0, 3.0]), 2)
    assert ids.tolist() == [[2, 1]] and float(w[0, 0]) == pytest.approx(1 / (1 + math.exp(-2)))
    x = torch.tensor([[1.0, 0.0, 0.0, 2.0]] * 2, dtype=torch.float64)
    y = plain.rotate(x, 100.0)[1]
    assert y.tolist() == pytest.approx([math.cos(1), math.sin(1), -2 * math.sin(0.1),
                                        2 * math.cos(0.1)])
