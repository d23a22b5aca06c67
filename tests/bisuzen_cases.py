"""Small Bisuzen models (own sizes, random weights) shared by the CPU and GPU tests.  The
oracle is :mod:`plain_bisuzen`; the drivers are those of the other layer-list families."""
import math

import plain_bisuzen as plain
import torch
from sivadra_cases import cut, error, replay, save, tokens  # noqa: F401


def window(heads=4, kv_heads=2, dim=24, vdim=40, rot=12, size=37, keep=3, base=10000.0,
           scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "scale": scale or 1.4 * dim ** -0.5, "rot": {"base": base, "dims": rot},
            "mask": {"size": size, "keep_first": keep}}


def linear(dim, vdim, decay):
    return {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}


def parallel(left, right, mlp=None):
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": mlp}


def chunked(heads=4, kv_heads=2, dim=16, vdim=24, size=29, scale=None, mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                      "scale": scale or 2.0 * dim ** -0.5, "mask": {"size": size}}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, groups=(1, 1), identity=0):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "identity": identity,
                       "groups": {"count": groups[0], "keep": groups[1]}}}


def model(layers, width=72, vocab=90, eps=1e-5, scale=0.6, loop=None):
    c = {"architecture": "Bisuzen", "width": width, "vocab": vocab, "norm": {"eps": eps},
         "layers": layers, "logit_scale": scale}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


CASES = {
    # every kind of layer, two of them looped
    "mixed": model([
        parallel(window(heads=6, size=37, keep=5), linear(20, 28, (0.5, 0.97, 0.9995)),
                 moe(40, 6, 2, (4, 2), 2)),
        chunked(mlp=dense(56)),
        parallel(window(size=64, keep=33, rot=24), linear(16, 16, (0.9,))),
        chunked(heads=3, kv_heads=1, dim=32, vdim=32, size=64, mlp=moe(24, 4, 3))],
        loop=(0, 2, 2)),
    # odd sizes: nothing a multiple of 8; identity experts outside a whole group
    "odd": model([
        parallel(window(heads=3, kv_heads=1, dim=22, vdim=13, rot=6, size=33, keep=1),
                 linear(9, 11, (0.8, 0.99)), moe(27, 5, 3, (3, 2), 1)),
        chunked(heads=3, kv_heads=3, dim=10, vdim=7, size=17, mlp=dense(35))],
        width=45, vocab=71, eps=1e-3, loop=(1, 2, 3)),
    # equal and smallest sizes: windows and chunks of one token, decays 0 and 1, one expert,
    # a loop that runs once
    "ones": model([
        parallel(window(heads=2, kv_heads=2, dim=16, vdim=16, rot=16, size=1, keep=1),
                 linear(16, 16, (0.0, 1.0)), moe(32, 1, 1)),
        chunked(heads=1, kv_heads=1, dim=8, vdim=8, size=1, mlp=moe(16, 1, 2, (1, 1), 1))],
        width=32, vocab=64, scale=1.0, loop=(0, 1, 1)),
    # more experts than a wave has lanes, ten query heads on a key head, more kept keys than
    # the window holds
    "many": model([
        parallel(window(heads=20, kv_heads=2, dim=32, vdim=64, rot=8, size=31, keep=40),
                 linear(32, 64, (0.6, 0.8, 0.95, 0.99, 0.999)), moe(16, 63, 5, (10, 4), 7)),
        chunked(heads=6, kv_heads=2, dim=64, vdim=32, size=33,
                mlp=moe(72, 20, 9, (12, 6), 4))], width=80, vocab=110),
    # heads past the MFMA widths and between them, no feed-forward at all
    "wide": model([
        parallel(window(heads=4, kv_heads=4, dim=136, vdim=130, rot=64, size=45, keep=2),
                 linear(72, 200, (0.9, 0.99))),
        parallel(window(heads=2, kv_heads=1, dim=300, vdim=260, rot=100, size=70, keep=20),
                 linear(300, 260, (0.95,))),
        chunked(heads=5, kv_heads=1, dim=64, vdim=96, size=40),
        chunked(heads=2, kv_heads=1, dim=280, vdim=264, size=70)], width=120, vocab=100),
    # sizes the prefill tiles take (long prompts), heads of a served shape
    "tile": model([
        parallel(window(heads=8, kv_heads=2, dim=128, vdim=128, rot=64, size=300, keep=70),
                 linear(128, 128, (0.5, 0.95, 0.995, 0.9995)), moe(256, 2, 1)),
        chunked(heads=4, kv_heads=2, dim=64, vdim=64, size=700, mlp=dense(512)),
        parallel(window(heads=4, kv_heads=4, dim=64, vdim=64, rot=32, size=900, keep=4),
                 linear(64, 64, (0.9, 0.999)), moe(256, 3, 2, (2, 1), 1))],
        width=512, vocab=256),
}

CODES = 8  # residual channels the routers read in whole-model tests


def _stable(cfg, W, codes, g):
    """[n] bool: every router chooses the same experts for a code however its input is
    rounded.  No sublayer adds to the code channels but the identity experts, which are
    followed here."""
    n = codes.shape[0]
    ok = torch.ones(n, dtype=torch.bool)
    x = codes.clone()
    for i in plain.order(cfg):
        mlp = cfg["layers"][i].get("mlp")
        if not mlp or mlp["kind"] != "moe":
            continue
        p, r = f"l{i}.", mlp["router"]
        router, corr = W[p + "mlp.router"][:, -CODES:], W[p + "mlp.correction"]
        h = plain.tanh_norm(x, W[p + "norm2.alpha"], 1.0, 0.0)

        def chosen(v):
            ids, w = plain.route(v, router, corr, r["top"], r["groups"]["count"],
                                 r["groups"]["keep"])
            return torch.zeros(n, corr.numel(), dtype=torch.float64).scatter_(1, ids, w)

        w = chosen(h)
        for _ in range(5):
            noise = 2.0 * torch.rand(h.shape, generator=g, dtype=torch.float64) - 1.0
            ok &= ((chosen(h * (1.0 + noise / 64)) > 0) == (w > 0)).all(1)
        x = x + w[:, r["experts"]:].sum(1, keepdim=True) * h
    return ok


def weights(cfg, seed=0):
    """name -> float64 tensor, bf16-representable.  The last ``CODES`` channels carry a code
    of the token through the whole model; the routers read those."""
    from omnia_amd.models.layers import DESIGNS, parse_layers, tensor_shapes

    g = torch.Generator().manual_seed(seed)
    W = {}

    def rnd(shape):
        return torch.randn(shape, generator=g, dtype=torch.float64)

    d = DESIGNS["bisuzen"]
    for n, shape in tensor_shapes(parse_layers(cfg["layers"], d, cfg.get("loop")), cfg["width"],
                                  cfg["vocab"], d).items():
        leaf = n.split(".")[-1]
        if leaf == "alpha":
            t = 0.4 + 0.5 * torch.rand(shape, generator=g, dtype=torch.float64)
        elif leaf == "sink":
            t = 1.5 * rnd(shape)
        elif leaf == "correction":  # choice scores of both signs
            t = 0.3 * rnd(shape) / shape[0] ** 0.5 - 1.0 / shape[0]
        elif leaf == "b":
            t = (0.1 if ".norm" in n else 0.3) * rnd(shape)
        elif leaf in ("norm1", "norm2", "norm", "out"):
            t = 1.0 + 0.2 * rnd(shape)
        elif leaf == "router":
            t = torch.zeros(shape, dtype=torch.float64)
            t[:, -CODES:] = rnd((shape[0], CODES)) * (3.0 if shape[0] > 16 else 1.5)
        elif n == "embed":
            t = rnd(shape)
        else:
            t = rnd(shape) * 1.5 / math.sqrt(shape[1])
        # what sublayers leave alone, and the norm the routers read through
        if leaf == "out":
            t[-CODES:] = 0.0
        elif leaf in ("o", "down"):
            t[-CODES:] = 0.0
        elif leaf == "norm2":
            t[-CODES:] = 1.0
        elif n.endswith("norm2.b"):
            t[-CODES:] = 0.0
        W[n] = t.to(torch.bfloat16).double()
    todo = torch.arange(cfg["vocab"])
    for _ in range(400):
        c = rnd((todo.numel(), CODES)).to(torch.bfloat16).double()
        ok = _stable(cfg, W, c, g)
        W["embed"][todo[ok], -CODES:] = c[ok]
        todo = todo[~ok]
        if not todo.numel():
            break
    assert not todo.numel()
    return W


_ORACLE: dict = {}


def oracle(key, cfg, W, toks):
    k = (key, tuple(toks))
    if k not in _ORACLE:
        _ORACLE[k] = plain.forward(cfg, W, toks)
    return _ORACLE[k]
