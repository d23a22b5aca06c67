"""Small Sekazen models (own sizes, random weights) shared by the CPU and GPU tests.  The
oracle is :mod:`plain_sekazen`; the drivers are those of the other layer-list family."""
import math

import plain_sekazen as plain
import torch
from sivadra_cases import cut, error, replay, save, tokens  # noqa: F401


def attn(heads=4, kv_heads=2, dim=24, vdim=40, rot=12, window=None, bands=None, base=10000.0,
         scale=None, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "scale": scale or 1.4 * dim ** -0.5, "rot": {"base": base, "dims": rot}}
    if bands:
        m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), bands))
    if window:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": None}


def moe(layer, ff, experts, top, limit=1.2):
    return {**layer, "mlp": {"kind": "moe", "expert": {"ff": ff, "limit": limit},
                             "router": {"experts": experts, "top": top}}}


def borrow(layers, j, window=None, scale=None):
    m = dict(layers[j]["mixer"], kv_from=j)
    m.pop("mask", None)
    if window:
        m["mask"] = {"size": window}
    if scale:
        m["scale"] = scale
    return {"type": "attention", "mixer": m, "mlp": None}


def model(layers, width=72, vocab=90, eps=1e-5, cap=12.0):
    c = {"architecture": "Sekazen", "width": width, "vocab": vocab, "norm": {"eps": eps},
         "layers": layers}
    if cap:
        c["logit_softcap"] = cap
    return c


def _mixed():
    ls = [moe(attn(window=37, bands=(4.0, 1.0, 4.0, 64)), 56, 6, 2)]
    ls.append(moe(borrow(ls, 0, window=20, scale=0.4), 40, 5, 1))
    ls.append(attn(heads=6, kv_heads=2, dim=32, vdim=16, rot=32))  # sees everything
    ls.append(moe(borrow(ls, 2, window=50), 24, 4, 3))
    ls.append(borrow(ls, 0, window=64))
    return model(ls)


def _wide():
    ls = [attn(heads=4, kv_heads=4, dim=136, vdim=130, rot=64, window=45)]
    ls.append(moe(attn(heads=2, kv_heads=1, dim=300, vdim=260, rot=100, window=70), 48, 3, 2))
    ls.append(borrow(ls, 1, window=30))
    ls.append(attn(heads=5, kv_heads=1, dim=64, vdim=96, rot=2, window=40))
    return model(ls, width=120, vocab=100)


CASES = {
    # borrowed keys with other windows and scales, an unlimited layer, layers without experts
    "mixed": _mixed(),
    # odd sizes: nothing a multiple of 8, one key head, a window of one page and one
    "odd": model([moe(attn(heads=3, kv_heads=1, dim=22, vdim=13, rot=6, window=33), 27, 5, 3)],
                 width=45, vocab=71, eps=1e-3),
    # equal sizes, everything rotated, window 1 (a token sees itself), one expert
    "ones": model([moe(attn(heads=2, kv_heads=2, dim=16, vdim=16, rot=16, window=1), 32, 1, 1),
                   attn(heads=2, kv_heads=2, dim=16, vdim=16, rot=16, window=1)],
                  width=32, vocab=64, cap=None),
    # more experts than a wave has lanes, ten query heads on a key head
    "many": model([moe(attn(heads=20, kv_heads=2, dim=32, vdim=64, rot=8, window=31), 16, 70, 5),
                   moe(attn(heads=6, kv_heads=2, dim=64, vdim=32, rot=64, window=64), 72, 9, 9)],
                  width=80, vocab=110),
    # heads past the MFMA widths and between them
    "wide": _wide(),
    # sizes the 256x256 grouped prefill tile takes (long prompts), heads of a served shape
    "tile": model([moe(attn(heads=8, kv_heads=2, dim=128, vdim=128, rot=64, window=300,
                            bands=(8.0, 1.0, 4.0, 512)), 128, 2, 1),
                   moe(attn(heads=4, kv_heads=2, dim=64, vdim=64, rot=64), 256, 2, 2)],
                  width=512, vocab=256),
}

CODES = 8  # residual channels the routers read in whole-model tests
MARGIN = 0.08


def _codes(cfg, routers, g):
    """One code per vocabulary entry whose chosen experts are chosen clearly by every
    router, so that no 16-bit rounding turns a choice."""
    out = []
    for _ in range(cfg["vocab"]):
        for _ in range(4000):
            c = torch.randn(CODES, generator=g, dtype=torch.float64).to(torch.bfloat16).double()
            ok = True
            for r, top in routers:
                z = (r @ c).sort(descending=True).values
                ok &= top == z.numel() or float(z[top - 1] - z[top]) > MARGIN * float(c.norm())
            if ok:
                break
        assert ok
        out.append(c)
    return torch.stack(out)


def weights(cfg, seed=0):
    """name -> float64 tensor, bf16-representable.  The last ``CODES`` channels carry a code
    of the token through the whole model (no sublayer adds to them); the routers read
    those."""
    from omnia_amd.models.layers import DESIGNS, parse_layers, tensor_shapes

    g = torch.Generator().manual_seed(seed)
    W, routers = {}, []

    def rnd(shape):
        return torch.randn(shape, generator=g, dtype=torch.float64)

    for n, shape in tensor_shapes(parse_layers(cfg["layers"], DESIGNS["sekazen"]), cfg["width"], cfg["vocab"],
                                  DESIGNS["sekazen"]).items():
        leaf = n.split(".")[-1]
        if leaf == "sink":
            t = 1.5 * rnd(shape)
        elif n == "final.norm" or n == "embed.norm":
            t = 0.2 * rnd(shape)
        elif leaf in ("norm1", "norm2"):
            t = 0.2 * rnd(shape)
            t[-CODES:] = -1.0
        elif leaf == "norm":
            t = 1.0 + 0.2 * rnd(shape)
        elif leaf == "router":
            t = torch.zeros(shape, dtype=torch.float64)
            t[:, -CODES:] = rnd((shape[0], CODES)) * (3.0 if shape[0] > 16 else 1.0)
        elif n == "embed":
            t = rnd(shape)
        else:
            t = rnd(shape) * 1.5 / math.sqrt(shape[1])
        W[n] = t.to(torch.bfloat16).double()
        if leaf == "router":
            top = cfg["layers"][int(n[1:].split(".")[0])]["mlp"]["router"]["top"]
            routers.append((W[n][:, -CODES:], top))
    W["embed.norm"][-CODES:] = 0.0
    W["embed"][:, -CODES:] = _codes(cfg, routers, g)
    return W


_ORACLE: dict = {}


def oracle(key, cfg, W, toks):
    k = (key, tuple(toks))
    if k not in _ORACLE:
        _ORACLE[k] = plain.forward(cfg, W, toks)
    return _ORACLE[k]
