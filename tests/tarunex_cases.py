"""Small Tarunex models (own sizes, random weights) shared by the CPU and GPU tests.  The
oracle is :mod:`plain_tarunex`; the drivers are those of the other layer-list families."""
import math

import plain_tarunex as plain
import torch
from sivadra_cases import cut, error, replay, save, tokens  # noqa: F401


def moe(ff, experts, top, shared):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top},
            "shared": {"ff": shared}}


def attention(heads=4, kv_heads=2, dim=24, vdim=40, cap=9.0, coef=0.4, every=19, scale=None,
              mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                      "scale": scale or 1.6 * dim ** -0.5, "softcap": cap,
                      "q_temp": {"coef": coef, "every": every}}}


def latent(heads=3, dim=20, rot=8, vdim=28, q_rank=36, kv_rank=44, base=10000.0, scale=None,
           mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
                      "q_rank": q_rank, "kv_rank": kv_rank,
                      "scale": scale or 1.4 * (dim + rot) ** -0.5,
                      "rot": {"base": base, "dims": rot}}}


def model(layers, width=72, vocab=90, eps=1e-5, embed=3.0, scale=0.6, cap=7.0, loop=None):
    c = {"architecture": "Tarunex", "width": width, "vocab": vocab, "norm": {"eps": eps},
         "embedding": {"scale": embed}, "layers": layers, "logit_scale": scale,
         "logit_softcap": cap}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


CASES = {
    # both mixers, two looped layers between others, a layer without a feed-forward
    "mixed": model([
        attention(heads=6, mlp=moe(40, 6, 2, 56)),
        attention(heads=4, kv_heads=1, dim=40, vdim=24, cap=5.0, every=50, mlp=moe(24, 4, 3, 16)),
        latent(mlp=moe(40, 5, 1, 72)),
        latent(heads=4, dim=32, rot=16, vdim=32, q_rank=64, kv_rank=96)], loop=(1, 3, 2)),
    # odd sizes: nothing a multiple of 8; the loop starts with the first layer
    "odd": model([
        latent(heads=1, dim=11, rot=6, vdim=9, q_rank=13, kv_rank=17, base=300.0,
               mlp=moe(27, 5, 3, 21)),
        attention(heads=3, kv_heads=1, dim=22, vdim=13, cap=3.0, coef=0.9, every=7,
                  mlp=moe(35, 3, 2, 9))], width=45, vocab=71, eps=1e-3, embed=0.7,
        loop=(0, 2, 3)),
    # equal and smallest sizes: one head, one expert, factors of 1, every pass once
    "ones": model([
        attention(heads=1, kv_heads=1, dim=16, vdim=16, cap=40.0, coef=0.25, every=1, scale=1.0,
                  mlp=moe(16, 1, 1, 16)),
        latent(heads=2, dim=16, rot=2, vdim=16, q_rank=16, kv_rank=16, mlp=moe(32, 2, 2, 32))],
        width=32, vocab=64, embed=1.0, scale=1.0, cap=30.0, loop=(1, 2, 1)),
    # more experts than a wave has lanes, ten query heads on a key head, no loop, no cap on
    # scores or logits
    "many": model([
        attention(heads=20, kv_heads=2, dim=32, vdim=64, cap=None, every=31,
                  mlp=moe(16, 70, 5, 24)),
        latent(heads=20, dim=8, rot=4, vdim=8, q_rank=32, kv_rank=32, mlp=moe(24, 20, 9, 8))],
        width=80, vocab=110, cap=None),
    # heads past the MFMA widths and between them; the loop ends with the last layer
    "wide": model([
        attention(heads=4, kv_heads=4, dim=136, vdim=130, mlp=moe(72, 4, 2, 40)),
        attention(heads=2, kv_heads=1, dim=300, vdim=260, cap=20.0),
        latent(heads=2, dim=200, rot=40, vdim=140, q_rank=150, kv_rank=300),
        latent(heads=5, dim=96, rot=32, vdim=90, q_rank=100, kv_rank=130)],
        width=120, vocab=100, loop=(2, 4, 2)),
    # sizes the prefill tiles take (long prompts), heads of a served shape
    "tile": model([
        attention(heads=8, kv_heads=2, dim=128, vdim=128, every=500, mlp=moe(256, 2, 1, 512)),
        latent(heads=4, dim=128, rot=64, vdim=128, q_rank=128, kv_rank=256,
               mlp=moe(256, 3, 2, 256)),
        attention(heads=4, kv_heads=4, dim=64, vdim=64, cap=15.0, every=300)],
        width=512, vocab=256, loop=(1, 2, 2)),
}

CODES = 8  # residual channels the routers read in whole-model tests, and nothing else does


def _inputs(cfg, W, toks):
    """Per layer run: (layer, times the embedding is in the residual, smallest and largest
    1 / rms over the tokens) of a routed layer."""
    trace: list = []
    plain.forward(cfg, W, toks, trace)
    x0 = W["embed"][torch.tensor(toks)] * cfg["embedding"]["scale"]
    out, k, x = [], 1, x0
    for at, (i, t) in enumerate(plain.passes(cfg)):
        if t is not None:
            x = x + (x0 if t else 0.0) + W["loop.step"][t]
            k += t > 0
        r = 1.0 / torch.sqrt((x * x).mean(-1) + cfg["norm"]["eps"])
        if cfg["layers"][i].get("mlp"):
            out.append((i, k, float(r.min()), float(r.max())))
        x = trace[at]
    return out


def _stable(cfg, W, runs, codes, g):
    """[n] bool: every router chooses the same experts for a code wherever 1 / rms lies in
    (a wider interval than) the one seen, and however its input is rounded."""
    ok = torch.ones(codes.shape[0], dtype=torch.bool)
    for i, k, lo, hi in runs:
        p, top = f"l{i}.", cfg["layers"][i]["mlp"]["router"]["top"]
        router, bias = W[p + "mlp.router"][:, -CODES:], W[p + "mlp.router.b"]
        x = codes * k * cfg["embedding"]["scale"] * float(W[p + "norm2"])

        def chosen(v):
            ids, _ = plain.route(v, router, bias, top)
            return torch.zeros(v.shape[0], bias.numel()).scatter_(1, ids, 1.0)

        want = chosen(x * lo)
        for s in torch.logspace(math.log10(lo / 1.25), math.log10(hi * 1.25), 6).tolist():
            noise = 2.0 * torch.rand(x.shape, generator=g, dtype=torch.float64) - 1.0
            ok &= (chosen(x * s * (1.0 + noise / 100)) == want).all(1)
    return ok


def weights(cfg, seed=0):
    """name -> float64 tensor, bf16-representable.  The last ``CODES`` channels carry a code
    of the token, of one length for all, through the whole model; the routers read those."""
    from omnia_amd.models.layers import DESIGNS, parse_layers, tensor_shapes

    g = torch.Generator().manual_seed(seed)
    W = {}

    def rnd(shape):
        return torch.randn(shape, generator=g, dtype=torch.float64)

    def codes(n):
        c = rnd((n, CODES))
        return (2.0 * c / c.norm(dim=1, keepdim=True)).to(torch.bfloat16).double()

    d = DESIGNS["tarunex"]
    for n, shape in tensor_shapes(parse_layers(cfg["layers"], d, cfg.get("loop")), cfg["width"],
                                  cfg["vocab"], d).items():
        leaf = n.split(".")[-1]
        if leaf in ("norm1", "norm2") or n == "final.norm":
            t = 0.8 + 0.5 * torch.rand(shape, generator=g, dtype=torch.float64)
        elif leaf == "norm":
            t = 1.0 + 0.2 * rnd(shape)
        elif leaf in ("r1", "r2"):
            t = 0.1 + torch.rand(shape, generator=g, dtype=torch.float64)
        elif leaf == "b":
            t = 0.3 * rnd(shape)
        elif leaf == "router":
            t = torch.zeros(shape, dtype=torch.float64)
            t[:, -CODES:] = rnd((shape[0], CODES)) * (3.0 if shape[0] > 16 else 1.5)
        elif n == "embed":
            t = rnd(shape)
        elif n == "loop.step":
            t = 0.7 * rnd(shape)
            t[:, -CODES:] = 0.0
        else:
            t = rnd(shape) * 1.5 / math.sqrt(shape[1])
            if shape[1] == cfg["width"]:
                t[:, -CODES:] = 0.0
        if leaf in ("o", "down"):
            t[-CODES:] = 0.0
        W[n] = t.to(torch.bfloat16).double()
    W["embed"][:, -CODES:] = codes(cfg["vocab"])
    runs = _inputs(cfg, W, tokens(cfg, 60, 99))
    todo = torch.arange(cfg["vocab"])
    for _ in range(3000):
        c = codes(todo.numel())
        ok = _stable(cfg, W, runs, c, g)
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
