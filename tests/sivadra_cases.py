"""Small Sivadra models (own sizes, random weights) and drivers shared by the CPU and
GPU tests.  The oracle is :mod:`plain_sivadra`; models reach the framework the way a
user's do, as a checkpoint folder."""
import json
import math
import os

import plain_sivadra as plain
import torch


def latent(heads=4, dim=20, rot=8, vdim=24, q_rank=28, kv_rank=36, window=None, scaling=None,
           base=10000.0, scale=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank,
         "kv_rank": kv_rank, "scale": scale or 1.3 * (dim + rot) ** -0.5,
         "rot": {"base": base, "dims": rot}}
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if window:
        m["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": m}


def delta(heads=4, kv_heads=2, dim=12, vdim=20, conv=3):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                                       "vdim": vdim, "conv": conv}}


def with_mlp(layer, ff):
    return {**layer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model(layers, width=48, vocab=90, eps=1e-5):
    return {"architecture": "Sivadra", "width": width, "vocab": vocab, "norm": {"eps": eps},
            "layers": layers}


def shared(of, layers):
    return {**layers[of], "weights_of": of}


def _mixed():
    ls = [with_mlp(delta(), None), with_mlp(latent(window=37, scaling=(4.0, 64, 20.0, 2.0)), 56),
          with_mlp(delta(heads=6, kv_heads=2, dim=16, vdim=16, conv=4), 40)]
    ls.append(shared(1, ls))
    ls.append(shared(0, ls))
    ls.append(with_mlp(latent(heads=3, dim=32, rot=16, vdim=40, q_rank=24, kv_rank=64), None))
    return model(ls)


CASES = {
    # every mechanism, shared tensors, a windowed and an unlimited attention
    "mixed": _mixed(),
    # odd sizes: nothing a multiple of 8; one head; 2 taps; window of one page and one
    "odd": model([with_mlp(delta(heads=3, kv_heads=1, dim=9, vdim=13, conv=2), 27),
                  with_mlp(latent(heads=1, dim=11, rot=6, vdim=9, q_rank=13, kv_rank=17,
                                  window=33), 30)], width=45, vocab=71, eps=1e-3),
    # equal sizes, single tap (no convolution state), window 1 (a token sees itself)
    "ones": model([with_mlp(delta(heads=2, kv_heads=2, dim=16, vdim=16, conv=1), 32),
                   with_mlp(latent(heads=2, dim=16, rot=2, vdim=16, q_rank=16, kv_rank=16,
                                   window=1), 32)], width=32, vocab=64),
    "recurrent": model([with_mlp(delta(heads=4, kv_heads=4, dim=32, vdim=8, conv=5), None),
                        with_mlp(delta(heads=4, kv_heads=1, dim=8, vdim=32, conv=4), 24)]),
    # widths the 256x256 prefill GEMM takes (long prompts), heads of the served shape
    "tile": model([with_mlp(delta(heads=4, kv_heads=2, dim=64, vdim=64, conv=4), 256),
                   with_mlp(latent(heads=4, dim=64, rot=32, vdim=64, q_rank=128, kv_rank=160,
                                   window=300, scaling=(4.0, 512, 32.0, 1.0)), 384)],
                  width=256, vocab=256),
    "attention": model([with_mlp(latent(heads=5, window=20), 40),
                        with_mlp(latent(heads=20, dim=8, rot=4, vdim=8, window=64), None)]),
}


def weights(cfg, seed=0):
    """name -> float64 tensor, bf16-representable."""
    from omnia_amd.models.layers import DESIGNS, parse_layers, tensor_shapes

    g = torch.Generator().manual_seed(seed)
    W = {}
    for n, shape in tensor_shapes(parse_layers(cfg["layers"], DESIGNS["sivadra"]), cfg["width"],
                                  cfg["vocab"]).items():
        t = torch.randn(shape, generator=g, dtype=torch.float64)
        leaf = n.split(".")[-1]
        if leaf == "alpha":
            t = 0.4 + 0.5 * torch.rand(shape, generator=g, dtype=torch.float64)
        elif leaf == "A_log":
            t = 0.5 * t - 0.5
        elif leaf == "dt_bias":
            t = t - 1.0
        elif leaf.startswith("norm") or n.startswith("final") or n.endswith(".norm"):
            t = 0.1 * t if leaf == "b" else 1.0 + 0.2 * t
        elif n.startswith("embed"):
            pass
        elif leaf == "conv":
            t = t * shape[1] ** -0.5
        elif leaf == "b" and len(shape) == 1:
            t = 0.3 * t
        else:
            t = t * 1.5 / math.sqrt(shape[1])
        W[n] = t.to(torch.bfloat16).double()
    return W


def save(cfg, W, path):
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in W.items()},
              os.path.join(path, "model.safetensors"))
    return str(path)


_ORACLE: dict = {}


def oracle(key, cfg, W, tokens):
    k = (key, tuple(tokens))
    if k not in _ORACLE:
        _ORACLE[k] = plain.forward(cfg, W, tokens)
    return _ORACLE[k]


def tokens(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def error(got, want):
    """Worst per-position rms error of the logits, relative to the logits' rms."""
    d = got.double() - want
    d = d - d.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()).max())


def replay(path, schedule, dtype, device, max_tokens=512, block_size=32, max_live=4):
    """schedule: steps of [(id, tokens)], None tokens = end of id.  Every position's
    logits per id."""
    from omnia_amd.engine.replay import TraceReplay

    rp = TraceReplay(path, dtype, max_tokens, device, max_live=max_live, block_size=block_size)
    out: dict = {}
    for step in schedule:
        ents = [{"id": i, "tokens": t, "want": list(range(len(t)))} for i, t in step
                if t is not None]
        rows = rp.step(ents, [i for i, t in step if t is None])
        o = 0
        for e in ents:
            n = len(e["tokens"])
            out.setdefault(e["id"], []).append(rows[o:o + n].clone())
            o += n
    return {i: torch.cat(r) for i, r in out.items()}, rp


def cut(toks, sizes):
    """Portions of cycling sizes."""
    out, o, k = [], 0, 0
    while o < len(toks):
        n = sizes[k % len(sizes)]
        out.append(toks[o:o + n])
        o, k = o + n, k + 1
    return out
