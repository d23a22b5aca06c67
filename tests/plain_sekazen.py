"""Plain, slow implementation of the Sekazen design: one function per mechanism, whole
sequences, no cache, one token and one expert at a time where that is clearest.

It is the oracle of the Sekazen tests and shares no code with ``omnia_amd``.
A model is a JSON-like config dict plus a flat ``name -> tensor`` dict in the
checkpoint's naming; everything is computed in the dtype of ``W`` (float32 or
float64)."""
import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_one_plus(x, w, eps):
    """RMS norm whose stored weight is the departure from one."""
    return rms(x, eps) * (1.0 + w)


def frequencies(rot):
    """Angle per position of every rotated pair, slow rotations stretched if asked."""
    out = []
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        sc = rot.get("scaling")
        if sc:
            turns = sc["original"] * f / (2.0 * math.pi)  # over the original length
            if turns < sc["low"]:
                f = f / sc["factor"]
            elif turns <= sc["high"]:
                s = (turns - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate(x, rot):
    """x [T, heads, dim]: the first ``dims`` of every head, pairs (i, i + dims/2), turned
    by position times frequency."""
    T, n = x.shape[0], rot["dims"]
    ang = torch.arange(T, dtype=torch.float64)[:, None] * torch.tensor(frequencies(rot),
                                                                      dtype=torch.float64)
    c, s = ang.cos().to(x.dtype)[:, None], ang.sin().to(x.dtype)[:, None]
    u, v = x[..., :n // 2], x[..., n // 2:n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., n:]], -1)


def keys_values(h, m, get, eps):
    """(keys [T, G, dim] normed and rotated, values [T, G, vdim])."""
    T, G = h.shape[0], m["kv_heads"]
    k = rms((h @ get("k").T).view(T, G, m["dim"]), eps) * get("k.norm")
    return rotate(k, m["rot"]), (h @ get("v").T).view(T, G, m["vdim"])


def visible(T, m):
    i = torch.arange(T)
    back = i[:, None] - i[None, :]
    seen = back >= 0
    if m.get("mask"):
        seen = seen & (back < m["mask"]["size"])
    return seen


def sink_softmax(scores, sink):
    """Softmax over the last axis with exp(sink) added to the denominator."""
    top = torch.maximum(scores.max(-1, keepdim=True).values, sink)
    e = torch.exp(scores - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def attention(h, m, get, eps, kv):
    """h [T, d] attends, head by head, to the (keys, values) of its own layer or of the
    layer it borrows from."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = rms((h @ get("q").T).view(T, H, m["dim"]), eps) * get("q.norm")
    q = rotate(q, m["rot"])
    seen = visible(T, m)
    out = []
    for hd in range(H):
        k, v = kv[0][:, hd // (H // G)], kv[1][:, hd // (H // G)]
        s = (q[:, hd] @ k.T) * m["scale"]
        out.append(sink_softmax(s.masked_fill(~seen, float("-inf")), get("sink")[hd]) @ v)
    return torch.cat(out, -1) @ get("o").T


def expert(x, get, limit):
    """One expert on its (already weighted) input rows."""
    g = torch.clamp(x @ get("gate").T, max=limit)
    u = torch.clamp(x @ get("up").T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ get("down").T


def route(h, router, top):
    """(expert ids [T, top], their sigmoid scores), largest first."""
    s = torch.sigmoid(h @ router.T)
    w, ids = s.sort(dim=-1, descending=True, stable=True)
    return ids[:, :top], w[:, :top]


def experts(h, mlp, get):
    ids, wt = route(h, get("router"), mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(ids[t].tolist(), wt[t]):
            out[t] += expert((w * h[t])[None], lambda n: get(f"e{e}.{n}"),
                             mlp["expert"]["limit"])[0]
    return out


def softcap(z, cap):
    return cap * torch.tanh(z / cap)


def forward(cfg, W, tokens, trace=None):
    """Logits [T, vocab] of every position; ``trace`` collects the residual stream after
    every layer."""
    eps = cfg["norm"]["eps"]
    x = norm_one_plus(W["embed"][torch.tensor(tokens)], W["embed.norm"], eps)
    kvs = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]

        def mix(n, p=p):
            return W[p + "mix." + n]

        src = m.get("kv_from")
        if src is None:
            src = i
            kvs[i] = keys_values(x, m, mix, eps)
        x = x + norm_one_plus(attention(x, m, mix, eps, kvs[src]), W[p + "norm1"], eps)
        if layer.get("mlp"):
            y = experts(x, layer["mlp"], lambda n, p=p: W[p + "mlp." + n])
            x = x + norm_one_plus(y, W[p + "norm2"], eps)
        if trace is not None:
            trace.append(x.clone())
    z = norm_one_plus(x, W["final.norm"], eps) @ W["embed"].T
    cap = cfg.get("logit_softcap")
    return softcap(z, cap) if cap else z
