"""Plain, slow implementation of the Tarunex design: one function per mechanism, whole
sequences, no cache, one head, token or expert at a time where that is clearest.

It is the oracle of the Tarunex tests and shares no code with ``omnia_amd``.  A model is a
JSON-like config dict plus a flat ``name -> tensor`` dict in the checkpoint's naming;
everything is computed in the dtype of ``W`` (float32 or float64)."""
import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def causal(T):
    return torch.arange(T)[None, :] <= torch.arange(T)[:, None]


def temperature(T, t, dtype):
    """[T]: what a query at each position is multiplied by."""
    if not t:
        return torch.ones(T, dtype=dtype)
    return torch.tensor([1.0 + t["coef"] * math.log(math.floor((p + 1) / t["every"]) + 1.0)
                         for p in range(T)], dtype=dtype)


def capped(s, cap):
    return cap * torch.tanh(s / cap) if cap else s


def distance_bias(T, r1, r2):
    """[T, T]: what one head's score of (query i, key j) loses; keys ahead: nothing."""
    d = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).clamp(min=0).to(r1.dtype)
    return r1 * torch.log(1.0 + r2 * d)


def softmax_one(s):
    """Over the last axis, with one added to the denominator."""
    top = s.max(-1, keepdim=True).values.clamp(min=0.0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def softmax(s):
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def attention(h, m, get):
    """Biased projections, no rotation; query temperature, capped scores, a logarithmic
    distance bias per head, gated heads."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]

    def lin(n):
        return h @ get(n).T + get(n + ".b")

    q = lin("q").view(T, H, m["dim"])
    q = q * temperature(T, m.get("q_temp"), h.dtype)[:, None, None]
    k, v = lin("k").view(T, G, m["dim"]), lin("v").view(T, G, m["vdim"])
    gate = sigmoid(h @ get("g").T)
    out = []
    for n in range(H):
        s = capped((q[:, n] @ k[:, n // (H // G)].T) * m["scale"], m.get("softcap"))
        s = s - distance_bias(T, get("r1")[n], get("r2")[n])
        p = softmax_one(s.masked_fill(~causal(T), float("-inf")))
        out.append(p @ v[:, n // (H // G)] * gate[:, n:n + 1])
    return torch.cat(out, -1) @ get("o").T


def rotate(x, base):
    """x [T, ..., dims]: neighbours (2i, 2i + 1) turned by position times frequency."""
    out, dims = x.clone(), x.shape[-1]
    for i in range(dims // 2):
        a = torch.arange(x.shape[0], dtype=torch.float64) * float(base) ** (-2.0 * i / dims)
        c, s = a.cos().to(x.dtype), a.sin().to(x.dtype)
        while c.dim() < x.dim() - 1:
            c, s = c[:, None], s[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def latent_attention(h, m, get, eps):
    """Queries through a latent of their own; keys and values are linear in a shared normed
    latent, beside one rotated key part for all heads; gated heads."""
    T, H, D, R, C = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    cq = rms(h @ get("dq").T, eps) * get("dq.norm")
    q = (cq @ get("uq").T).view(T, H, D + R)
    low = h @ get("dkv").T
    c, kr = rms(low[:, :C], eps) * get("dkv.norm"), rotate(low[:, C:], m["rot"]["base"])
    k, v = (c @ get("uk").T).view(T, H, D), (c @ get("uv").T).view(T, H, m["vdim"])
    gate = sigmoid(h @ get("g").T)
    out = []
    for n in range(H):
        qr = rotate(q[:, n, D:], m["rot"]["base"])
        s = (q[:, n, :D] @ k[:, n].T + qr @ kr.T) * m["scale"]
        out.append(softmax(s.masked_fill(~causal(T), float("-inf"))) @ v[:, n] * gate[:, n:n + 1])
    return torch.cat(out, -1) @ get("o").T


def route(h, router, bias, top):
    """(ids [T, top], weights [T, top]): the largest logits, softmax over those alone."""
    z = h @ router.T + bias
    ids = z.sort(dim=-1, descending=True, stable=True).indices[:, :top]
    return ids, softmax(z.gather(1, ids))


def glu(x, gate, up, down):
    return (silu(x @ gate.T) * (x @ up.T)) @ down.T


def experts(h, mlp, get):
    ids, wts = route(h, get("router"), get("router.b"), mlp["router"]["top"])

    def one(n, x):
        return glu(x, get(n + ".gate"), get(n + ".up"), get(n + ".down"))

    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(ids[t].tolist(), wts[t]):
            out[t] += w * one(f"e{e}", h[t])
    return out + one("shared", h) if mlp.get("shared") else out


def passes(cfg):
    """(layer, number of the pass that starts with it or None) in the order they run."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        out += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return out + [(i, None) for i in range(lp["stop"], n)]


def forward(cfg, W, tokens, trace=None):
    """Logits [T, vocab] of every position; ``trace`` collects the residual stream after
    every layer run."""
    eps = cfg["norm"]["eps"]
    x0 = x = W["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    for i, t in passes(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        if t is not None:
            if t > 0:
                x = x + x0
            x = x + W["loop.step"][t]

        def mix(n):
            return W[p + "mix." + n]

        h = rms(x, eps) * W[p + "norm1"]
        y = (attention(h, layer["mixer"], mix) if layer["type"] == "attention"
             else latent_attention(h, layer["mixer"], mix, eps))
        if layer.get("mlp"):
            y = y + experts(rms(x, eps) * W[p + "norm2"], layer["mlp"],
                            lambda n: W[p + "mlp." + n])
        x = x + y
        if trace is not None:
            trace.append(x.clone())
    z = (rms(x, eps) * W["final.norm"]) @ W["head"].T * cfg["logit_scale"]
    return capped(z, cfg.get("logit_softcap"))
