"""Plain, slow implementation of the Bisuzen design: one function per mechanism, whole
sequences, no cache, one head, token or expert at a time where that is clearest.

It is the oracle of the Bisuzen tests and shares no code with ``omnia_amd``.  A model is a
JSON-like config dict plus a flat ``name -> tensor`` dict in the checkpoint's naming;
everything is computed in the dtype of ``W`` (float32 or float64)."""
import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def tanh_norm(x, alpha, w, b):
    return torch.tanh(alpha * x) * w + b


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def silu(z):
    return z / (1.0 + torch.exp(-z))


def rotate(x, rot):
    """x [T, heads, dim]: neighbours (2i, 2i + 1) of the first ``dims`` of every head, turned
    by position times frequency."""
    out = x.clone()
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        a = torch.arange(x.shape[0], dtype=torch.float64) * f
        c, s = a.cos().to(x.dtype)[:, None], a.sin().to(x.dtype)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def sees_window(T, size, first):
    """[T, T]: the last ``size`` positions, and the sequence's first ones for good."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < first))


def sees_chunk(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def softmax(scores, sink=None):
    """Over the last axis; exp(sink) joins the denominator."""
    top = scores.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.clamp(top, min=float(sink))
    e = torch.exp(scores - top)
    den = e.sum(-1, keepdim=True)
    return e / (den if sink is None else den + torch.exp(sink - top))


def heads_attend(q, k, v, seen, scale, sinks=None):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H * vdim]."""
    H, G, out = q.shape[1], k.shape[1], []
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        p = softmax(s.masked_fill(~seen, float("-inf")), None if sinks is None else sinks[h])
        out.append(p @ v[:, g])
    return torch.cat(out, -1)


def chunked_attention(h, m, get, eps):
    """No positions; unit (RMS) queries and keys; a token sees its own chunk."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = rms((h @ get("q").T).view(T, H, m["dim"]), eps)
    k = rms((h @ get("k").T).view(T, G, m["dim"]), eps)
    v = (h @ get("v").T).view(T, G, m["vdim"])
    return heads_attend(q, k, v, sees_chunk(T, m["mask"]["size"]), m["scale"]) @ get("o").T


def window_attention(h, m, get):
    """Biased projections, rotated queries and keys, window with kept first tokens, sinks."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]

    def lin(n, x):
        return x @ get(n).T + get(n + ".b")

    q = rotate(lin("q", h).view(T, H, m["dim"]), m["rot"])
    k = rotate(lin("k", h).view(T, G, m["dim"]), m["rot"])
    v = lin("v", h).view(T, G, m["vdim"])
    seen = sees_window(T, m["mask"]["size"], m["mask"]["keep_first"])
    return lin("o", heads_attend(q, k, v, seen, m["scale"], get("sink")))


def recurrence(q, k, v, decay, state=None):
    """Token by token: S <- decay S + k v^T, o = S^T q.  q, k [T, H, dim], v [T, H, vdim];
    returns (o, states after the last token)."""
    T, H, D = q.shape
    V = v.shape[-1]
    S = torch.zeros(H, D, V, dtype=q.dtype) if state is None else state.clone()
    lam = torch.tensor(decay, dtype=q.dtype)[:, None, None]
    o = torch.zeros(T, H, V, dtype=q.dtype)
    for t in range(T):
        S = lam * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o, S


def gated_out(o, g, w, eps):
    """Concatenated heads [T, H * vdim]: one RMS norm over all of them, sigmoid gate."""
    return rms(o, eps) * w / (1.0 + torch.exp(-g))


def lightning(h, m, get, eps):
    T, H = h.shape[0], m["heads"]
    q = silu(h @ get("q").T).view(T, H, m["dim"])
    k = silu(h @ get("k").T).view(T, H, m["dim"])
    v = silu(h @ get("v").T).view(T, H, m["vdim"])
    o, _ = recurrence(q, k, v, m["decay"])
    return gated_out(o.reshape(T, -1), h @ get("g").T, get("norm"), eps) @ get("o").T


def branches(a, b, wa, wb, eps):
    """Half the sum of two branch outputs, each RMS-normed over the width."""
    return 0.5 * (rms(a, eps) * wa + rms(b, eps) * wb)


def parallel(h, m, get, eps):
    a = window_attention(h, m["left"], lambda n: get("left." + n))
    b = lightning(h, m["right"], lambda n: get("right." + n), eps)
    return branches(a, b, get("left.out"), get("right.out"), eps)


def route(h, router, correction, top, groups, keep):
    """(ids [T, top], weights [T, top]): softmax scores; chosen by corrected scores among the
    best ``keep`` of ``groups`` neighbourhoods; weighted by plain scores."""
    s = torch.softmax(h @ router.T, -1)
    ids, wts = [], []
    n = s.shape[1] // groups
    for t in range(h.shape[0]):
        c = s[t] + correction
        best = c.view(groups, n).max(-1).values.sort(descending=True, stable=True).indices[:keep]
        ok = torch.zeros(groups, dtype=torch.bool)
        ok[best] = True
        c = c.masked_fill(~ok.repeat_interleave(n), float("-inf"))
        e = c.sort(descending=True, stable=True).indices[:top]
        ids.append(e)
        wts.append(s[t, e] / (s[t, e].sum() + 1e-20))
    return torch.stack(ids), torch.stack(wts)


def expert(x, up, down):
    return gelu_erf(x @ up.T) @ down.T


def experts(h, mlp, get):
    r = mlp["router"]
    ids, wts = route(h, get("router"), get("correction"), r["top"], r["groups"]["count"],
                     r["groups"]["keep"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(ids[t].tolist(), wts[t]):
            y = h[t] if e >= r["experts"] else expert(h[t], get(f"e{e}.up"), get(f"e{e}.down"))
            out[t] += w * y
    return out


def dense(h, get):
    return (gelu_tanh(h @ get("gate").T) * (h @ get("up").T)) @ get("down").T


def order(cfg):
    """Layer indices in the order they run."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return list(range(n))
    body = list(range(lp["start"], lp["stop"]))
    return list(range(lp["start"])) + body * lp["times"] + list(range(lp["stop"], n))


def forward(cfg, W, tokens, trace=None):
    """Logits [T, vocab] of every position; ``trace`` collects the residual stream after
    every layer run."""
    eps = cfg["norm"]["eps"]

    def norm(x, name):
        return tanh_norm(x, W[name + ".alpha"], W[name], W[name + ".b"])

    x = W["embed"][torch.tensor(tokens)]
    for i in order(cfg):
        layer, p = cfg["layers"][i], f"l{i}."

        def mix(n):
            return W[p + "mix." + n]

        def ff(n):
            return W[p + "mlp." + n]

        h = norm(x, p + "norm1")
        mixer = parallel if layer["type"] == "parallel" else chunked_attention
        x = x + mixer(h, layer["mixer"], mix, eps)
        if layer.get("mlp"):
            h = norm(x, p + "norm2")
            x = x + (dense(h, ff) if layer["mlp"]["kind"] == "dense"
                     else experts(h, layer["mlp"], ff))
        if trace is not None:
            trace.append(x.clone())
    return (norm(x, "final.norm") @ W["head"].T) * cfg["logit_scale"]
