"""Plain-PyTorch semantics of the kernels behind :mod:`omnia_amd.ops.mixers` (the
CPU execution path of the CPU test-suite, and the numerics oracle of the kernel
tests).  Same operands, same in-place effects on pages and states."""
from __future__ import annotations

import torch
import torch.nn.functional as F


def slab_sum(m: torch.Tensor) -> torch.Tensor:
    return m.float().sum(0) if m.dim() == 3 else m.float()


def tanh_norm(x, alpha, w, b):
    return torch.tanh(alpha * x) * w + b


def slot_sum(m, identity):
    """Parts [M, S, N] summed; identity parts stand for weight * input."""
    m = m.float()
    if identity is not None:
        ids, wts, inp, first = identity
        m = torch.where((ids >= first)[..., None], wts[..., None] * inp.float()[:, None], m)
    return m.sum(1)


def tanh_norm_residual(x, m, bias, post, a2, w2, b2, dtype):
    v = slab_sum(m)
    if bias is not None:
        v = v + bias
    x += v if post is None else tanh_norm(v, *post.args)
    return tanh_norm(x, a2, w2, b2).to(dtype)


def glu(m, bias, dtype, act):
    v = slab_sum(m)
    if bias is not None:
        v = v + bias
    g, u = v.chunk(2, -1)
    return ((F.gelu(g, approximate="tanh") if act == "gelu_tanh" else F.silu(g)) * u).to(dtype)


def _spans(q_start, n):
    """(sequence, first row, rows) of a step's rows."""
    if q_start is None:
        return [(t, t, 1) for t in range(n)]
    qs = q_start.tolist()
    return [(s, qs[s], qs[s + 1] - qs[s]) for s in range(len(qs) - 1)]


def delta_prep(x, conv_w, conv_state, a_log, dt_bias, q_start, positions, slots, KH, H, D, Dp, V):
    T = positions.numel()
    C = 2 * KH * D + H * V
    taps = conv_w.numel() // C
    w = conv_w.view(C, taps).float()
    y = torch.zeros(T, C)
    for s, r0, n in _spans(q_start, T):
        slot = int(slots[s])
        if slot < 0 or int(positions[r0]) == 0:
            old = torch.zeros(taps - 1, C)
        else:
            old = conv_state[slot].float()
        full = torch.cat([old, x[r0:r0 + n, :C].float()])
        for j in range(taps):
            y[r0:r0 + n] += full[j:j + n] * w[:, j]
    y = F.silu(y)
    q, k = y[:, :KH * D].view(T, KH, D), y[:, KH * D:2 * KH * D].view(T, KH, D)

    def unit(z):
        return F.pad(z / torch.sqrt((z * z).sum(-1, keepdim=True) + 1e-6), (0, Dp - D))

    b, a = x[:, C + H * V:C + H * V + H].float(), x[:, C + H * V + H:C + H * V + 2 * H].float()
    decay = torch.exp(-torch.exp(a_log) * F.softplus(a + dt_bias))
    return (unit(q) * D ** -0.5, unit(k), y[:, 2 * KH * D:].to(x.dtype), decay,
            torch.sigmoid(b))


def delta_run(state, conv_state, qn, kn, vc, decay, beta, x, q_start, positions, slots, KH, H, D,
              V):
    """The recurrence over every row; o [T, H, Vs]; shifts both states."""
    T = positions.numel()
    Vs = state.shape[-1]
    C = 2 * KH * D + H * V
    taps1 = conv_state.shape[1]
    kh = torch.arange(H) // (H // KH)
    o = torch.zeros(T, H, Vs)
    v = F.pad(vc.float().view(T, H, V), (0, Vs - V))
    for s, r0, n in _spans(q_start, T):
        slot = int(slots[s])
        if slot < 0:
            continue
        fresh = int(positions[r0]) == 0
        S = torch.zeros(H, D, Vs) if fresh else state[slot].clone()
        for t in range(r0, r0 + n):
            k, q = kn[t, kh, :D], qn[t, kh, :D]
            S = S * decay[t][:, None, None]
            u = beta[t][:, None] * (v[t] - torch.matmul(k[:, None], S)[:, 0])
            S = S + k[:, :, None] * u[:, None, :]
            o[t] = torch.matmul(q[:, None], S)[:, 0]
        state[slot] = S
        if taps1:
            old = torch.zeros(taps1, C, dtype=x.dtype) if fresh else conv_state[slot].clone()
            conv_state[slot] = torch.cat([old, x[r0:r0 + n, :C]])[-taps1:]
    return o


def delta_norm(o, x, zoff, norm_w, H, V, Vp, eps):
    T = x.shape[0]
    ov = o[..., :V]
    y = ov / torch.sqrt(ov.pow(2).mean(-1, keepdim=True) + eps) * norm_w
    y = y * F.silu(x[:, zoff:zoff + H * V].float().view(T, H, V))
    return F.pad(y, (0, Vp - V)).to(x.dtype).reshape(T, H * Vp)


def lightning(x, w, spec, state, q_start, positions, slots, eps):
    T, H, Dp, Vp = positions.numel(), spec.heads, spec.dim_pad, spec.v_pad
    x = slab_sum(x)[:, :spec.in_cols]
    q, k, v, g = x.split([H * Dp, H * Dp, H * Vp, H * Vp], 1)
    q, k, v = (F.silu(t).view(T, H, -1) for t in (q, k, v))
    a = w["pow"][:, 1, None, None]
    o = torch.zeros(T, H, Vp)
    for s, r0, n in _spans(q_start, T):
        slot = int(slots[s])
        if slot < 0:
            continue
        S = torch.zeros(H, Dp, Vp) if int(positions[r0]) == 0 else state[slot].clone()
        for t in range(r0, r0 + n):
            S = S * a + k[t][:, :, None] * v[t][:, None, :]
            o[t] = torch.matmul(q[t][:, None], S)[:, 0]
        state[slot] = S
    o = o.view(T, H * Vp)
    o = o / torch.sqrt(o.pow(2).sum(-1, keepdim=True) / (H * spec.vdim) + eps) * w["norm"]
    return o * torch.sigmoid(g)


def _rotate(v, positions, cos_sin):
    half = v.shape[-1] // 2
    cs = cos_sin[positions.long()]
    while cs.dim() < v.dim():
        cs = cs[:, None]
    c, s = cs[..., :half], cs[..., half:]
    a, b = v[..., :half].float(), v[..., half:].float()
    return torch.cat([a * c - b * s, b * c + a * s], -1)


def latent_prep(cache, x, wq, wc, positions, slots, cos_sin, Qp, Cp, R, eps):
    Q, C = wq.numel(), wc.numel()

    def rms(v, w):
        v = v.float()
        return (v / torch.sqrt(v.pow(2).mean(-1, keepdim=True) + eps) * w).to(x.dtype)

    cq = F.pad(rms(x[:, :Q], wq), (0, Qp - Q))
    c = rms(x[:, Qp:Qp + C], wc)
    kr = _rotate(x[:, Qp + Cp:Qp + Cp + R], positions, cos_sin).to(x.dtype)
    keep = slots >= 0
    flat = cache.view(-1, cache.shape[-1])
    flat[slots[keep], :C] = c[keep]
    flat[slots[keep], Cp:Cp + R] = kr[keep]
    return cq


def latent_rotate(q, hstride, off, positions, cos_sin, H, R):
    v = q[:, :H * hstride].view(q.shape[0], H, hstride)
    v[..., off:off + R] = _rotate(v[..., off:off + R], positions, cos_sin).to(q.dtype)


def latent_heads(out, ho, x, hx, W, gate, positions, cos_sin, R, Rp, rotx):
    H, N, K = W.shape
    T = x.shape[0]
    xv = x[:, :H * hx].reshape(T, H, hx)
    y = torch.matmul(xv[..., :K].float().transpose(0, 1), W.float().transpose(1, 2)).transpose(0, 1)
    if gate is not None:
        y = y * torch.sigmoid(gate[:, :H].float())[..., None]
    ov = out.view(T, H, ho)
    ov[..., :N] = y.to(out.dtype)
    if positions is not None:
        ov[..., N:] = 0
        ov[..., N:N + R] = _rotate(xv[..., rotx:rotx + R], positions, cos_sin).to(out.dtype)


def latent_attend(q, cache, block_tables, q_start, positions, H, Cp, window, scale):
    """q [T, H*Lp] absorbed queries -> [T, H*Cp]."""
    T, (_, page, Lp) = positions.numel(), cache.shape
    out = torch.zeros(T, H, Cp, dtype=q.dtype)
    qv = q.view(T, H, Lp).float()
    for s, r0, n in _spans(q_start, T):
        for t in range(r0, r0 + n):
            pos = int(positions[t])
            lo = max(0, pos - window + 1) if window > 0 else 0
            key = torch.arange(lo, pos + 1)
            rows = cache[block_tables[s, key // page].long(), key % page].float()
            p = torch.softmax(qv[t] @ rows.T * scale, -1)
            out[t] = (p @ rows[:, :Cp]).to(q.dtype)
    return out.view(T, H * Cp)


def rms_norm(x, n):
    x = x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) * n.inv_n + n.eps) * n.gain
    return x if n.w is None else x * n.w


def route(h, router, spec, corr=None, bias=None):
    """(ids int32 [T, top], weights fp32 [T, top])."""
    z = h.float() @ router.float().T
    if bias is not None:
        z = z + bias
    s = torch.sigmoid(z) if spec.score == "sigmoid" else torch.softmax(z, -1)
    c = z if corr is None else s + corr
    if spec.groups > 1:
        best = c.view(c.shape[0], spec.groups, -1).amax(-1)
        order = best.sort(dim=-1, descending=True, stable=True).indices[:, spec.keep:]
        out = torch.zeros_like(best, dtype=torch.bool).scatter_(1, order, True)
        c = c.masked_fill(out.repeat_interleave(c.shape[1] // spec.groups, 1), float("-inf"))
    ids = c.sort(dim=-1, descending=True, stable=True).indices[:, :spec.top]
    wt = s.gather(1, ids)
    if spec.renorm:
        wt = wt / (wt.sum(-1, keepdim=True) + 1e-20)
    return ids.int(), wt


def experts(h, ids, wts, up, down, spec):
    """[T, top, d]: the chosen experts' weighted outputs (clamped GLUs take the weight on
    their input)."""
    clamped = spec.expert == "clamped_glu"
    T, d = h.shape
    out = torch.zeros(T, spec.top, d, dtype=h.dtype)
    for e in ids.unique().tolist():
        if e >= spec.experts:
            continue
        t, j = (ids == e).nonzero(as_tuple=True)
        v, wt = h[t].float() @ up[e].float().T, wts[t, j, None]
        if spec.expert == "glu":
            g, u = v.chunk(2, -1)
            a = F.silu(g) * u
        elif clamped:
            g, u = (v * wt).chunk(2, -1)
            g, u = g.clamp(max=spec.limit), u.clamp(-spec.limit, spec.limit)
            a, wt = g * torch.sigmoid(spec.alpha * g) * (u + 1.0), 1.0
        else:
            a = F.gelu(v)
        out[t, j] = (a.to(h.dtype).float() @ down[e].float().T * wt).to(h.dtype)
    return out


def _rotate_pairs(v, positions, cos_sin):
    """Neighbours (2i, 2i + 1) turn together."""
    half = v.shape[-1] // 2
    cs = cos_sin[positions.long()][:, None]
    c, s = cs[..., :half], cs[..., half:]
    a, b = v[..., 0::2], v[..., 1::2]
    return torch.stack([a * c - b * s, b * c + a * s], -1).flatten(-2)


def gqa_prep(x, w, spec, k, v, positions, slots, cos_sin, dtype, eps, temp=None, gate=None):
    T, H, D, Dp = positions.numel(), spec.heads, spec.dim, spec.dim_pad
    R = 0 if cos_sin is None else cos_sin.shape[1]
    x = slab_sum(x)
    if gate is not None:
        gate.copy_(torch.sigmoid(x[:, spec.qkv_cols:spec.in_cols]))
    if w.get("in_b") is not None:
        x = x[:, :w["in_b"].numel()] + w["in_b"]

    def turned(z, wn, heads, factor=None):
        z = z.reshape(T, heads, Dp)
        if wn is not None:
            z = z / torch.sqrt(z.pow(2).sum(-1, keepdim=True) / D + eps) * wn
        if R:
            turn = _rotate_pairs if spec.rotary.interleaved else _rotate
            z = torch.cat([turn(z[..., :R], positions, cos_sin), z[..., R:]], -1)
        if factor is not None:
            z = z * factor[positions.long()][:, None, None]
        return z.to(dtype)

    if k is not None:
        G, page, Vp = k.shape[1], k.shape[2], v.shape[3]
        kk = turned(x[:, H * Dp:(H + G) * Dp], w.get("k_norm"), G)
        vv = x[:, (H + G) * Dp:(H + G) * Dp + G * Vp].reshape(T, G, Vp).to(dtype)
        keep = slots >= 0
        b, o = slots[keep] // page, slots[keep] % page
        k[b, :, o], v[b, :, o] = kk[keep], vv[keep]
    return turned(x[:, :H * Dp], w.get("q_norm"), H, temp).reshape(T, H * Dp)


def _visible(pos, mask):
    window, first, chunk = mask
    if chunk:
        return torch.arange(pos // chunk * chunk, pos + 1)
    lo = max(0, pos - window + 1) if window > 0 else 0
    return torch.cat([torch.arange(0, min(first, lo)), torch.arange(lo, pos + 1)])


def gqa_attend(out, q, k, v, block_tables, q_start, positions, H, mask, scale, sinks, cap=0.0,
               dist=None, gate=None):
    T, G, page = positions.numel(), k.shape[1], k.shape[2]
    qv = q.view(T, G, H // G, -1).float()
    ov = out.view(T, H, -1)
    for s, r0, n in _spans(q_start, T):
        for t in range(r0, r0 + n):
            key = _visible(int(positions[t]), mask)
            b = block_tables[s, key // page].long()
            kr, vr = k[b, :, key % page].float(), v[b, :, key % page].float()  # [n, G, w]
            sc = torch.matmul(qv[t], kr.permute(1, 2, 0)).reshape(H, -1) * scale
            if cap:
                sc = cap * torch.tanh(sc / cap)
            if dist is not None:
                far = (int(positions[t]) - key).float()
                sc = sc - dist[0][:, None] * torch.log(1.0 + dist[1][:, None] * far)
            if sinks is not None:
                sc = torch.cat([sc, sinks[:, None]], 1)
            p = torch.softmax(sc, -1)[:, :key.numel()].view(G, H // G, -1)
            o = torch.matmul(p, vr.permute(1, 0, 2)).reshape(H, -1)
            ov[t] = (o if gate is None else o * gate[t][:, None]).to(q.dtype)
