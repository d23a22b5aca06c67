"""Front-end of the kernels behind layer-list models: Dynamic-Tanh and RMS norms fused
with the residual (``csrc/tanh_norm.hip``, ``csrc/rms_residual.hip``,
``csrc/branch_residual.hip``, ``csrc/joined_residual.hip``), the gated delta rule (``csrc/delta.hip``), fixed-decay
linear attention (``csrc/lightning.hip``), latent attention (``csrc/latent.hip``),
grouped-query attention (``csrc/gqa.hip``, ``csrc/gqa_prefill.hip``) and routed experts
(``csrc/moe.hip``, ``csrc/pgemm.hip``).

GPU tensors (bf16 or fp32) run the HIP kernels and nothing else; CPU tensors run
:mod:`omnia_amd.ops.reference_mixers`."""
from __future__ import annotations

import torch

from . import MOE_TILE256_ROWS, _moe_grouped, checks, kernels
from . import reference_mixers as ref


# ------------------------------------------------------------------ tanh norm
class TanhNorm:
    """``tanh(alpha x) w + b`` with fp32 parameters."""

    __slots__ = ("alpha", "w", "b")

    def __init__(self, alpha: float, w: torch.Tensor, b: torch.Tensor):
        self.alpha, self.w, self.b = float(alpha), w, b

    @property
    def args(self):
        return self.alpha, self.w, self.b


def tanh_norm_embed(ids, table, vocab: int, norm: TanhNorm, src=None, tok_slots=None):
    """(fp32 residual rows, first normed input).  ``src`` / ``tok_slots``: rows whose
    token is still on the device, as :func:`omnia_amd.ops.embedding`."""
    T, d = ids.numel(), table.shape[1]
    if ids.is_cuda:
        x = torch.empty(T, d, dtype=torch.float32, device=ids.device)
        h = torch.empty(T, d, dtype=table.dtype, device=ids.device)
        kernels().tanh_norm_embed(h, x, ids, table, vocab, *norm.args, src, tok_slots)
        return x, h
    if src is not None:
        ids = torch.where(src >= 0, tok_slots.index_select(0, src.clamp(min=0).long()), ids)
    ok = (ids >= 0) & (ids < vocab)
    x = table[torch.where(ok, ids, torch.zeros_like(ids)).long()].float() * ok[:, None]
    return x, ref.tanh_norm(x, *norm.args).to(table.dtype)


def tanh_norm_residual(x, m, post: TanhNorm | None, pre: TanhNorm, dtype, bias=None,
                       slots: bool = False, identity=None):
    """In place ``x += post(m + bias)`` (no post: ``m + bias`` itself); returns ``pre(x)`` in
    ``dtype``.  ``m``: a projection [M, N], its split-K slabs [S, M, N], or (``slots``)
    parts [M, S, N], where ``identity`` = (ids [M, S], weights [M, S], input [M, N], first)
    makes the parts with ids >= first stand for weight * input."""
    if x.is_cuda:
        h = torch.empty(x.shape, dtype=dtype, device=x.device)
        kernels().tanh_norm_residual(h, x, m, slots, bias,
                                     *(post.args if post else (0.0, None, None)), *pre.args,
                                     *(identity or (None, None, None, 0)))
        return h
    if slots:
        m = ref.slot_sum(m, identity)
    return ref.tanh_norm_residual(x, m, bias, post, *pre.args, dtype)


def glu(m, bias, dtype, act: str = "silu"):
    """``act(g + bg) * (u + bu)`` of a [gate | up] projection (or its slabs)."""
    if m.is_cuda:
        out = torch.empty(m.shape[-2], m.shape[-1] // 2, dtype=dtype, device=m.device)
        kernels().glu(out, m, bias, act == "gelu_tanh")
        return out
    return ref.glu(m, bias, dtype, act)


# ------------------------------------------------------------------- RMS norm
class RMSNorm:
    """``x / sqrt(mean(x^2) + eps) * gain * w`` over ``n`` real columns (``w`` fp32, zero on
    the padding columns, or None: ``gain`` alone)."""

    __slots__ = ("w", "gain", "inv_n", "eps")

    def __init__(self, w: torch.Tensor | None, n: int, eps: float, gain: float = 1.0):
        self.w, self.gain, self.inv_n, self.eps = w, float(gain), 1.0 / n, float(eps)


def rms_embed(ids, table, vocab: int, emb: RMSNorm, pre: RMSNorm | None, src=None,
              tok_slots=None):
    """(fp32 residual rows ``emb(table[ids])``, first sublayer input ``pre(x)`` or x)."""
    T, d = ids.numel(), table.shape[1]
    if ids.is_cuda:
        x = torch.empty(T, d, dtype=torch.float32, device=ids.device)
        h = torch.empty(T, d, dtype=table.dtype, device=ids.device)
        kernels().rms_embed(h, x, ids, table, vocab, emb.w, None if pre is None else pre.w,
                            emb.inv_n, emb.eps, src, tok_slots)
        return x, h
    if src is not None:
        ids = torch.where(src >= 0, tok_slots.index_select(0, src.clamp(min=0).long()), ids)
    ok = (ids >= 0) & (ids < vocab)
    x = table[torch.where(ok, ids, torch.zeros_like(ids)).long()].float() * ok[:, None]
    x = ref.rms_norm(x, emb)
    return x, (x if pre is None else ref.rms_norm(x, pre)).to(table.dtype)


def rms_residual(x, m, post: RMSNorm, pre: RMSNorm | None, dtype, bias=None,
                 slots: bool = False):
    """In place ``x += post(m + bias)``; returns ``pre(x)``, or x itself, in ``dtype``.  ``m``: a
    projection [M, d], its split-K slabs [S, M, d], or (``slots``) parts [M, S, d]."""
    if x.is_cuda:
        h = torch.empty(x.shape, dtype=dtype, device=x.device)
        kernels().rms_residual(h, x, m, slots, bias, post.w, None if pre is None else pre.w,
                               post.inv_n, post.eps)
        return h
    v = m.float().sum(1) if slots else ref.slab_sum(m)
    if bias is not None:
        v = v + bias
    x += ref.rms_norm(v, post)
    return (x if pre is None else ref.rms_norm(x, pre)).to(dtype)


def norm_embed(ids, table, vocab: int, emb, pre, src=None, tok_slots=None):
    """Residual rows and first sublayer input of either norm kind."""
    if isinstance(emb or pre, TanhNorm):
        if emb is not None:
            raise ValueError("no embedding norm of the tanh kind")
        return tanh_norm_embed(ids, table, vocab, pre, src, tok_slots)
    return rms_embed(ids, table, vocab, emb, pre, src, tok_slots)


def branch_residual(x, branches, pre, dtype):
    """In place ``x += sum of norm(m + bias)`` over two branches (m, bias, RMSNorm), m a
    projection or its slabs; returns ``pre(x)`` (either kind, None: x) in ``dtype``."""
    (a, ab, an), (b, bb, bn) = branches
    if x.is_cuda:
        h = torch.empty(x.shape, dtype=dtype, device=x.device)
        alpha, nw, nb = pre.args if isinstance(pre, TanhNorm) else (
            0.0, None if pre is None else pre.w, None)
        kernels().branch_residual(h, x, a, ab, an.w, b, bb, bn.w, an.inv_n, an.eps, alpha, nw, nb)
        return h
    for m, bias, norm in branches:
        v = ref.slab_sum(m)
        x += ref.rms_norm(v if bias is None else v + bias, norm)
    if isinstance(pre, TanhNorm):
        return ref.tanh_norm(x, *pre.args).to(dtype)
    return (x if pre is None else ref.rms_norm(x, pre)).to(dtype)


class PassInput:
    """What a pass of a looped stretch adds to the residual before its first layer: ``scale``
    times the embedding of each row's token (``scale`` 0: nothing), and ``step`` [d] (fp32,
    or None).  ``ids`` / ``src`` / ``tok_slots``: the rows' tokens, as
    :func:`omnia_amd.ops.embedding`."""

    __slots__ = ("ids", "table", "vocab", "scale", "step", "src", "tok_slots")

    def __init__(self, ids, table, vocab: int, scale: float, step=None, src=None, tok_slots=None):
        self.ids, self.table, self.vocab, self.scale = ids, table, vocab, float(scale)
        self.step, self.src, self.tok_slots = step, src, tok_slots


def joined_residual(x, parts, pres, dtype, enter: PassInput | None = None, fresh: bool = False):
    """In place ``x += sum of parts`` and what a pass enters with (``fresh``: x starts from
    zero); returns one normed row set in ``dtype`` for each of ``pres`` (one or two RMS
    norms of one mean).  ``parts``: up to three (m, slots): a projection [M, d], its split-K
    slabs [S, M, d], or (slots) per-row parts [M, S, d]."""
    if x.is_cuda:
        out = [torch.empty(x.shape, dtype=dtype, device=x.device) for _ in pres]
        p = list(parts) + [(None, False)] * (3 - len(parts))
        e = (enter.ids, enter.table, enter.vocab, enter.scale, enter.step, enter.src,
             enter.tok_slots) if enter else (None, None, 0, 0.0, None, None, None)
        a, b = pres[0], pres[-1]
        kernels().joined_residual(out[0], out[1] if len(out) > 1 else None, x, fresh, *p[0],
                                  *p[1], *p[2], *e, a.w, a.gain, b.w, b.gain, a.inv_n, a.eps)
        return out
    if fresh:
        x.zero_()
    for m, slots in parts:
        x += m.float().sum(1) if slots else ref.slab_sum(m)
    if enter is not None:
        if enter.scale:
            ids = enter.ids
            if enter.src is not None:
                ids = torch.where(enter.src >= 0, enter.tok_slots.index_select(
                    0, enter.src.clamp(min=0).long()), ids)
            ok = (ids >= 0) & (ids < enter.vocab)
            x += enter.scale * enter.table[torch.where(
                ok, ids, torch.zeros_like(ids)).long()].float() * ok[:, None]
        if enter.step is not None:
            x += enter.step
    return [ref.rms_norm(x, n).to(dtype) for n in pres]


def norm_residual(x, m=None, post=None, pre=None, dtype=None, bias=None, slots: bool = False,
                  identity=None, branches=None):
    """What follows a sublayer, of either norm kind (see the functions above)."""
    if branches is not None:
        if post is not None:
            raise ValueError("branches carry their own norms")
        return branch_residual(x, branches, pre, dtype)
    if isinstance(post or pre, TanhNorm):
        return tanh_norm_residual(x, m, post, pre, dtype, bias, slots, identity)
    if post is None or identity is not None:
        raise ValueError("RMS residual steps need a post-norm and no identity parts")
    return rms_residual(x, m, post, pre, dtype, bias, slots)


def softcap_(logits: torch.Tensor, cap: float) -> torch.Tensor:
    """In place ``cap tanh(logits / cap)``."""
    if logits.is_cuda:
        kernels().softcap(logits, cap)
        return logits
    return logits.copy_((cap * torch.tanh(logits.float() / cap)).to(logits.dtype))


# -------------------------------------------------------------------- experts
def experts(h, w: dict, spec):
    """Routed experts: (parts [T, top, d], ids, weights), the parts summed by the residual
    kernel; those of identity experts (ids >= spec.experts) are not written.  The weights
    are padded to whole tiles (``ff_pad``; d a multiple of 64)."""
    T, d = h.shape
    k, E, ff = spec.top, spec.outputs, w["down"].shape[2]
    corr, bias = w.get("correction"), w.get("router_b")
    if not h.is_cuda:
        ids, wts = ref.route(h, w["router"], spec, corr, bias)
        return ref.experts(h, ids, wts, w["up"], w["down"], spec), ids, wts
    kk = kernels()
    ids = torch.empty(T, k, dtype=torch.int32, device=h.device)
    wts = torch.empty(T, k, dtype=torch.float32, device=h.device)
    kk.moe_route(ids, wts, h, w["router"], k, spec.score == "sigmoid", spec.renorm, corr,
                 spec.groups, spec.keep, bias)
    # column tiles of the 256-row prefill GEMM: 128 gate and up columns, or 256
    tile = h.dtype == torch.bfloat16 and T * k >= MOE_TILE256_ROWS * E and d % 256 == 0 and \
        ff % (128 if spec.gated else 256) == 0
    y = _moe_grouped(h, w["up"], w["down"], ids, wts, k, E, 0, spec.experts, 256 if tile else 64,
                     (spec.alpha, spec.limit) if spec.expert == "clamped_glu" else None,
                     not spec.gated)
    return y.view(T, k, d), ids, wts


# ----------------------------------------------------------------- delta rule
def delta_rule(x, w: dict, spec, state, conv_state, q_start, positions, slots, eps: float,
               out: torch.Tensor | None = None) -> torch.Tensor:
    """Gated delta rule over one set of rows: decode (``q_start`` None, one row per
    sequence) or prefill portions.  ``x`` rows are the fused input projection
    [q | k | v | z | b | a]; states of ``slots`` advance in place.  Returns
    [T, heads * v_pad], the output projection's input."""
    T = positions.numel()
    KH, H, D, V = spec.kv_heads, spec.heads, spec.dim, spec.vdim
    Dp, Vs, Vp, taps = spec.dim_pad, spec.v_state_pad, spec.v_pad, spec.conv
    C = spec.conv_channels
    if not x.is_cuda:
        qn, kn, vc, decay, beta = ref.delta_prep(x, w["conv"], conv_state, w["a_log"],
                                                 w["dt_bias"], q_start, positions, slots, KH, H,
                                                 D, Dp, V)
        o = ref.delta_run(state, conv_state, qn, kn, vc, decay, beta, x, q_start, positions,
                          slots, KH, H, D, V)
        y = ref.delta_norm(o, x, C, w["norm"], H, V, Vp, eps)
        if out is not None:
            out.copy_(y)
            return out
        return y
    kk, dev = kernels(), x.device
    if checks.active(x):
        checks.state_slots("delta_rule", slots, state)
    qn = torch.empty(T, KH, Dp, dtype=torch.float32, device=dev)
    kn = torch.empty_like(qn)
    vc = torch.empty(T, H * V, dtype=x.dtype, device=dev)
    decay = torch.empty(T, H, dtype=torch.float32, device=dev)
    beta = torch.empty_like(decay)
    y = torch.empty(T, H * Vp, dtype=x.dtype, device=dev) if out is None else out
    kk.delta_prep(qn, kn, vc, decay, beta, x, w["conv"], conv_state, w["a_log"], w["dt_bias"],
                  q_start, positions, slots, KH, H, D, Dp, V, taps)
    if q_start is None:
        kk.delta_step(y, state, conv_state, qn, kn, vc, decay, beta, x, w["norm"], positions,
                      slots, KH, H, D, Dp, V, Vp, taps, eps)
        return y
    o = torch.empty(T, H, Vs, dtype=torch.float32, device=dev)
    rec = torch.empty(kk.delta_records(T, slots.numel(), H), dtype=torch.float32, device=dev)
    kk.delta_scan(o, state, conv_state, rec, qn, kn, vc, decay, beta, x, q_start, positions, slots, KH,
                  H, D, Dp, V, taps)
    kk.delta_norm(y, o, x, C, w["norm"], H, V, Vs, Vp, eps)
    return y


# ---------------------------------------------------- fixed-decay linear attention
def decay_powers(decay, device) -> torch.Tensor:
    """fp32 [heads, 48]: a^0 .. a^32, then a^64, a^128, a^256, ... (double precision)."""
    n = torch.tensor([*range(33), *(64 << i for i in range(15))], dtype=torch.float64)
    a = torch.tensor(decay, dtype=torch.float64)
    return torch.pow(a[:, None], n).float().to(device)


def lightning(x, w: dict, spec, state, q_start, positions, slots, eps: float, dtype,
              out: torch.Tensor | None = None) -> torch.Tensor:
    """Linear attention over one set of rows: decode (``q_start`` None, one row per
    sequence) or prefill portions.  ``x`` rows are projections [q | k | v | gate], of a
    decode step also their split-K slabs; states of ``slots`` advance in place.  Returns
    [T, heads * v_pad], the output projection's input."""
    T, H, Dp, Vp = positions.numel(), spec.heads, spec.dim_pad, spec.v_pad
    n, inv_n, goff = H * Vp, 1.0 / (H * spec.vdim), H * (2 * Dp + Vp)
    y = torch.empty(T, n, dtype=dtype, device=x.device) if out is None else out
    if not x.is_cuda:
        return y.copy_(ref.lightning(x, w, spec, state, q_start, positions, slots, eps))
    kk, dev = kernels(), x.device
    if checks.active(x):
        checks.state_slots("lightning", slots, state)
    o = torch.empty(T, H, Vp, dtype=torch.float32, device=dev)
    if q_start is None:
        kk.lightning_step(o, state, x, w["pow"], positions, slots)
    else:
        need = kk.lightning_scratch(T, slots.numel(), H, Dp, Vp)
        seg = torch.empty(need, dtype=torch.float32, device=dev) if need else None
        kk.lightning_scan(o, state, seg, x, w["pow"], q_start, positions, slots)
    kk.lightning_norm(y, o, x, goff, w["norm"], inv_n, eps)
    return y


# ----------------------------------------------------------- latent attention
def latent_prep(cache, x, wq, wc, positions, slots, cos_sin, Qp: int, Cp: int, eps: float):
    """Normed query latent [T, Qp]; writes the token's cache row at ``slots``."""
    R = cos_sin.shape[1]
    if x.is_cuda:
        if checks.active(x):
            checks.slots("latent_prep", slots, cache[:, None])
        cq = torch.empty(x.shape[0], Qp, dtype=x.dtype, device=x.device)
        kernels().latent_prep(cq, cache, x, wq, wc, positions, slots, cos_sin, Cp, R, eps)
        return cq
    return ref.latent_prep(cache, x, wq, wc, positions, slots, cos_sin, Qp, Cp, R, eps)


def latent_rotate(q, spec, positions, cos_sin):
    """Rotate the rotated part of q [T, H * qk_pad] in place."""
    args = (q, spec.qk_pad, spec.dim_pad, positions, cos_sin, spec.heads, spec.rot_dim)
    (kernels().latent_rotate if q.is_cuda else ref.latent_rotate)(*args)


def latent_absorb(q, w_uk, spec, positions, cos_sin):
    """q [T, H * qk_pad] -> absorbed queries [T, H * padded_cache_width]."""
    Lp = spec.padded_cache_width
    out = torch.empty(q.shape[0], spec.heads * Lp, dtype=q.dtype, device=q.device)
    args = (out, Lp, q, spec.qk_pad, w_uk, None, positions, cos_sin, spec.rot_dim, spec.rot_pad,
            spec.dim_pad)
    (kernels().latent_heads if q.is_cuda else ref.latent_heads)(*args)
    return out


def latent_expand(o, w_uv, spec, gate, out=None):
    """Attended latents [T, H * latent_pad] -> gated head outputs [T, H * v_pad]."""
    if out is None:
        out = torch.empty(o.shape[0], spec.heads * spec.v_pad, dtype=o.dtype, device=o.device)
    args = (out, spec.v_pad, o, spec.latent_pad, w_uv, gate, None, None, 0, 0, 0)
    (kernels().latent_heads if o.is_cuda else ref.latent_heads)(*args)
    return out


def latent_attend(q, cache, block_tables, q_start, positions, spec):
    """Generic absorbed attention (any size, bf16 / fp32)."""
    H, Cp = spec.heads, spec.latent_pad
    if q.is_cuda:
        out = torch.empty(q.shape[0], H * Cp, dtype=q.dtype, device=q.device)
        kernels().latent_attend(out, q, cache, block_tables, q_start, positions, H, Cp,
                                spec.window, spec.scale)
        return out
    return ref.latent_attend(q, cache, block_tables, q_start, positions, H, Cp, spec.window,
                             spec.scale)


def latent_decode_covers(spec) -> bool:
    """The MFMA decode kernel covers this size (any power-of-two page)."""
    return bool(kernels().latent_decode_covers(spec.latent_pad, spec.padded_cache_width))


def latent_decode(q, cache, block_tables, positions, spec, splits: int):
    """MFMA decode over absorbed queries, each row's keys in up to ``splits`` parts."""
    T, H, Cp = positions.numel(), spec.heads, spec.latent_pad
    out = torch.empty(T, H * Cp, dtype=q.dtype, device=q.device)
    po = pm = None
    if splits > 1:
        po = torch.empty(T * H * splits * Cp, dtype=torch.float32, device=q.device)
        pm = torch.empty(T * H * splits * 2, dtype=torch.float32, device=q.device)
    kernels().latent_decode(out, po, pm, q, cache, block_tables, positions, H, Cp, spec.window,
                            spec.scale, splits)
    return out


def latent_gather(cache, block_tables, kv_start, kv_first, seq_lens, rows: int, spec):
    """Dense cached rows of each sequence's visible range: (c [rows, latent_pad],
    k_rot [rows, rot_pad])."""
    c = torch.empty(rows, spec.latent_pad, dtype=cache.dtype, device=cache.device)
    kr = torch.empty(rows, spec.rot_pad, dtype=cache.dtype, device=cache.device)
    kernels().latent_gather(c, kr, cache, block_tables, kv_start, kv_first, seq_lens)
    return c, kr


def latent_prefill(q, kx, kr, vt, fb, spec, gate, out=None):
    """MFMA prefill attention over expanded keys; gated [T, H * v_pad]."""
    T, H = q.shape[0], spec.heads
    if out is None:
        out = torch.empty(T, H * spec.v_pad, dtype=q.dtype, device=q.device)
    kernels().latent_prefill(out.view(T, H, spec.v_pad), q.view(T, H, spec.qk_pad), kx, kr, vt,
                             fb.q_start_loc, fb.seq_lens, fb.kv_start, fb.kv_first, fb.tile_seq,
                             fb.tile_q0, spec.window, spec.scale, gate)
    return out


# ------------------------------------------------------ grouped-query attention
def temperature_table(t, positions: int, device) -> torch.Tensor:
    """fp32 [positions]: a query's factor at each position (double precision)."""
    p = torch.arange(1, positions + 1, dtype=torch.float64)
    return (1.0 + t.coef * torch.log(torch.floor(p / t.every) + 1.0)).float().to(device)


def gqa_prep(x, w: dict, spec, pages, positions, slots, cos_sin, dtype, eps: float, temp=None,
             gate=None):
    """Fused projection rows (or split-K slabs) -> queries [T, H * dim_pad], with bias, norm,
    rotation and temperature (``temp``: :func:`temperature_table`) as the spec says; writes
    the tokens' keys and values at ``slots`` of ``pages`` = (k, v), or, with ``pages`` None,
    none (the layer borrows another one's).  ``gate`` [T, H] fp32 receives the sigmoid of
    the row's gate columns."""
    k, v = pages if pages is not None else (None, None)
    if x.is_cuda:
        if pages is not None and checks.active(x):
            checks.slots("gqa_prep", slots, k)
        q = torch.empty(positions.numel(), spec.heads * spec.dim_pad, dtype=dtype,
                        device=x.device)
        kernels().gqa_prep(q, k, v, x, w.get("q_norm"), w.get("k_norm"), w.get("in_b"), positions,
                           slots, cos_sin, spec.rotary is not None and spec.rotary.interleaved,
                           spec.heads, spec.dim, spec.dim_pad, eps, temp, gate)
        return q
    return ref.gqa_prep(x, w, spec, k, v, positions, slots, cos_sin, dtype, eps, temp, gate)


# ``dist`` [2, H] fp32: the heads' distance biases (r1, r2), or None; ``gate`` [T, H] fp32:
# factors of the head outputs, or None
def gqa_attend(q, pages, block_tables, q_start, positions, spec, sinks, out=None, dist=None,
               gate=None):
    """Generic attention (any size, bf16 / fp32): [T, H * v_pad]."""
    if out is None:
        out = torch.empty(positions.numel(), spec.heads * spec.v_pad, dtype=q.dtype,
                          device=q.device)
    args = (out, q, *pages, block_tables, q_start, positions, spec.heads, spec.mask,
            spec.scale, sinks, spec.softcap, dist, gate)
    (kernels().gqa_attend if q.is_cuda else ref.gqa_attend)(*args)
    return out


def gqa_decode(q, pages, block_tables, positions, spec, sinks, splits: int, out=None, dist=None,
               gate=None):
    """bf16 decode: each row's visible keys in up to ``splits`` parts."""
    T, H, V = positions.numel(), spec.heads, spec.v_pad
    if out is None:
        out = torch.empty(T, H * V, dtype=q.dtype, device=q.device)
    po = pm = None
    if splits > 1:
        po = torch.empty(T * H * splits * V, dtype=torch.float32, device=q.device)
        pm = torch.empty(T * H * splits * 2, dtype=torch.float32, device=q.device)
    if checks.active(q):
        checks.paged("gqa_decode", block_tables, positions + 1, pages[0], T)
    kernels().gqa_decode(out, po, pm, q, *pages, block_tables, positions, H, spec.mask,
                         spec.scale, sinks, splits, spec.softcap, dist, gate)
    return out


def scores_bounded(spec, dist) -> bool:
    """Capped scores that distance only lowers, with no learned sink: their exponentials need
    no maximum taken off (fp32 holds exp(40) times any context)."""
    return (0.0 < spec.softcap <= 40.0 and spec.sink != "learned" and dist is not None
            and bool((dist >= 0).all()))


def gqa_prefill(q, pages, fb, spec, sinks, out=None, dist=None, gate=None, bounded=False):
    """bf16 prefill portions (``fb``'s query tiles of 128 rows).  ``bounded``:
    :func:`scores_bounded`."""
    if out is None:
        out = torch.empty(q.shape[0], spec.heads * spec.v_pad, dtype=q.dtype, device=q.device)
    if checks.active(q):
        checks.paged("gqa_prefill", fb.block_tables, fb.seq_lens, pages[0])
    kernels().gqa_prefill(out, q, *pages, fb.block_tables, fb.q_start_loc, fb.seq_lens,
                          fb.tile_seq, fb.tile_q0, spec.heads, spec.mask, spec.scale, sinks,
                          spec.softcap, dist, gate, bounded)
    return out
