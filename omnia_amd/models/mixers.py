"""Mixers of layer-list models: how each one packs its checkpoint tensors, what it
keeps per token or per sequence, and how it runs a step.

A mixer projects the (normed) input of every row of a step -- decode rows first, then
prefill portions -- with one fused weight ``in``; ``mix(w, x, fb, cache)`` takes the
projected rows to the input of its output projection ``o``, and pages and states advance
in place; ``sublayer`` returns the operands of the residual kernel that follows.  All
padding happens in ``pack`` (zero weight rows and columns), so the kernels only see
aligned sizes.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F

from .. import ops
from ..ops import mixers as mops
from .layers import GQA_WIDTHS


def _pad2(w: torch.Tensor, rows: int, cols: int) -> torch.Tensor:
    return F.pad(w, (0, cols - w.shape[1], 0, rows - w.shape[0]))


def _head_cols(w: torch.Tensor, heads: int, width: int, d: int) -> torch.Tensor:
    """[d, H*V] output projection -> [d_pad, H*width], each head's columns padded."""
    V = w.shape[1] // heads
    t = F.pad(w.view(w.shape[0], heads, V), (0, width - V)).reshape(w.shape[0], heads * width)
    return _pad2(t, d, t.shape[1]).contiguous()


def _rows_to(ws: list[torch.Tensor], d: int) -> torch.Tensor:
    """Row-concatenated projections over the padded width ``d``, a multiple of 8 rows;
    of 256 (whole column tiles of the prefill GEMM) where that adds little."""
    w = torch.cat(ws)
    n = w.shape[0]
    up = (n + 255) // 256 * 256
    return _pad2(w, up if up * 16 <= n * 17 else (n + 7) // 8 * 8, d).contiguous()


def rotary_table(rot, positions: int, device) -> torch.Tensor:
    """fp32 [positions, dims] = (cos | sin), angles in double precision."""
    ang = torch.outer(torch.arange(positions, dtype=torch.float64),
                      torch.tensor(rot.frequencies(), dtype=torch.float64))
    return (torch.cat([ang.cos(), ang.sin()], 1) * rot.magnitude).float().to(device)


class Mixer:
    cache_tensors = 0, 0  # page and state tensors of its cache entry
    slab_input = False  # its kernels also reduce split-K slabs of a prefill projection
    slab_decode = False  # ... of a decode step's

    def __init__(self, spec, model):
        self.spec, self.model = spec, model

    def inputs(self, w: dict, h: torch.Tensor, is_decode: bool) -> torch.Tensor:
        if self.slab_input or (is_decode and self.slab_decode):
            return self.model._slabs("in", h, w["in"], is_decode)
        return self.model.project(h, w["in"], is_decode)

    def forward(self, w: dict, h: torch.Tensor, fb, cache) -> torch.Tensor:
        return self.mix(w, self.inputs(w, h, fb.is_decode), fb, cache)

    def output(self, w: dict, y: torch.Tensor, is_decode: bool, tag: str = "o") -> dict:
        return {"m": self.model._slabs(tag, y, w["o"], is_decode), "bias": w.get("o_b")}

    def sublayer(self, w: dict, h: torch.Tensor, fb, cache) -> dict:
        return self.output(w, self.forward(w, h, fb, cache), fb.is_decode)


class LatentAttention(Mixer):
    """Low-rank latent attention over one shared cached row per token.  Decode
    attends in the latent space (absorbed queries); bf16 prefill expands keys and
    values of each sequence's visible range and attends per head."""

    cache_tensors = 1, 0

    def __init__(self, spec, model):
        super().__init__(spec, model)
        self.table = model.rotary(spec.rotary)
        gpu16 = model.device.type == "cuda" and model.dtype == torch.bfloat16
        self.mfma_decode = gpu16 and mops.latent_decode_covers(spec)
        from .layers import QK_WIDTHS, V_WIDTHS

        self.mfma_prefill = gpu16 and spec.qk_pad in QK_WIDTHS and spec.v_pad in V_WIDTHS

    def pack(self, get, d: int) -> dict:
        s = self.spec
        H, D, R, C = s.heads, s.dim, s.rot_dim, s.kv_rank
        dkv = get("dkv")
        uq = get("uq").view(H, D + R, s.q_rank)
        kr, qr = dkv[C:], uq[:, D:]
        if s.rotary.interleaved:  # neighbours to halves: scores do not see a common order
            kr, qr = (torch.cat([t[..., 0::2, :], t[..., 1::2, :]], -2) for t in (kr, qr))
        wq = uq.new_zeros(H, s.qk_pad, s.q_rank_pad)
        wq[:, :D, :s.q_rank] = uq[:, :D]
        wq[:, s.dim_pad:s.dim_pad + R, :s.q_rank] = qr
        uk = F.pad(get("uk").view(H, D, C), (0, s.latent_pad - C, 0, s.dim_pad - D))
        # absorbed form: whole 32-wide k-steps (the columns past dim_pad meet the rotated
        # part of the query row with zero weight)
        ua = F.pad(uk, (0, 0, 0, -s.dim_pad % 32))
        uv = F.pad(get("uv").view(H, s.vdim, C), (0, s.latent_pad - C, 0, s.v_pad - s.vdim))
        return {
            "in": _rows_to([_pad2(get("dq"), s.q_rank_pad, d), _pad2(dkv[:C], s.latent_pad, d),
                            _pad2(kr, s.rot_pad, d), _pad2(get("g"), H, d)], d),
            "q_norm": get("dq.norm").float(), "kv_norm": get("dkv.norm").float(),
            "uq": wq.view(H * s.qk_pad, s.q_rank_pad),
            "uk_absorb": ua.transpose(1, 2).contiguous(),  # [H, latent, dim]
            "uk": uk.reshape(H * s.dim_pad, s.latent_pad).contiguous(),
            "uv": uv.contiguous(),
            "o": _head_cols(get("o"), H, s.v_pad, d),
        }

    def alloc(self, num_blocks: int, block_size: int, n_slots: int):
        # zeros: the padding columns of a row are never written, and a page's unwritten
        # rows stay finite under the masked tail of a tile
        return (torch.zeros(num_blocks, block_size, self.spec.padded_cache_width,
                            dtype=self.model.dtype, device=self.model.device),), None

    def splits(self, rows: int, max_keys: int) -> int:
        """Parts each row's keys are cut into: enough workgroups to fill the chip."""
        s = self.spec
        keys = min(max_keys, s.window) if s.window else max_keys
        groups = rows * -(-s.heads // (32 if s.heads > 16 else 16))
        return max(1, min(-(-512 // groups), -(-keys // 128), 32))

    def _decode(self, w, q, gate, pages, bt, positions, out):
        s = self.spec
        qa = mops.latent_absorb(q, w["uk_absorb"], s, positions, self.table)
        if self.mfma_decode and pages.shape[1] & (pages.shape[1] - 1) == 0:
            o = mops.latent_decode(qa, pages, bt, positions, s,
                                   self.splits(q.shape[0], bt.shape[1] * pages.shape[1]))
        else:
            o = mops.latent_attend(qa, pages, bt, None, positions, s)
        return mops.latent_expand(o, w["uv"], s, gate, out)

    def _prefill(self, w, q, gate, pages, fb, positions, out):
        s = self.spec
        if not self.mfma_prefill:
            qa = mops.latent_absorb(q, w["uk_absorb"], s, positions, self.table)
            o = mops.latent_attend(qa, pages, fb.block_tables, fb.q_start_loc, positions, s)
            return mops.latent_expand(o, w["uv"], s, gate, out)
        mops.latent_rotate(q, s, positions, self.table)
        c, kr = mops.latent_gather(pages, fb.block_tables, fb.kv_start, fb.kv_first, fb.seq_lens,
                                   fb.kv_rows, s)
        kx = ops.linear(c, w["uk"])
        # values transposed ([head dims, keys]): the product with swapped operands
        vt = ops.linear(w["uv"].view(s.heads * s.v_pad, s.latent_pad), c)
        return mops.latent_prefill(q, kx, kr, vt, fb, s, gate, out)

    def mix(self, w: dict, x: torch.Tensor, fb, cache) -> torch.Tensor:
        s, m = self.spec, self.model
        (pages,), _ = cache
        cq = mops.latent_prep(pages, x, w["q_norm"], w["kv_norm"], fb.positions, fb.slots,
                              self.table, s.q_rank_pad, s.latent_pad, m.cfg.rms_eps)
        q = m.project(cq, w["uq"], fb.is_decode)
        g0 = s.q_rank_pad + s.latent_pad + s.rot_pad
        gate = x[:, g0:g0 + s.heads]
        if fb.is_decode:
            return self._decode(w, q, gate, pages, fb.block_tables, fb.positions, None)
        nd, T = fb.num_decode, x.shape[0]
        if not nd:
            return self._prefill(w, q, gate, pages, fb, fb.positions, None)
        out = torch.empty(T, s.heads * s.v_pad, dtype=x.dtype, device=x.device)
        self._decode(w, q[:nd], gate[:nd], pages, fb.dec_block_tables, fb.positions[:nd],
                     out[:nd])
        if T > nd:
            self._prefill(w, q[nd:], gate[nd:], pages, fb, fb.positions[nd:], out[nd:])
        return out


class GatedDelta(Mixer):
    """Gated delta rule with short convolutions; a state slot per sequence."""

    cache_tensors = 0, 2

    def pack(self, get, d: int) -> dict:
        s = self.spec
        return {
            "in": _rows_to([_pad2(get(n), get(n).shape[0], d) for n in "qkvgba"], d),
            "conv": torch.cat([get(n + ".conv") for n in "qkv"]).contiguous(),
            "a_log": get("A_log").float(), "dt_bias": get("dt_bias").float(),
            "norm": get("norm").float(),
            "o": _head_cols(get("o"), s.heads, s.v_pad, d),
        }

    def alloc(self, num_blocks: int, block_size: int, n_slots: int):
        s, m = self.spec, self.model
        return None, (torch.zeros(n_slots, s.heads, s.dim, s.v_state_pad, dtype=torch.float32,
                                  device=m.device),
                      torch.zeros(n_slots, s.conv - 1, s.conv_channels, dtype=m.dtype,
                                  device=m.device))

    def mix(self, w: dict, x: torch.Tensor, fb, cache) -> torch.Tensor:
        s, m = self.spec, self.model
        _, (state, conv) = cache
        eps = m.cfg.rms_eps
        if fb.is_decode:
            return mops.delta_rule(x, w, s, state, conv, None, fb.positions, fb.state_slots, eps)
        nd, T = fb.num_decode, x.shape[0]
        if not nd:
            return mops.delta_rule(x, w, s, state, conv, fb.q_start_loc, fb.positions,
                                   fb.state_slots, eps)
        y = torch.empty(T, s.heads * s.v_pad, dtype=x.dtype, device=x.device)
        mops.delta_rule(x[:nd], w, s, state, conv, None, fb.positions[:nd], fb.state_slots[:nd],
                        eps, y[:nd])
        if T > nd:
            mops.delta_rule(x[nd:], w, s, state, conv, fb.q_start_loc, fb.positions[nd:],
                            fb.state_slots[nd:], eps, y[nd:])
        return y


class Lightning(Mixer):
    """Fixed-decay linear attention; a state slot per sequence."""

    cache_tensors = 0, 1
    slab_decode = True

    def pack(self, get, d: int) -> dict:
        s = self.spec

        def heads(n, dim, pad):
            t = get(n).view(s.heads, dim, -1)
            return F.pad(t, (0, d - t.shape[2], 0, pad - dim)).reshape(s.heads * pad, d)

        D, Dp, V, Vp = s.dim, s.dim_pad, s.vdim, s.v_pad
        norm = F.pad(get("norm").float().view(s.heads, V), (0, Vp - V)).reshape(-1)
        return {"in": _rows_to([heads("q", D, Dp), heads("k", D, Dp), heads("v", V, Vp),
                                heads("g", V, Vp)], d),
                "norm": norm.contiguous(), "pow": mops.decay_powers(s.decay, self.model.device),
                "o": _head_cols(get("o"), s.heads, Vp, d)}

    def alloc(self, num_blocks: int, block_size: int, n_slots: int):
        s, m = self.spec, self.model
        return None, (torch.zeros(n_slots, s.heads, s.dim_pad, s.v_pad, dtype=torch.float32,
                                  device=m.device),)

    def mix(self, w: dict, x: torch.Tensor, fb, cache) -> torch.Tensor:
        s, m = self.spec, self.model
        _, (state,) = cache
        pos, slots, eps = fb.positions, fb.state_slots, m.cfg.rms_eps
        if fb.is_decode:
            return mops.lightning(x, w, s, state, None, pos, slots, eps, m.dtype)
        nd, T = fb.num_decode, x.shape[0]
        if not nd:
            return mops.lightning(x, w, s, state, fb.q_start_loc, pos, slots, eps, m.dtype)
        y = torch.empty(T, s.heads * s.v_pad, dtype=m.dtype, device=x.device)
        mops.lightning(x[:nd], w, s, state, None, pos[:nd], slots[:nd], eps, m.dtype, y[:nd])
        if T > nd:
            mops.lightning(x[nd:], w, s, state, fb.q_start_loc, pos[nd:], slots[nd:], eps,
                           m.dtype, y[nd:])
        return y


class GroupedQueryAttention(Mixer):
    """Masked attention over pages of keys and values -- its own, or (spec ``kv_from``) those
    of an earlier layer, whose cache entry it is handed; with or without sinks, query
    temperature, capped scores, distance bias and gated heads."""

    cache_tensors = 2, 0
    slab_input = slab_decode = True

    def __init__(self, spec, model):
        super().__init__(spec, model)
        self.table = None if spec.rotary is None else model.rotary(spec.rotary)
        self.temp = None if spec.temperature is None else model.temperature(spec.temperature)
        self.mfma = (model.device.type == "cuda" and model.dtype == torch.bfloat16
                     and spec.dim_pad in GQA_WIDTHS and spec.v_pad in GQA_WIDTHS)

    def pack(self, get, d: int) -> dict:
        s = self.spec
        own = s.kv_from is None

        def heads(n, count, dim, pad):
            t = get(n).view(count, dim, -1)
            return F.pad(t, (0, d - t.shape[2], 0, pad - dim)).reshape(count * pad, d)

        def norm(n):
            t = get(n) if s.qk_norm == "weight" else torch.ones(s.dim, device=self.model.device)
            return F.pad(t.float(), (0, s.dim_pad - s.dim)).contiguous()

        def bias(n, count, dim, pad):
            if n not in s.bias:
                return torch.zeros(count * pad, device=self.model.device)
            return F.pad(get(n + ".b").float().view(count, dim), (0, pad - dim)).reshape(-1)

        rows = [heads("q", s.heads, s.dim, s.dim_pad)]
        if own:
            rows += [heads("k", s.kv_heads, s.dim, s.dim_pad),
                     heads("v", s.kv_heads, s.vdim, s.v_pad)]
        if s.gate:
            rows.append(_pad2(get("g"), s.heads, d))
        w = {"in": _rows_to(rows, d), "o": _head_cols(get("o"), s.heads, s.v_pad, d),
             "sink": get("sink").float().contiguous() if s.sink == "learned" else
             torch.zeros(s.heads, device=self.model.device) if s.sink else None}
        if s.distance_bias:
            w["dist"] = torch.stack([get("r1").float(), get("r2").float()]).contiguous()
            w["bounded"] = mops.scores_bounded(s, w["dist"])
        if s.qk_norm:
            w["q_norm"] = norm("q.norm")
            if own:
                w["k_norm"] = norm("k.norm")
        if set(s.bias) & set("qkv"):
            bs = [bias("q", s.heads, s.dim, s.dim_pad)]
            if own:
                bs += [bias("k", s.kv_heads, s.dim, s.dim_pad),
                       bias("v", s.kv_heads, s.vdim, s.v_pad)]
            w["in_b"] = torch.cat(bs).contiguous()
        if "o" in s.bias:
            ob = get("o.b").float()
            w["o_b"] = F.pad(ob, (0, d - ob.numel())).contiguous()
        return w

    def alloc(self, num_blocks: int, block_size: int, n_slots: int):
        s, m = self.spec, self.model
        # zeros: the null page that padded rows read stays finite
        return tuple(torch.zeros(num_blocks, s.kv_heads, block_size, w, dtype=m.dtype,
                                 device=m.device) for w in (s.dim_pad, s.v_pad)), None

    # decode workgroups wanted before a row's keys are cut no further, and the fewest
    # keys of a part
    DECODE_GROUPS, MIN_PART, MAX_PART = 1024, 128, 1024

    def splits(self, rows: int, max_keys: int) -> int:
        s = self.spec
        keys = s.most_visible(max_keys)
        groups = rows * s.kv_heads * -(-(s.heads // s.kv_heads) // 8)
        return max(1, -(-keys // self.MAX_PART),
                   min(-(-self.DECODE_GROUPS // groups), -(-keys // self.MIN_PART)))

    def _decode(self, w, q, pages, bt, positions, out, gate=None):
        page, more = pages[0].shape[2], dict(out=out, dist=w.get("dist"), gate=gate)
        if self.mfma and page & (page - 1) == 0:
            return mops.gqa_decode(q, pages, bt, positions, self.spec, w["sink"],
                                   self.splits(q.shape[0], bt.shape[1] * page), **more)
        return mops.gqa_attend(q, pages, bt, None, positions, self.spec, w["sink"], **more)

    def _prefill(self, w, q, pages, fb, positions, out, gate=None):
        page, more = pages[0].shape[2], dict(out=out, dist=w.get("dist"), gate=gate)
        if self.mfma and page & (page - 1) == 0:
            return mops.gqa_prefill(q, pages, fb, self.spec, w["sink"],
                                    bounded=w.get("bounded", False), **more)
        return mops.gqa_attend(q, pages, fb.block_tables, fb.q_start_loc, positions, self.spec,
                               w["sink"], **more)

    def mix(self, w: dict, x: torch.Tensor, fb, cache) -> torch.Tensor:
        s, m = self.spec, self.model
        pages, _ = cache
        nd, T = fb.num_decode, fb.positions.numel()
        gate = torch.empty(T, s.heads, dtype=torch.float32, device=x.device) if s.gate else None
        q = mops.gqa_prep(x, w, s, pages if s.kv_from is None else None, fb.positions, fb.slots,
                          self.table, m.dtype, m.cfg.rms_eps, self.temp, gate)
        if fb.is_decode:
            return self._decode(w, q, pages, fb.block_tables, fb.positions, None, gate)
        if not nd:
            return self._prefill(w, q, pages, fb, fb.positions, None, gate)
        out = torch.empty(T, s.heads * s.v_pad, dtype=m.dtype, device=x.device)
        gd, gp = (None, None) if gate is None else (gate[:nd], gate[nd:])
        self._decode(w, q[:nd], pages, fb.dec_block_tables, fb.positions[:nd], out[:nd], gd)
        if T > nd:
            self._prefill(w, q[nd:], pages, fb, fb.positions[nd:], out[nd:], gp)
        return out


class Parallel(Mixer):
    """Two mixers on the same input: one fused input projection, whose columns each takes
    its part of; their normed outputs meet in the residual kernel."""

    def __init__(self, spec, model):
        super().__init__(spec, model)
        self.left, self.right = (MIXERS[m.kind](m, model) for m in (spec.left, spec.right))
        both = (self.left, self.right)
        self.slab_input = all(m.slab_input for m in both)
        self.slab_decode = all(m.slab_decode for m in both)

    def pack(self, get, d: int) -> dict:
        sides, rows = {}, []
        for name, m in (("left", self.left), ("right", self.right)):
            w = m.pack(lambda n, p=name + ".": get(p + n), d)
            rows.append(w.pop("in")[:m.spec.in_cols])
            t = get(name + ".out").float()
            # the mean of the two: half of each weight
            sides[name] = w, mops.RMSNorm(F.pad(0.5 * t, (0, d - t.numel())).contiguous(),
                                          self.model.cfg.hidden_size, self.model.cfg.rms_eps)
        return {"in": _rows_to(rows, d), **sides}

    def alloc(self, num_blocks: int, block_size: int, n_slots: int):
        pages, states = (), ()
        for m in (self.left, self.right):
            p, s = m.alloc(num_blocks, block_size, n_slots)
            pages, states = pages + (p or ()), states + (s or ())
        return pages or None, states or None

    def sublayer(self, w: dict, h: torch.Tensor, fb, cache) -> dict:
        x = self.inputs(w, h, fb.is_decode)
        pages, states = cache
        np, ns, at, out = 0, 0, 0, []
        for name, m in (("left", self.left), ("right", self.right)):
            sub, norm = w[name]
            kp, ks = m.cache_tensors
            part = (pages[np:np + kp] if kp else None, states[ns:ns + ks] if ks else None)
            y = m.mix(sub, x[..., at:at + m.spec.in_cols], fb, part)
            o = m.output(sub, y, fb.is_decode, "o_" + name)
            out.append((o["m"], o["bias"], norm))
            np, ns, at = np + kp, ns + ks, at + m.spec.in_cols
        return {"branches": out}


MIXERS = {"latent_attention": LatentAttention, "delta": GatedDelta, "lightning": Lightning,
          "attention": GroupedQueryAttention, "parallel": Parallel}
