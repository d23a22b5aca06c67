"""Feed-forwards of layer-list models: how each one packs its checkpoint tensors and runs
a step.

``forward(w, h, is_decode)`` returns the operands of the residual kernel that follows:
``{"m": projection, slabs or per-slot parts, "bias": ..., "slots": ..., ...}``.  Padding
happens in ``pack``, as in the mixers.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F

from .. import ops
from ..ops import mixers as mops


def _up8(n: int) -> int:
    return (n + 7) // 8 * 8


class DenseGLU:
    """``W_down(act(W_gate h + b) * (W_up h + b)) + b``, silu or gelu, biases or none."""

    def __init__(self, spec, model, tag: str = ""):
        self.spec, self.model, self.tag = spec, model, tag

    def pack(self, get, d: int) -> dict:
        ff = _up8(self.spec.ff)

        def rows(n):
            t = get(n)
            return F.pad(t, (0, d - t.shape[1], 0, ff - t.shape[0]))

        def vec(n, width):
            t = get(n).float()
            return F.pad(t, (0, width - t.numel())).contiguous()

        down = get("down")
        w = {"gate_up": torch.cat([rows("gate"), rows("up")]).contiguous(),
             "gate_up_b": None, "down_b": None,
             "down": F.pad(down, (0, ff - down.shape[1], 0, d - down.shape[0])).contiguous()}
        if self.spec.bias:
            w["gate_up_b"] = torch.cat([vec("gate.b", ff), vec("up.b", ff)])
            w["down_b"] = vec("down.b", d)
        return w

    def _act(self, h, w: dict, is_decode) -> torch.Tensor:
        """One fused prefill GEMM, or a GEMM whose bias / activation kernel also reduces
        split-K slabs."""
        m, W, b, act = self.model, w["gate_up"], w["gate_up_b"], self.spec.act
        M, K = h.shape
        N = W.shape[0]
        if m._pgemm_ok(M, K, N // 2, is_decode, 128) and (b is None or act == "silu"):
            return ops.pgemm(1, h, W, bias=b, gelu=act == "gelu_tanh")
        cfg = m._wcfg(M, N // 2, K, 1, is_decode)
        if cfg is not None:  # a tuned SwiGLU shape, as slabs (bias and activation follow)
            nw, nwaves, S = cfg
            p = m._wgemm(2, h, W, S, nw, nwaves,
                         out=m._parts(self.tag + "gu", S, M, N, m._slab_dtype(nwaves)))
        else:
            p = m._slabs(self.tag + "gate_up", h, W, is_decode)
        return mops.glu(p, b, m.dtype, act)

    def forward(self, w: dict, h: torch.Tensor, is_decode: bool) -> dict:
        a = self._act(h, w, is_decode)
        return {"m": self.model._slabs(self.tag + "down", a, w["down"], is_decode),
                "bias": w["down_b"]}


class Experts:
    """Sparse mixture of small feed-forwards (grouped MFMA kernels, no host sync), with a
    shared one for every token if asked."""

    def __init__(self, spec, model):
        self.spec, self.model = spec, model
        self.shared = None if spec.shared is None else DenseGLU(spec.shared, model, "shared_")

    def pack(self, get, d: int) -> dict:
        s, m = self.spec, self.model
        E, ff, fp = s.experts, s.ff, s.ff_pad
        r = get("router")
        ups = ["gate", "up"] if s.gated else ["up"]  # rows of one expert's first product
        up = torch.zeros(E, len(ups) * fp, d, dtype=m.dtype, device=m.device)
        down = torch.zeros(E, d, fp, dtype=m.dtype, device=m.device)
        for e in range(E):
            for i, n in enumerate(ups):
                t = get(f"e{e}.{n}")
                up[e, i * fp:i * fp + ff, :t.shape[1]] = t
            t = get(f"e{e}.down")
            down[e, :t.shape[0], :ff] = t
        w = {"router": F.pad(r, (0, d - r.shape[1])).contiguous(), "up": up, "down": down}
        if s.correction:
            w["correction"] = get("correction").float().contiguous()
        if s.router_bias:
            w["router_b"] = get("router.b").float().contiguous()
        if self.shared is not None:
            w["shared"] = self.shared.pack(lambda n: get("shared." + n), d)
        return w

    def forward(self, w: dict, h: torch.Tensor, is_decode: bool) -> dict:
        parts, ids, wts = mops.experts(h, w, self.spec)
        out = {"m": parts, "slots": True}
        if self.spec.identity:
            out["identity"] = (ids, wts, h, self.spec.experts)
        if self.shared is not None:
            out["shared"] = self.shared.forward(w["shared"], h, is_decode)["m"]
        return out


MLPS = {"dense": DenseGLU, "moe": Experts}
