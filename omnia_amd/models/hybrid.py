"""Layer-list models (``ModelConfig.layers``) on the engine's paged cache: Sivadra, Sekazen,
Bisuzen, Tarunex.

Every layer is ``x += post(mixer(pre(x)))`` and, with a feed-forward,
``x += post(ff(pre(x)))`` around an fp32 residual stream; mixers
(:mod:`omnia_amd.models.mixers`) and feed-forwards (:mod:`omnia_amd.models.feedforward`)
are chosen per layer, norms and head per family (``layers.DesignSpec``; either norm may be
missing).  The post-norm, the residual update and the next sublayer's pre-norm are one
kernel behind each sublayer, which also reduces split-K slabs, sums a token's experts or
joins the two branches of a parallel mixer:

    norm_embed -> [ in GEMM -> mixer kernels -> o GEMM -> norm_residual
                    (-> feed-forward -> norm_residual) ] * layers -> head GEMM
                    (-> softcap)

In a family with ``joined`` sublayers a layer is ``x += mixer(norm1(x)) + ff(norm2(x))``: one
kernel behind both adds their outputs (a token's experts and the shared one among them),
what a loop's pass enters with, and writes the next layer's two inputs.

A layer may use another layer's tensors (its pages / state are its own; the later passes
of a looped layer do), or attend to another layer's pages.  bf16 models keep what feeds a
softmax, a router or a recurrence in fp32; fp32 models run every kernel and GEMM in fp32.
"""
from __future__ import annotations

import math
import os
from dataclasses import dataclass

import torch
import torch.nn.functional as F

from .. import ops
from ..ops import mixers as mops
from ..parallel import state as pstate
from ..parallel.overlap import side_stream
from .config import ModelConfig
from .feedforward import MLPS
from .layers import tensor_shapes
from .mixers import MIXERS, rotary_table
from .projection import Parts, Projections


# rows of a decode step, and of any other, that run a joined layer's sublayers on two
# streams: below, an eager step waits for its launches; above, either one fills the chip
FORK_DECODE = int(os.environ.get("OMNIA_FORK_DECODE", "256"))
FORK_PREFILL = 1024, int(os.environ.get("OMNIA_FORK_PREFILL", "8192"))


@dataclass
class HybridCache:
    """Per layer: the page tensors [num_blocks, ...] of an attention layer, or the
    (recurrent state, convolution inputs) pools of a recurrent one, indexed by the
    sequence's state slot.  A layer that borrows another one's keys and values has that
    layer's entry.  Block 0 is the null page of padded rows; slot 0 is unused (padded
    rows carry slot -1)."""

    layers: list  # (page tensors | None, (state, conv) | None)
    block_size: int
    num_blocks: int
    n_slots: int

    def page_tensors(self) -> list:
        seen = {id(t): t for pages, _ in self.layers if pages is not None for t in pages}
        return list(seen.values())

    def state_tensors(self) -> list:
        return [t for _, st in self.layers if st is not None for t in st]


def random_tensor(name: str, shape: tuple, cfg: ModelConfig, gen, device) -> torch.Tensor:
    """Random-init checkpoint tensor (no checkpoint at hand), fp32."""
    leaf = name.split(".", 1)[1] if "." in name else name
    leaf = leaf.replace("mix.left.", "mix.").replace("mix.right.", "mix.")
    if leaf.endswith("alpha"):
        return torch.full(shape, 0.5, device=device)
    if leaf in ("mix.r1", "mix.r2"):
        return torch.empty(shape, device=device).uniform_(0.05, 1.0, generator=gen)
    if leaf == "mix.sink" or (cfg.design.norm == "rms" and leaf.startswith("norm")):
        return torch.zeros(shape, device=device)  # norm weights stored around zero
    if leaf.startswith("norm") or name.startswith("final.") or leaf.endswith(".norm"):
        return torch.zeros(shape, device=device) if leaf.endswith(".b") else \
            torch.ones(shape, device=device)
    t = torch.empty(shape, device=device)
    if leaf in ("mix.norm", "mix.out"):
        return t.fill_(1.0)
    if leaf == "mix.A_log":
        return t.uniform_(1.0, 16.0, generator=gen).log_()
    if leaf == "mix.dt_bias":  # softplus^-1 of step sizes in [1e-3, 1e-1]
        dt = t.uniform_(math.log(1e-3), math.log(1e-1), generator=gen).exp_()
        return dt + torch.log(-torch.expm1(-dt))
    if leaf.endswith(".b") or leaf == "mlp.correction":
        return t.zero_()
    if leaf.endswith(".conv"):
        return t.normal_(0.0, shape[1] ** -0.5, generator=gen)
    std = 0.02
    if leaf == "mix.o" or leaf.endswith("down"):
        std /= math.sqrt(2 * cfg.num_layers)
    return t.normal_(0.0, std, generator=gen)


class HybridModel(Projections):
    q_tile = 128  # query rows of one prefill attention tile (latent.hip, gqa_prefill.hip)

    def __init__(self, cfg: ModelConfig, device="cpu", dtype=torch.bfloat16, seed: int = 0,
                 weights=None, decode_part_size: int = 512):
        if not cfg.layers:
            raise ValueError(f"{cfg.name}: no layers")
        st = pstate.get_state()
        if st.tp_size != 1:
            raise ValueError("layer-list models run on one GPU per replica (tp = 1)")
        self.tp, self.tpr = 1, 0
        self.cfg, self.device, self.dtype, self.seed = cfg, torch.device(device), dtype, seed
        self.stateful = cfg.stateful
        # prefill works on a dense copy of each portion's visible keys
        self.key_ranges = any(l.mixer.kind == "latent_attention" for l in cfg.layers)
        self.vocab_local, self.vocab_start = cfg.vocab_size, 0
        # padded width (zero columns stay zero): whole k-tiles of the grouped expert GEMMs
        m = 64 if any(l.mlp is not None and l.mlp.kind == "moe" for l in cfg.layers) else 8
        self.d = -(-cfg.hidden_size // m) * m
        self._ws: dict = {}
        self._tables: dict = {}
        self.mixers = [MIXERS[l.mixer.kind](l.mixer, self) for l in cfg.layers]
        self.mlps = [None if l.mlp is None else MLPS[l.mlp.kind](l.mlp, self)
                     for l in cfg.layers]
        if cfg.design.joined and any("o" in getattr(l.mixer, "bias", "") or
                                     getattr(l.mlp, "bias", False) for l in cfg.layers):
            raise ValueError(f"{cfg.name}: joined sublayers have no output biases")
        self.w = self._pack(weights if weights is not None else self._random())
        for branch in range(2 if cfg.design.joined else 1):
            ops.dgemm_prepare(self.device, branch)

    # ------------------------------------------------------------ weights
    def rotary(self, rot) -> torch.Tensor:
        if rot not in self._tables:
            self._tables[rot] = rotary_table(rot, self.cfg.max_position, self.device)
        return self._tables[rot]

    def _random(self):
        cfg = self.cfg
        shapes = tensor_shapes(cfg.layers, cfg.hidden_size, cfg.vocab_size, cfg.design)
        g = torch.Generator(device=self.device).manual_seed(self.seed)

        def get(name):
            return random_tensor(name, shapes[name], cfg, g, self.device)

        return get

    def _pack(self, get) -> dict:
        """``get(name)`` -> checkpoint tensor; kernel-ready weights."""
        cfg, d, dev, design = self.cfg, self.d, self.device, self.cfg.design
        seen: dict = {}

        def raw(name):
            return get(name).to(device=dev, dtype=self.dtype)

        def part(prefix):
            made: dict = {}

            def one(n):
                if n not in made:
                    made[n] = raw(prefix + n)
                return made[n]

            return one

        def vec(t):
            t = t.float()
            return F.pad(t, (0, d - t.numel())).contiguous()

        def norm(name, scale=1.0):
            if name is None:
                return None
            if design.norm == "tanh":
                return mops.TanhNorm(float(raw(name + ".alpha")), scale * vec(raw(name)),
                                     scale * vec(raw(name + ".b")))
            if design.norm == "rms_scalar":
                return mops.RMSNorm(None, cfg.hidden_size, cfg.rms_eps, scale * float(raw(name)))
            return mops.RMSNorm(scale * vec(1.0 + raw(name).float()), cfg.hidden_size, cfg.rms_eps)

        def norms(p, k):
            return [norm(p + n if n else None) for n in design.sublayer_norms(k)]

        def cols(t):
            return F.pad(t, (0, d - t.shape[1])).contiguous()

        w = {"embed": cols(raw("embed")), "layers": [],
             # the head is linear: its scale rides the norm before it
             "final_norm": norm("final.norm", cfg.logit_scale),
             "embed_norm": norm("embed.norm") if design.embed_norm else None}
        w["head"] = w["embed"] if design.tied else cols(raw("head"))
        if design.pass_inputs and any(l.starts is not None for l in cfg.layers):
            w["step"] = [vec(t) for t in raw("loop.step")]
        for i, l in enumerate(cfg.layers):
            own = i if l.weights_of is None else l.weights_of
            if own not in seen:
                n = cfg.layers[own].index
                p = f"l{own if n is None else n}."
                layer = {"mix": self.mixers[i].pack(part(p + "mix."), d), "mlp": None}
                layer["pre1"], layer["post1"] = norms(p, 1)
                if l.mlp is not None:
                    layer["mlp"] = self.mlps[i].pack(part(p + "mlp."), d)
                    layer["pre2"], layer["post2"] = norms(p, 2)
                seen[own] = layer
            w["layers"].append(seen[own])
        return w

    # ------------------------------------------------------------ cache
    def allocate_cache(self, num_blocks: int, block_size: int, n_slots: int) -> HybridCache:
        layers: list = []
        for m in self.mixers:
            j = m.spec.kv_from
            layers.append(m.alloc(num_blocks, block_size, n_slots) if j is None else layers[j])
        return HybridCache(layers, block_size, num_blocks, n_slots)

    # ------------------------------------------------------------ forward
    def project(self, x: torch.Tensor, w: torch.Tensor, is_decode: bool) -> torch.Tensor:
        """A projection whose consumer reads plain rows (no split-K slabs)."""
        if self._pgemm_ok(x.shape[0], x.shape[1], w.shape[0], is_decode):
            return ops.pgemm(0, x, w)
        return ops.linear(x, w)

    def _slabs(self, tag, x, w, is_decode) -> torch.Tensor:
        """A projection whose consumer also reduces split-K slabs."""
        m = self._proj(tag, x, w, is_decode)
        return m.t if isinstance(m, Parts) else m

    def temperature(self, t) -> torch.Tensor:
        if t not in self._tables:
            self._tables[t] = mops.temperature_table(t, self.cfg.max_position, self.device)
        return self._tables[t]

    def _pass_input(self, fb, i: int) -> mops.PassInput | None:
        """What joins the residual before layer ``i``: at the first layer the embedding, and
        where a loop's pass starts its inputs."""
        t = None
        if self.cfg.design.pass_inputs and i < len(self.cfg.layers):
            t = self.cfg.layers[i].starts
        if i and t is None:
            return None
        return mops.PassInput(fb.input_ids, self.w["embed"], self.cfg.vocab_size,
                              self.cfg.embed_scale if i == 0 or t else 0.0,
                              None if t is None else self.w["step"][t], fb.ids_src, fb.tok_slots)

    def _run_joined(self, fb, kv: HybridCache, trace: list | None) -> torch.Tensor:
        ws, dt, dec = self.w["layers"], self.dtype, fb.is_decode
        x = torch.empty(fb.input_ids.numel(), self.d, dtype=torch.float32, device=self.device)

        def norms(i):  # of layer i's sublayers, or the final one
            if i == len(ws):
                return [self.w["final_norm"]]
            return [ws[i]["pre1"]] + ([ws[i]["pre2"]] if self.mlps[i] else [])

        rows = x.shape[0]
        fork = x.is_cuda and (rows <= FORK_DECODE if dec else
                              FORK_PREFILL[0] <= rows <= FORK_PREFILL[1])
        h = mops.joined_residual(x, [], norms(0), dt, self._pass_input(fb, 0), fresh=True)
        for i, (w, mixer, mlp) in enumerate(zip(ws, self.mixers, self.mlps)):
            if fork and mlp:
                # the sublayers do not need each other: the feed-forward on a stream of its
                # own.  Tensors of either stream live until the streams have met
                main, side = torch.cuda.current_stream(), side_stream(self.device)
                side.wait_stream(main)
                with ops.on_branch(1, side):
                    f = mlp.forward(w["mlp"], h[1], dec)
                y = mixer.sublayer(w["mix"], h[0], fb, kv.layers[i])["m"]
                main.wait_stream(side)
            else:
                y = mixer.sublayer(w["mix"], h[0], fb, kv.layers[i])["m"]
                f = mlp.forward(w["mlp"], h[1], dec) if mlp else None
            parts = [(y, False)]
            if mlp:
                parts.append((f["m"], f.get("slots", False)))
                if "shared" in f:
                    parts.append((f["shared"], False))
            enter = self._pass_input(fb, i + 1)
            if trace is not None:
                mops.joined_residual(x, parts, norms(i + 1), dt)
                trace.append(x[:, :self.cfg.hidden_size].clone())
                parts = []
            h = mops.joined_residual(x, parts, norms(i + 1), dt, enter)
        return h[0]

    def run_layers(self, fb, kv: HybridCache, trace: list | None = None) -> torch.Tensor:
        """Final-normed rows of the step; ``trace`` receives the residual stream after
        every layer (tests)."""
        self._min_rows = self.PGEMM_MIXED_MIN_ROWS if fb.num_decode else self.PGEMM_MIN_ROWS
        if self.cfg.design.joined:
            return self._run_joined(fb, kv, trace)
        ws, dt, dec = self.w["layers"], self.dtype, fb.is_decode
        x, h = mops.norm_embed(fb.input_ids, self.w["embed"], self.cfg.vocab_size,
                               self.w["embed_norm"], ws[0]["pre1"], fb.ids_src, fb.tok_slots)
        for i, (w, mixer, mlp) in enumerate(zip(ws, self.mixers, self.mlps)):
            after = ws[i + 1]["pre1"] if i + 1 < len(ws) else self.w["final_norm"]
            h = mops.norm_residual(x, post=w["post1"], pre=w["pre2"] if mlp else after, dtype=dt,
                                   **mixer.sublayer(w["mix"], h, fb, kv.layers[i]))
            if mlp:
                h = mops.norm_residual(x, post=w["post2"], pre=after, dtype=dt,
                                       **mlp.forward(w["mlp"], h, dec))
            if trace is not None:
                trace.append(x[:, :self.cfg.hidden_size].clone())
        return h

    def logits(self, h: torch.Tensor, is_decode: bool = False) -> torch.Tensor:
        W = self.w["head"]
        cfg = self._wcfg(h.shape[0], W.shape[0], h.shape[1], 0, is_decode)
        if cfg is not None and cfg[2] == 1:
            z = ops.wgemm(0, h, W, 1, cfg[0], cfg[1])
        else:
            z = ops.linear(h, W)
        cap = self.cfg.logit_softcap
        return mops.softcap_(z, cap) if cap else z

    def forward(self, fb, kv: HybridCache, gather: bool = True) -> torch.Tensor:
        h = self.run_layers(fb, kv)
        if not (fb.is_decode and fb.logits_indices.shape[0] == h.shape[0]):
            h = h.index_select(0, fb.logits_indices)
        return self.logits(h, fb.is_decode)
