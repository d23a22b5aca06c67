"""Layer descriptions of layer-list models (``ModelConfig.layers``).

A layer-list model names, per layer, its mixer (a kind of attention or a
recurrence, with its own sizes and constants) and its feed-forward, instead of
repeating one block ``num_layers`` times.  The specs are plain frozen data: the
mechanisms behind them live in :mod:`omnia_amd.models.mixers`, and the reader of
the checkpoint's ``config.json`` builds them here.
"""
from __future__ import annotations

import math
from dataclasses import dataclass


# head widths the MFMA prefill attention is instantiated for (latent.hip); wider
# heads run the generic kernel
QK_WIDTHS = (32, 64, 96, 128, 192, 256)
V_WIDTHS = (32, 64, 128)
# key / value widths of the MFMA grouped-query kernels (gqa.hip, gqa_prefill.hip)
GQA_WIDTHS = (32, 64, 96, 128, 192, 256)
# cached row widths of the MFMA decode attention
LATENT_WIDTHS = (64, 96, 128, 192, 256, 320, 448, 576, 640)


def _up(n: int, m: int) -> int:
    return (n + m - 1) // m * m


@dataclass(frozen=True)
class YarnSpec:
    """YaRN frequency interpolation: rotations slower than ``slow`` turns over
    ``original`` positions are slowed down by ``factor``, those faster than
    ``fast`` turns are kept, with a linear ramp over the dimensions between."""

    factor: float
    original: float
    fast: float = 32.0
    slow: float = 1.0


@dataclass(frozen=True)
class BandSpec:
    """Frequency scaling by wavelength (Llama 3.1): pairs that turn at least ``high``
    times over ``original`` positions keep their frequency, those that turn at most
    ``low`` times are slowed down by ``factor``, with a linear blend between."""

    factor: float
    low: float
    high: float
    original: float

    def apply(self, f: float) -> float:
        turns = self.original * f / (2.0 * math.pi)
        if turns > self.high:
            return f
        if turns < self.low:
            return f / self.factor
        s = (turns - self.low) / (self.high - self.low) if self.high > self.low else 1.0
        return (1.0 - s) * f / self.factor + s * f


@dataclass(frozen=True)
class RotarySpec:
    """Rotate-half rotary positions over ``dims`` dimensions."""

    dims: int
    base: float
    yarn: YarnSpec | None = None
    bands: BandSpec | None = None

    def frequencies(self) -> list[float]:
        """Angle per position of every rotated pair (double precision)."""
        n, base, y = self.dims, self.base, self.yarn
        freq = [base ** (-2.0 * i / n) for i in range(n // 2)]
        if self.bands is not None:
            freq = [self.bands.apply(f) for f in freq]
        if y is None:
            return freq

        def pair_of(turns: float) -> float:  # pair that makes `turns` turns over y.original
            return n * math.log(y.original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

        lo = max(math.floor(pair_of(y.fast)), 0)
        hi = min(math.ceil(pair_of(y.slow)), n - 1)
        width = max(hi - lo, 0.001)
        out = []
        for i, f in enumerate(freq):
            r = min(max((i - lo) / width, 0.0), 1.0)
            out.append(f / y.factor * r + f * (1.0 - r))
        return out

    @property
    def magnitude(self) -> float:
        """Factor on both cos and sin."""
        return 1.0 if self.yarn is None else 0.1 * math.log(self.yarn.factor) + 1.0


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Attention over a low-rank latent: per token the cache holds one normed
    latent of ``kv_rank`` numbers (every head's unrotated key and value are
    linear maps of it) and one rotated key part of ``rot_dim`` numbers shared by
    all heads.  ``window`` > 0 limits a query to its last ``window`` positions,
    itself included; 0 = the whole past."""

    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rotary: RotarySpec
    window: int = 0

    kind = "latent_attention"
    kv_from = None

    # Kernel geometry: every operand is zero-padded at load (weight rows / columns)
    # so that the MFMA tiles never see a ragged edge and rows stay 16-B aligned.
    @property
    def q_rank_pad(self) -> int:
        return _up(self.q_rank, 32)

    @property
    def dim_pad(self) -> int:  # unrotated part of a query / expanded key row
        return _up(self.dim, 8)

    @property
    def rot_pad(self) -> int:
        return _up(self.rot_dim, 8)

    @property
    def qk_pad(self) -> int:  # [dim_pad | rot_pad | 0] row of one head
        n = self.dim_pad + self.rot_pad
        return next((w for w in QK_WIDTHS if n <= w), _up(n, 32))

    @property
    def v_pad(self) -> int:
        return next((w for w in V_WIDTHS if self.vdim <= w), _up(self.vdim, 32))

    @property
    def latent_pad(self) -> int:
        return _up(self.kv_rank, 32)

    @property
    def padded_cache_width(self) -> int:
        """[latent_pad | rot_pad | 0]: one cached token row, and one absorbed query."""
        n = self.latent_pad + self.rot_pad
        return next((w for w in LATENT_WIDTHS if n <= w), _up(n, 32))


@dataclass(frozen=True)
class DeltaSpec:
    """Gated delta rule: per head a ``dim x vdim`` fp32 state, one decay and one
    step size per head and token; ``kv_heads`` query/key heads are shared by
    ``heads`` value heads; q, k and v pass a causal convolution of ``conv`` taps."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    kind = "delta"
    kv_from = None
    padded_cache_width = 0  # no pages

    @property
    def conv_channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def dim_pad(self) -> int:
        return _up(self.dim, 4)

    @property
    def v_state_pad(self) -> int:  # fp32 state row of one key dimension
        return _up(self.vdim, 4)

    @property
    def v_pad(self) -> int:  # one head of the output projection's input
        return _up(self.vdim, 8)


@dataclass(frozen=True)
class AttentionSpec:
    """Grouped-query attention over paged keys and values: ``kv_heads`` key/value heads
    shared by ``heads`` query heads, per-head RMS norms of queries and keys, rotary on
    the first ``rotary.dims`` dimensions, a sliding ``window`` (0 = the whole past) and,
    with ``sink``, a learned number per head in the softmax denominator.  ``kv_from``:
    the layer whose cached keys and values this one attends to instead of its own."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rotary: RotarySpec
    window: int = 0
    sink: bool = True
    kv_from: int | None = None

    kind = "attention"

    @property
    def dim_pad(self) -> int:
        return next((w for w in GQA_WIDTHS if self.dim <= w), _up(self.dim, 32))

    @property
    def v_pad(self) -> int:
        return next((w for w in GQA_WIDTHS if self.vdim <= w), _up(self.vdim, 32))

    @property
    def padded_cache_width(self) -> int:
        """Elements one token adds to the pages."""
        return 0 if self.kv_from is not None else self.kv_heads * (self.dim_pad + self.v_pad)


@dataclass(frozen=True)
class DenseMLPSpec:
    """``W_down(silu(W_gate h + b) * (W_up h + b)) + b``."""

    ff: int

    kind = "dense"


@dataclass(frozen=True)
class ExpertsSpec:
    """Mixture of ``experts`` clamped GLUs, ``top`` per token.  Routing scores are
    ``sigmoid`` or ``softmax`` of fp32 logits, renormalised over the chosen experts if
    asked; a token's weight multiplies its expert's input.  Expert:
    ``W_down(g sigmoid(alpha g) (u + 1))`` with ``g = min(W_gate h, limit)`` and
    ``u = clamp(W_up h, -limit, limit)``."""

    ff: int
    experts: int
    top: int
    limit: float
    alpha: float = 1.702
    score: str = "sigmoid"
    renorm: bool = False

    kind = "moe"

    @property
    def ff_pad(self) -> int:  # whole k-tiles of the grouped GEMMs
        return _up(self.ff, 64)


@dataclass(frozen=True)
class LayerSpec:
    mixer: object  # LatentAttentionSpec | DeltaSpec | AttentionSpec
    mlp: object | None = None  # DenseMLPSpec | ExpertsSpec | None
    weights_of: int | None = None  # share layer j's tensors (own cache / state)


@dataclass(frozen=True)
class DesignSpec:
    """What a layer-list family fixes around its layers."""

    norm: str  # "tanh": Dynamic Tanh; "rms": RMS with a weight stored around zero
    pre_norm: bool  # sublayers read the normed residual (else the residual itself)
    embed_norm: bool  # the residual starts at norm(embedding)
    tied: bool  # the embedding table is the output head

    def sublayer_norms(self, k: int) -> tuple[str | None, str]:
        """(pre, post) norm names of a layer's k-th sublayer (1 mixer, 2 feed-forward)."""
        return (f"norm{k}", f"norm{k}b") if self.pre_norm else (None, f"norm{k}")


DESIGNS = {
    "sivadra": DesignSpec("tanh", pre_norm=True, embed_norm=False, tied=False),
    "sekazen": DesignSpec("rms", pre_norm=False, embed_norm=True, tied=True),
}


# ------------------------------------------------------------ config.json reader
def _rotary(c: dict) -> RotarySpec:
    sc = c.get("scaling")
    yarn = bands = None
    if sc and "fast" in sc:
        yarn = YarnSpec(float(sc["factor"]), float(sc["original"]), float(sc["fast"]),
                        float(sc["slow"]))
    elif sc:
        bands = BandSpec(float(sc["factor"]), float(sc["low"]), float(sc["high"]),
                         float(sc["original"]))
    return RotarySpec(int(c["dims"]), float(c["base"]), yarn, bands)


def _latent_attention(c: dict) -> LatentAttentionSpec:
    mask = c.get("mask") or {}
    spec = LatentAttentionSpec(
        heads=int(c["heads"]), dim=int(c["dim"]), rot_dim=int(c["rot_dim"]),
        vdim=int(c["vdim"]), q_rank=int(c["q_rank"]), kv_rank=int(c["kv_rank"]),
        scale=float(c["scale"]), rotary=_rotary(c["rot"]), window=int(mask.get("size") or 0))
    if spec.rotary.dims != spec.rot_dim or spec.rot_dim % 2:
        raise ValueError(f"latent attention rotates its whole rot_dim part: rot.dims "
                         f"{spec.rotary.dims}, rot_dim {spec.rot_dim}")
    return spec


def _delta(c: dict) -> DeltaSpec:
    spec = DeltaSpec(heads=int(c["heads"]), kv_heads=int(c["kv_heads"]), dim=int(c["dim"]),
                     vdim=int(c["vdim"]), conv=int(c["conv"]))
    if spec.heads % spec.kv_heads:
        raise ValueError(f"delta: {spec.heads} heads over {spec.kv_heads} q/k heads")
    return spec


def _attention(c: dict) -> AttentionSpec:
    src = c.get("kv_from")
    spec = AttentionSpec(
        heads=int(c["heads"]), kv_heads=int(c["kv_heads"]), dim=int(c["dim"]),
        vdim=int(c["vdim"]), scale=float(c["scale"]), rotary=_rotary(c["rot"]),
        window=int((c.get("mask") or {}).get("size") or 0),
        kv_from=None if src is None else int(src))
    if spec.heads % spec.kv_heads:
        raise ValueError(f"attention: {spec.heads} heads over {spec.kv_heads} k/v heads")
    if spec.rotary.dims % 2 or not 0 < spec.rotary.dims <= spec.dim:
        raise ValueError(f"attention: rot.dims {spec.rotary.dims} of dim {spec.dim}")
    return spec


def _dense(c: dict) -> DenseMLPSpec:
    return DenseMLPSpec(int(c["ff"]))


def _experts(c: dict) -> ExpertsSpec:
    e, r = c["expert"], c["router"]
    spec = ExpertsSpec(ff=int(e["ff"]), experts=int(r["experts"]), top=int(r["top"]),
                       limit=float(e["limit"]))
    if not 1 <= spec.top <= min(spec.experts, 64) or spec.experts > 256:
        raise ValueError(f"moe: top {spec.top} of {spec.experts} experts")
    return spec


MIXER_SPECS = {"latent_attention": _latent_attention, "delta": _delta, "attention": _attention}
MLP_SPECS = {"dense": _dense, "moe": _experts}


def parse_layers(entries: list[dict]) -> tuple[LayerSpec, ...]:
    """``config.json`` ``layers`` -> specs.  ``weights_of`` chains are resolved to
    the layer that owns the tensors."""
    out: list[LayerSpec] = []
    for i, e in enumerate(entries):
        if e["type"] not in MIXER_SPECS:
            raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
        mlp = e.get("mlp")
        if mlp is not None and mlp.get("kind") not in MLP_SPECS:
            raise ValueError(f"layer {i}: unknown feed-forward {mlp.get('kind')!r}")
        owner = e.get("weights_of")
        if owner is not None:
            owner = int(owner)
            if not 0 <= owner < len(entries) or owner == i:
                raise ValueError(f"layer {i}: weights_of {owner}")
            seen = {i}
            while entries[owner].get("weights_of") is not None:
                if owner in seen:
                    raise ValueError(f"layer {i}: weights_of cycle")
                seen.add(owner)
                owner = int(entries[owner]["weights_of"])
        out.append(LayerSpec(MIXER_SPECS[e["type"]](e["mixer"]),
                             None if mlp is None else MLP_SPECS[mlp["kind"]](mlp), owner))
    for i, l in enumerate(out):
        if l.weights_of is not None:
            o = out[l.weights_of]
            if (o.mixer, o.mlp) != (l.mixer, l.mlp):
                raise ValueError(f"layer {i} differs from layer {l.weights_of} whose "
                                 "weights it uses")
        j = l.mixer.kv_from
        if j is not None:
            o = out[j].mixer if 0 <= j < i else None
            if o is None or o.kind != l.mixer.kind or o.kv_from is not None:
                raise ValueError(f"layer {i}: kv_from {j} names no earlier attention layer "
                                 "with keys and values of its own")
            m = l.mixer
            if (o.heads, o.kv_heads, o.dim, o.vdim, o.rotary) != (
                    m.heads, m.kv_heads, m.dim, m.vdim, m.rotary):
                raise ValueError(f"layer {i}: heads or rotation differ from layer {j} whose "
                                 "keys and values it uses")
    return tuple(out)


# --------------------------------------------------------------- tensor shapes
def _mixer_shapes(m, d: int) -> dict[str, tuple]:
    if m.kind == "latent_attention":
        return {"dq": (m.q_rank, d), "dq.norm": (m.q_rank,),
                "uq": (m.heads * (m.dim + m.rot_dim), m.q_rank),
                "dkv": (m.kv_rank + m.rot_dim, d), "dkv.norm": (m.kv_rank,),
                "uk": (m.heads * m.dim, m.kv_rank), "uv": (m.heads * m.vdim, m.kv_rank),
                "g": (m.heads, d), "o": (d, m.heads * m.vdim)}
    if m.kind == "attention":
        out = {"q": (m.heads * m.dim, d), "q.norm": (m.dim,), "o": (d, m.heads * m.vdim)}
        if m.kv_from is None:
            out.update({"k": (m.kv_heads * m.dim, d), "k.norm": (m.dim,),
                        "v": (m.kv_heads * m.vdim, d)})
        if m.sink:
            out["sink"] = (m.heads,)
        return out
    kd, hv = m.kv_heads * m.dim, m.heads * m.vdim
    return {"q": (kd, d), "q.conv": (kd, m.conv), "k": (kd, d), "k.conv": (kd, m.conv),
            "v": (hv, d), "v.conv": (hv, m.conv), "b": (m.heads, d), "A_log": (m.heads,),
            "norm": (m.vdim,), "a": (m.heads, d), "dt_bias": (m.heads,), "g": (hv, d),
            "o": (d, hv)}


def _mlp_shapes(m, d: int) -> dict[str, tuple]:
    if m.kind == "moe":
        out = {"router": (m.experts, d)}
        for e in range(m.experts):
            out.update({f"e{e}.gate": (m.ff, d), f"e{e}.up": (m.ff, d), f"e{e}.down": (d, m.ff)})
        return out
    return {"gate": (m.ff, d), "gate.b": (m.ff,), "up": (m.ff, d), "up.b": (m.ff,),
            "down": (d, m.ff), "down.b": (d,)}


def tensor_shapes(layers, d: int, vocab: int,
                  design: DesignSpec = DESIGNS["sivadra"]) -> dict[str, tuple]:
    """Every checkpoint tensor of a layer-list model and its shape."""

    def norm(name):
        if name is None:
            return {}
        if design.norm == "tanh":
            return {name: (d,), name + ".b": (d,), name + ".alpha": ()}
        return {name: (d,)}

    out = {"embed": (vocab, d)}
    if design.embed_norm:
        out.update(norm("embed.norm"))
    for i, l in enumerate(layers):
        if l.weights_of is not None:
            continue
        p = f"l{i}."
        for k, part in ((1, l.mixer), (2, l.mlp)):
            if part is None:
                continue
            for n in design.sublayer_norms(k):
                out.update(norm(p + n if n else None))
        out.update({p + "mix." + k: s for k, s in _mixer_shapes(l.mixer, d).items()})
        if l.mlp is not None:
            out.update({p + "mlp." + k: s for k, s in _mlp_shapes(l.mlp, d).items()})
    out.update(norm("final.norm"))
    if not design.tied:
        out["head"] = (vocab, d)
    return out
