"""Layer descriptions of layer-list models (``ModelConfig.layers``).

A layer-list model names, per layer, its mixer (a kind of attention or a
recurrence, with its own sizes and constants) and its feed-forward, instead of
repeating one block ``num_layers`` times.  The specs are plain frozen data: the
mechanisms behind them live in :mod:`omnia_amd.models.mixers`, and the reader of
the checkpoint's ``config.json`` builds them here.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, replace


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
    """Rotary positions over ``dims`` dimensions: pairs (i, i + dims / 2), or, if
    ``interleaved``, neighbours (2i, 2i + 1)."""

    dims: int
    base: float
    yarn: YarnSpec | None = None
    bands: BandSpec | None = None
    interleaved: bool = False

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
class TemperatureSpec:
    """Queries grow with their position p: times ``1 + coef ln(floor((p + 1) / every) + 1)``."""

    coef: float
    every: float

    def factor(self, p: int) -> float:
        return 1.0 + self.coef * math.log(math.floor((p + 1) / self.every) + 1.0)


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
    stateful = False

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
    stateful = True
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

    def state_bytes(self, dtype_bytes: int) -> int:
        """fp32 matrices and convolution inputs of one sequence."""
        return (4 * self.heads * self.dim * self.v_state_pad
                + dtype_bytes * (self.conv - 1) * self.conv_channels)


@dataclass(frozen=True)
class LightningSpec:
    """Linear attention with one fixed ``decay`` per head: a ``dim x vdim`` fp32 state
    ``S <- decay S + k v^T`` read as ``S^T q``, silu on q, k and v, one RMS norm over all
    heads together and a sigmoid output gate."""

    heads: int
    dim: int
    vdim: int
    decay: tuple

    kind = "lightning"
    kv_from = None
    stateful = True
    padded_cache_width = 0  # no pages

    # whole 16-B chunks of a projection row
    @property
    def dim_pad(self) -> int:
        return _up(self.dim, 8)

    @property
    def v_pad(self) -> int:
        return _up(self.vdim, 8)

    @property
    def in_cols(self) -> int:
        """[q | k | v | gate] of one projected row."""
        return 2 * self.heads * (self.dim_pad + self.v_pad)

    def state_bytes(self, dtype_bytes: int) -> int:
        return 4 * self.heads * self.dim_pad * self.v_pad


@dataclass(frozen=True)
class AttentionSpec:
    """Grouped-query attention over paged keys and values: ``kv_heads`` key/value heads
    shared by ``heads`` query heads.

    ``qk_norm``: per-head RMS norms of queries and keys, with a learned ``"weight"``,
    ``"unit"`` (none) or None.  ``rotary`` on the first ``rotary.dims`` dimensions, or
    None.  ``bias``: letters of the projections (q, k, v, o) that have one.  A query sees its
    last ``window`` positions (0 = the whole past) and the sequence's first ``keep_first``,
    or, with ``chunk``, the positions of its own chunk of that many up to itself.  ``sink``:
    a number per head in the softmax denominator beside the scores, ``"learned"``, ``"zero"``
    (one is added to the denominator) or None.  ``kv_from``: the layer whose cached keys and
    values this one attends to instead of its own.

    ``temperature`` scales queries by position.  Scores are capped, ``softcap tanh(s /
    softcap)`` (0: not), then lose ``r1 ln(1 + r2 (i - j))`` with two learned numbers per
    head (``distance_bias``).  ``gate``: a head's output times a sigmoid of the layer's
    input."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rotary: RotarySpec | None
    window: int = 0
    sink: str | None = "learned"
    kv_from: int | None = None
    qk_norm: str | None = "weight"
    bias: str = ""
    keep_first: int = 0
    chunk: int = 0
    temperature: TemperatureSpec | None = None
    softcap: float = 0.0
    distance_bias: bool = False
    gate: bool = False

    kind = "attention"
    stateful = False

    @property
    def mask(self) -> tuple[int, int, int]:
        return self.window, self.keep_first, self.chunk

    def most_visible(self, keys: int) -> int:
        """Most keys a query sees of a context of ``keys``."""
        if self.chunk:
            return min(keys, self.chunk)
        return min(keys, self.window + self.keep_first) if self.window else keys

    @property
    def in_cols(self) -> int:
        """[q | k | v | gate] of one projected row."""
        return self.qkv_cols + (self.heads if self.gate else 0)

    @property
    def qkv_cols(self) -> int:
        own = 0 if self.kv_from is not None else self.kv_heads * (self.dim_pad + self.v_pad)
        return self.heads * self.dim_pad + own

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
class ParallelSpec:
    """Two mixers side by side on the same input; their outputs, each RMS-normed over the
    model width, are averaged."""

    left: object
    right: object

    kind = "parallel"
    kv_from = None

    @property
    def stateful(self) -> bool:
        return self.left.stateful or self.right.stateful

    @property
    def padded_cache_width(self) -> int:
        return self.left.padded_cache_width + self.right.padded_cache_width

    def state_bytes(self, dtype_bytes: int) -> int:
        return sum(m.state_bytes(dtype_bytes) for m in (self.left, self.right) if m.stateful)


@dataclass(frozen=True)
class DenseMLPSpec:
    """``W_down(act(W_gate h + b) * (W_up h + b)) + b``, the biases if ``bias``; ``act``
    is silu or the tanh form of gelu (``gelu_tanh``)."""

    ff: int
    act: str = "silu"
    bias: bool = True

    kind = "dense"


@dataclass(frozen=True)
class ExpertsSpec:
    """Mixture of ``experts`` small feed-forwards, ``top`` per token.

    ``expert`` "clamped_glu": ``W_down(g sigmoid(alpha g) (u + 1))`` with ``g = min(W_gate
    h, limit)`` and ``u = clamp(W_up h, -limit, limit)``, a token's weight on its expert's
    input; "glu": ``W_down(silu(W_gate h) * (W_up h))`` and "gelu": ``W_down gelu(W_up h)``
    (erf form), the weight on the output.

    Routing scores are ``sigmoid`` or ``softmax`` of fp32 logits (``router_bias``: with a
    learned number per expert in them), renormalised over the chosen experts if asked.
    ``correction``: a learned number per expert joins the score for the choice alone.  The
    choice is limited to the ``keep`` best of ``groups`` equal groups of neighbours (a group
    counts as its best choice score).  The last ``identity`` router outputs are experts that
    return their input.  ``shared``: a feed-forward that every token passes as well."""

    ff: int
    experts: int
    top: int
    limit: float = 0.0
    alpha: float = 1.702
    score: str = "sigmoid"
    renorm: bool = False
    expert: str = "clamped_glu"
    correction: bool = False
    groups: int = 1
    keep: int = 1
    identity: int = 0
    router_bias: bool = False
    shared: DenseMLPSpec | None = None

    kind = "moe"

    @property
    def outputs(self) -> int:
        """Router outputs."""
        return self.experts + self.identity

    @property
    def gated(self) -> bool:
        """An expert's first product has gate and up halves."""
        return self.expert != "gelu"

    @property
    def ff_pad(self) -> int:  # whole k-tiles of the grouped GEMMs
        return _up(self.ff, 64)


@dataclass(frozen=True)
class LayerSpec:
    mixer: object  # a mixer spec
    mlp: object | None = None  # DenseMLPSpec | ExpertsSpec | None
    weights_of: int | None = None  # share layer j's tensors (own cache / state)
    index: int | None = None  # number in the checkpoint's tensor names (None: its place)
    starts: int | None = None  # number of the loop's pass that starts with this layer


@dataclass(frozen=True)
class DesignSpec:
    """What a layer-list family fixes around its layers, and which checkpoint entries
    its ``config.json`` may hold (the same entry name can mean different mixers)."""

    norm: str  # "tanh": Dynamic Tanh; "rms": RMS with a weight stored around zero;
    #            "rms_scalar": RMS with one number for all coordinates
    pre_norm: bool  # sublayers read the normed residual (else the residual itself)
    embed_norm: bool  # the residual starts at norm(embedding)
    tied: bool  # the embedding table is the output head
    mixers: dict
    mlps: dict
    post_norm: bool = True  # a sublayer's output is normed before it is added
    joined: bool = False  # mixer and feed-forward read the same residual, each normed by
    #                       its own norm, and their outputs are added together
    pass_inputs: bool = False  # before a loop's pass t: + the embedding (t > 0), + step[t]

    def sublayer_norms(self, k: int) -> tuple[str | None, str | None]:
        """(pre, post) norm names of a layer's k-th sublayer (1 mixer, 2 feed-forward)."""
        if not self.post_norm:
            return f"norm{k}", None
        return (f"norm{k}", f"norm{k}b") if self.pre_norm else (None, f"norm{k}")


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


def _grouped(spec: AttentionSpec) -> AttentionSpec:
    if spec.kv_heads < 1 or spec.heads % spec.kv_heads:
        raise ValueError(f"attention: {spec.heads} heads over {spec.kv_heads} k/v heads")
    rot = spec.rotary
    if rot is not None and (rot.dims % 2 or not 0 < rot.dims <= spec.dim):
        raise ValueError(f"attention: rot.dims {rot.dims} of dim {spec.dim}")
    return spec


def _chunked_attention(c: dict) -> AttentionSpec:
    return _grouped(AttentionSpec(
        heads=int(c["heads"]), kv_heads=int(c["kv_heads"]), dim=int(c["dim"]),
        vdim=int(c["vdim"]), scale=float(c["scale"]), rotary=None, sink=None, qk_norm="unit",
        chunk=int((c.get("mask") or {}).get("size") or 0)))


def _biased_attention(c: dict) -> AttentionSpec:
    t, cap = c.get("q_temp"), float(c.get("softcap") or 0.0)
    if cap < 0.0 or (t and not float(t["every"]) > 0.0):
        raise ValueError(f"attention: softcap {cap}, q_temp {t}")
    return _grouped(AttentionSpec(
        heads=int(c["heads"]), kv_heads=int(c["kv_heads"]), dim=int(c["dim"]),
        vdim=int(c["vdim"]), scale=float(c["scale"]), rotary=None, sink="zero", qk_norm=None,
        bias="qkv", softcap=cap, distance_bias=True, gate=True,
        temperature=TemperatureSpec(float(t["coef"]), float(t["every"])) if t else None))


def _paired_latent_attention(c: dict) -> LatentAttentionSpec:
    spec = _latent_attention(c)
    return replace(spec, rotary=replace(spec.rotary, interleaved=True))


def _anchored_attention(c: dict) -> AttentionSpec:
    mask = c.get("mask") or {}
    rot = c.get("rot")
    return _grouped(AttentionSpec(
        heads=int(c["heads"]), kv_heads=int(c["kv_heads"]), dim=int(c["dim"]),
        vdim=int(c["vdim"]), scale=float(c["scale"]),
        rotary=replace(_rotary(rot), interleaved=True) if rot and int(rot["dims"]) else None,
        window=int(mask.get("size") or 0), keep_first=int(mask.get("keep_first") or 0),
        qk_norm=None, bias="qkvo"))


def _lightning(c: dict) -> LightningSpec:
    spec = LightningSpec(heads=int(c["heads"]), dim=int(c["dim"]), vdim=int(c["vdim"]),
                         decay=tuple(float(x) for x in c["decay"]))
    if len(spec.decay) != spec.heads or not all(0.0 <= x <= 1.0 for x in spec.decay):
        raise ValueError(f"lightning: {spec.heads} heads need as many decays in [0, 1]")
    return spec


def _parallel(c: dict) -> ParallelSpec:
    return ParallelSpec(_anchored_attention(c["left"]), _lightning(c["right"]))


def _dense(c: dict) -> DenseMLPSpec:
    return DenseMLPSpec(int(c["ff"]))


def _dense_gelu(c: dict) -> DenseMLPSpec:
    return DenseMLPSpec(int(c["ff"]), act="gelu_tanh", bias=False)


def _checked(spec: ExpertsSpec) -> ExpertsSpec:
    n, g = spec.outputs, spec.groups
    if not 1 <= spec.top <= min(n, 64) or n > 256 or spec.experts < 1 or spec.identity < 0:
        raise ValueError(f"moe: top {spec.top} of {n} experts")
    if g < 1 or n % g or not 1 <= spec.keep <= g or spec.top > spec.keep * (n // g):
        raise ValueError(f"moe: top {spec.top} in {spec.keep} of {g} groups of {n} experts")
    return spec


def _gelu_experts(c: dict) -> ExpertsSpec:
    e, r = c["expert"], c["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    return _checked(ExpertsSpec(
        ff=int(e["ff"]), experts=int(r["experts"]), top=int(r["top"]), score="softmax",
        renorm=True, expert="gelu", correction=True, groups=int(g["count"]), keep=int(g["keep"]),
        identity=int(r.get("identity") or 0)))


def _shared_experts(c: dict) -> ExpertsSpec:
    e, r, s = c["expert"], c["router"], c.get("shared")
    return _checked(ExpertsSpec(
        ff=int(e["ff"]), experts=int(r["experts"]), top=int(r["top"]), score="softmax",
        renorm=True, expert="glu", router_bias=True,
        shared=DenseMLPSpec(int(s["ff"]), bias=False) if s else None))


def _experts(c: dict) -> ExpertsSpec:
    e, r = c["expert"], c["router"]
    return _checked(ExpertsSpec(ff=int(e["ff"]), experts=int(r["experts"]), top=int(r["top"]),
                                limit=float(e["limit"])))


DESIGNS = {
    "sivadra": DesignSpec("tanh", pre_norm=True, embed_norm=False, tied=False,
                          mixers={"latent_attention": _latent_attention, "delta": _delta},
                          mlps={"dense": _dense}),
    "sekazen": DesignSpec("rms", pre_norm=False, embed_norm=True, tied=True,
                          mixers={"attention": _attention}, mlps={"moe": _experts}),
    "bisuzen": DesignSpec("tanh", pre_norm=True, post_norm=False, embed_norm=False, tied=False,
                          mixers={"attention": _chunked_attention, "parallel": _parallel},
                          mlps={"dense": _dense_gelu, "moe": _gelu_experts}),
    "tarunex": DesignSpec("rms_scalar", pre_norm=True, post_norm=False, embed_norm=False,
                          tied=False, joined=True, pass_inputs=True,
                          mixers={"attention": _biased_attention,
                                  "latent_attention": _paired_latent_attention},
                          mlps={"moe": _shared_experts}),
}


def _run_order(n: int, loop: dict | None) -> list[int]:
    """Checkpoint layers in the order they run: ``start`` .. ``stop`` - 1 ``times`` times."""
    if not loop:
        return list(range(n))
    a, b, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    if not 0 <= a <= b <= n or times < 1:
        raise ValueError(f"loop {a} .. {b} x {times} of {n} layers")
    return list(range(a)) + list(range(a, b)) * times + list(range(b, n))


def _passes(n: int, loop: dict | None) -> dict[int, int]:
    """Place in the run order -> number of the pass that starts there."""
    if not loop:
        return {}
    a, b = int(loop["start"]), int(loop["stop"])
    return {a + t * (b - a): t for t in range(int(loop["times"]))} if b > a else {}


def looped(layers: tuple, start: int, stop: int, times: int) -> tuple[LayerSpec, ...]:
    """A preset's layers with a loop unrolled, as :func:`parse_layers` does."""
    out: list[LayerSpec] = []
    loop = dict(start=start, stop=stop, times=times)
    starts = _passes(len(layers), loop)
    for at, i in enumerate(_run_order(len(layers), loop)):
        again = at >= stop and start <= i < stop
        out.append(replace(layers[i], weights_of=i if again else None, index=i,
                           starts=starts.get(at)))
    return tuple(out)


def _tensors_of(mixer):
    """The mixer without which layer it borrows from: passes of a loop differ in that."""
    return mixer if mixer.kv_from is None else replace(mixer, kv_from=-1)


def parse_layers(entries: list[dict], design: DesignSpec,
                 loop: dict | None = None) -> tuple[LayerSpec, ...]:
    """``config.json`` ``layers`` (and ``loop``) -> the layers in the order they run.
    ``weights_of`` chains are resolved to the layer that owns the tensors; a layer's later
    passes use the tensors of its first, with a cache or state of their own."""
    owners: list = []
    for i, e in enumerate(entries):
        if e["type"] not in design.mixers:
            raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
        mlp = e.get("mlp")
        if mlp is not None and mlp.get("kind") not in design.mlps:
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
        owners.append(owner)
    order = _run_order(len(entries), loop)
    first: dict = {}
    for at, i in enumerate(order):
        first.setdefault(i, at)
    starts = _passes(len(entries), loop)
    out: list[LayerSpec] = []
    last: dict = {}  # latest pass of a checkpoint layer so far
    for at, i in enumerate(order):
        e = entries[i]
        mixer = design.mixers[e["type"]](e["mixer"])
        if mixer.kv_from is not None and loop:
            mixer = replace(mixer, kv_from=last.get(mixer.kv_from, -1))
        owner = owners[i] if owners[i] is not None else i
        out.append(LayerSpec(
            mixer, None if e.get("mlp") is None else design.mlps[e["mlp"]["kind"]](e["mlp"]),
            None if first[owner] == at else first[owner], i if loop else None,
            starts.get(at)))
        last[i] = at
    for i, l in enumerate(out):
        if l.weights_of is not None:
            o = out[l.weights_of]
            if (_tensors_of(o.mixer), o.mlp) != (_tensors_of(l.mixer), l.mlp):
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
        out = {"q": (m.heads * m.dim, d), "o": (d, m.heads * m.vdim)}
        if m.kv_from is None:
            out.update({"k": (m.kv_heads * m.dim, d), "v": (m.kv_heads * m.vdim, d)})
        out.update({n + ".b": (w[0],) for n, w in list(out.items()) if n in m.bias})
        if m.distance_bias:
            out.update({"r1": (m.heads,), "r2": (m.heads,)})
        if m.gate:
            out["g"] = (m.heads, d)
        if m.qk_norm == "weight":
            out["q.norm"] = (m.dim,)
            if m.kv_from is None:
                out["k.norm"] = (m.dim,)
        if m.sink == "learned":
            out["sink"] = (m.heads,)
        return out
    if m.kind == "lightning":
        hd, hv = m.heads * m.dim, m.heads * m.vdim
        return {"q": (hd, d), "k": (hd, d), "v": (hv, d), "g": (hv, d), "norm": (hv,),
                "o": (d, hv)}
    if m.kind == "parallel":
        out = {}
        for side, sub in (("left.", m.left), ("right.", m.right)):
            out.update({side + n: s for n, s in _mixer_shapes(sub, d).items()})
            out[side + "out"] = (d,)
        return out
    kd, hv = m.kv_heads * m.dim, m.heads * m.vdim
    return {"q": (kd, d), "q.conv": (kd, m.conv), "k": (kd, d), "k.conv": (kd, m.conv),
            "v": (hv, d), "v.conv": (hv, m.conv), "b": (m.heads, d), "A_log": (m.heads,),
            "norm": (m.vdim,), "a": (m.heads, d), "dt_bias": (m.heads,), "g": (hv, d),
            "o": (d, hv)}


def _mlp_shapes(m, d: int) -> dict[str, tuple]:
    if m.kind == "moe":
        out = {"router": (m.outputs, d)}
        if m.router_bias:
            out["router.b"] = (m.outputs,)
        if m.correction:
            out["correction"] = (m.outputs,)
        for e in range(m.experts):
            if m.gated:
                out[f"e{e}.gate"] = (m.ff, d)
            out.update({f"e{e}.up": (m.ff, d), f"e{e}.down": (d, m.ff)})
        if m.shared is not None:
            out.update({"shared." + n: s for n, s in _mlp_shapes(m.shared, d).items()})
        return out
    out = {"gate": (m.ff, d), "up": (m.ff, d), "down": (d, m.ff)}
    if m.bias:
        out.update({n + ".b": (w[0],) for n, w in list(out.items())})
    return out


def tensor_shapes(layers, d: int, vocab: int,
                  design: DesignSpec = DESIGNS["sivadra"]) -> dict[str, tuple]:
    """Every checkpoint tensor of a layer-list model and its shape."""

    def norm(name):
        if name is None:
            return {}
        if design.norm == "tanh":
            return {name: (d,), name + ".b": (d,), name + ".alpha": ()}
        return {name: () if design.norm == "rms_scalar" else (d,)}

    out = {"embed": (vocab, d)}
    if design.pass_inputs:
        times = sum(l.starts is not None for l in layers)
        if times:
            out["loop.step"] = (times, d)
    if design.embed_norm:
        out.update(norm("embed.norm"))
    for i, l in enumerate(layers):
        if l.weights_of is not None:
            continue
        p = f"l{i if l.index is None else l.index}."
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
