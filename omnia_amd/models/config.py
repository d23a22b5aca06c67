"""Model architecture configs (public HF shapes, random-init weights in this repo).

The reference (AltairaLabs/Omnia) never runs a model -- its Provider CRD points
at remote vendors (``api/v1alpha1/provider_types.go:273-413``).  These configs
are the in-node engine's model registry; the Provider CRD ``spec.model`` name is
resolved here (``resolve``).
"""
from __future__ import annotations

import dataclasses
import math
from dataclasses import dataclass, field

from .layers import (DESIGNS, AttentionSpec, BandSpec, DeltaSpec, DenseMLPSpec, DesignSpec,
                     ExpertsSpec, LatentAttentionSpec, LayerSpec, LightningSpec, ParallelSpec,
                     RotarySpec, TemperatureSpec, YarnSpec, looped, tensor_shapes)


@dataclass(frozen=True)
class ModelConfig:
    name: str
    arch: str = "llama"  # llama | mixtral | a layer-list family (layers.DESIGNS)
    vocab_size: int = 128256
    hidden_size: int = 4096
    intermediate_size: int = 14336
    num_layers: int = 32
    num_heads: int = 32
    num_kv_heads: int = 8
    head_dim: int = 128
    rope_theta: float = 500000.0
    rope_scaling: dict | None = None
    rms_eps: float = 1e-5
    max_position: int = 8192
    tie_embeddings: bool = False
    # MoE
    num_experts: int = 0
    experts_per_token: int = 0
    # layer-list models (models/hybrid.py): one LayerSpec per layer; the uniform
    # head / intermediate sizes above do not apply to them
    layers: tuple = ()
    embed_scale: float = 1.0  # the residual starts at the embedding times this
    logit_scale: float = 1.0  # the head's output times this
    logit_softcap: float = 0.0  # > 0: logits <- cap tanh(logits / cap)
    # tokenizer special ids (llama-3 layout)
    bos_token_id: int = 128000
    eos_token_ids: tuple = (128001, 128009)

    @property
    def q_size(self) -> int:
        return self.num_heads * self.head_dim

    @property
    def kv_size(self) -> int:
        return self.num_kv_heads * self.head_dim

    @property
    def is_moe(self) -> bool:
        return self.num_experts > 0

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        if self.layers:
            return dtype_bytes * sum(l.mixer.padded_cache_width for l in self.layers)
        return 2 * self.num_layers * self.kv_size * dtype_bytes

    @property
    def stateful(self) -> bool:
        """Some layer carries a recurrent state per sequence (beside or instead of
        cached keys): a cached prefix is usable only with the state at its end."""
        return any(l.mixer.stateful for l in self.layers)

    def state_bytes_per_slot(self, dtype_bytes: int = 2) -> int:
        """Recurrent state of one sequence."""
        return sum(l.mixer.state_bytes(dtype_bytes) for l in self.layers if l.mixer.stateful)

    @property
    def design(self) -> DesignSpec:
        return DESIGNS[self.arch]

    @property
    def key_window(self) -> int:
        """Longest window of any latent-attention layer (0: some layer sees the whole
        past, or no layer gathers keys)."""
        w = [l.mixer.window for l in self.layers if l.mixer.kind == "latent_attention"]
        return 0 if not w or min(w) == 0 else max(w)

    def num_params(self) -> int:
        if self.layers:
            return sum(math.prod(s) for s in tensor_shapes(
                self.layers, self.hidden_size, self.vocab_size, self.design).values())
        d, i, L = self.hidden_size, self.intermediate_size, self.num_layers
        attn = d * (self.q_size + 2 * self.kv_size) + self.q_size * d
        mlp = 3 * d * i * max(1, self.num_experts) + (d * self.num_experts if self.is_moe else 0)
        emb = self.vocab_size * d * (1 if self.tie_embeddings else 2)
        return L * (attn + mlp + 2 * d) + emb + d

    def replace(self, **kw) -> "ModelConfig":
        return dataclasses.replace(self, **kw)


LLAMA3_8B = ModelConfig(name="llama-3-8b")
LLAMA31_8B = ModelConfig(
    name="llama-3.1-8b",
    max_position=131072,
    rope_scaling={"rope_type": "llama3", "factor": 8.0, "low_freq_factor": 1.0,
                  "high_freq_factor": 4.0, "original_max_position_embeddings": 8192},
)
LLAMA3_70B = ModelConfig(name="llama-3-70b", hidden_size=8192, intermediate_size=28672,
                         num_layers=80, num_heads=64, num_kv_heads=8)
MIXTRAL_8X7B = ModelConfig(name="mixtral-8x7b", arch="mixtral", vocab_size=32000,
                           hidden_size=4096, intermediate_size=14336, num_layers=32,
                           num_heads=32, num_kv_heads=8, rope_theta=1e6, max_position=32768,
                           num_experts=8, experts_per_token=2, bos_token_id=1,
                           eos_token_ids=(2,))
# in-node embedding model for the memory tier (K17): a small Llama-shaped encoder
# whose last hidden states are mean-pooled + L2-normalised (1024-d vectors)
EMBED_1B = ModelConfig(name="omnia-embed-1b", vocab_size=128256, hidden_size=1024,
                       intermediate_size=4096, num_layers=16, num_heads=8, num_kv_heads=8,
                       max_position=8192, tie_embeddings=True)
TINY_EMBED = ModelConfig(name="tiny-embed", vocab_size=512, hidden_size=256,
                         intermediate_size=512, num_layers=2, num_heads=2, num_kv_heads=2,
                         max_position=4096, tie_embeddings=True, bos_token_id=256,
                         eos_token_ids=(257,))
# tiny shapes for CPU tests / smoke (same code paths, head_dim fixed at 128)
TINY_LLAMA = ModelConfig(name="tiny-llama", vocab_size=512, hidden_size=256,
                         intermediate_size=512, num_layers=2, num_heads=4, num_kv_heads=2,
                         max_position=4096, bos_token_id=256, eos_token_ids=(257,))
# TP=4/8 rehearsal shape: 8 q heads over 2 kv heads, so at TP 4 and 8 every rank
# holds ONE replicated kv head -- the per-rank layout of Llama-3-70B at TP=8
TINY_LLAMA_H8 = ModelConfig(name="tiny-llama-h8", vocab_size=512, hidden_size=1024,
                            intermediate_size=1024, num_layers=2, num_heads=8, num_kv_heads=2,
                            max_position=4096, bos_token_id=256, eos_token_ids=(257,))
TINY_MIXTRAL = ModelConfig(name="tiny-mixtral", arch="mixtral", vocab_size=512,
                           hidden_size=256, intermediate_size=256, num_layers=2, num_heads=4,
                           num_kv_heads=2, max_position=4096, num_experts=4,
                           experts_per_token=2, bos_token_id=256, eos_token_ids=(257,))
# 8 experts: one per rank of an 8-way expert-parallel group (EP world-8 tests)
TINY_MIXTRAL_E8 = ModelConfig(name="tiny-mixtral-e8", arch="mixtral", vocab_size=512,
                              hidden_size=256, intermediate_size=128, num_layers=2,
                              num_heads=4, num_kv_heads=2, max_position=4096, num_experts=8,
                              experts_per_token=2, bos_token_id=256, eos_token_ids=(257,))



def _alternating(groups: int, delta: DeltaSpec, attn: LatentAttentionSpec, ff: int,
                 deltas: int = 3) -> tuple:
    """``groups`` x (``deltas`` recurrent layers, then one attention layer), each
    with a feed-forward."""
    mlp = DenseMLPSpec(ff)
    return ((LayerSpec(delta, mlp),) * deltas + (LayerSpec(attn, mlp),)) * groups


# Sivadra: tanh-normed layer list of gated-delta and windowed latent-attention mixers
TINY_SIVADRA = ModelConfig(
    name="tiny-sivadra", arch="sivadra", vocab_size=512, hidden_size=192, num_layers=4,
    rms_eps=1e-5, max_position=4096, bos_token_id=256, eos_token_ids=(257,),
    layers=(
        LayerSpec(DeltaSpec(heads=6, kv_heads=3, dim=24, vdim=40, conv=3), DenseMLPSpec(320)),
        LayerSpec(LatentAttentionSpec(
            heads=5, dim=40, rot_dim=12, vdim=48, q_rank=56, kv_rank=72, scale=0.14, window=48,
            rotary=RotarySpec(12, 20000.0, YarnSpec(4.0, 256, 24.0, 1.5)))),
        LayerSpec(DeltaSpec(heads=6, kv_heads=3, dim=24, vdim=40, conv=3), DenseMLPSpec(320), 0),
        LayerSpec(LatentAttentionSpec(
            heads=3, dim=32, rot_dim=16, vdim=24, q_rank=40, kv_rank=48, scale=0.15, window=0,
            rotary=RotarySpec(16, 10000.0)), DenseMLPSpec(256)),
    ))
# serving-sized shapes (random-init): the width, depth and feed-forward of the Llama
# config of the same size, attention / recurrent heads of 128
SIVADRA_1B = ModelConfig(
    name="sivadra-1b", arch="sivadra", vocab_size=32768, hidden_size=2048, num_layers=16,
    intermediate_size=8192, max_position=131072, bos_token_id=256, eos_token_ids=(257,),
    layers=_alternating(
        4, DeltaSpec(heads=16, kv_heads=8, dim=128, vdim=128, conv=4),
        LatentAttentionSpec(heads=16, dim=128, rot_dim=64, vdim=128, q_rank=1024, kv_rank=512,
                            scale=192 ** -0.5, window=1024,
                            rotary=RotarySpec(64, 50000.0, YarnSpec(8.0, 4096))), 8192))
SIVADRA_8B = ModelConfig(
    name="sivadra-8b", arch="sivadra", vocab_size=128256, hidden_size=4096, num_layers=32,
    intermediate_size=14336, max_position=131072, bos_token_id=256, eos_token_ids=(257,),
    layers=_alternating(
        8, DeltaSpec(heads=32, kv_heads=16, dim=128, vdim=128, conv=4),
        LatentAttentionSpec(heads=32, dim=128, rot_dim=64, vdim=128, q_rank=1536, kv_rank=512,
                            scale=192 ** -0.5, window=2048,
                            rotary=RotarySpec(64, 50000.0, YarnSpec(8.0, 4096))), 14336))
# the Llama of sivadra-1b's width, depth and feed-forward (design comparison)
LLAMA_1B = ModelConfig(name="llama-1b-shape", vocab_size=32768, hidden_size=2048,
                       intermediate_size=8192, num_layers=16, num_heads=16, num_kv_heads=8,
                       bos_token_id=256, eos_token_ids=(257,))



def _paired(pairs: int, attn: AttentionSpec, window: int, mlp: ExpertsSpec) -> tuple:
    """``pairs`` x (an attention layer with keys of its own, then one with ``window``
    that attends to the same keys), each with a mixture of experts."""
    out: list = []
    for _ in range(pairs):
        out.append(LayerSpec(attn, mlp))
        out.append(LayerSpec(dataclasses.replace(attn, window=window, kv_from=len(out) - 1),
                             mlp))
    return tuple(out)


# Sekazen: post-normed layer list of windowed grouped-query attention with sinks, key /
# value borrowing and sparse experts
TINY_SEKAZEN = ModelConfig(
    name="tiny-sekazen", arch="sekazen", vocab_size=512, hidden_size=160, num_layers=4,
    intermediate_size=96, max_position=4096, logit_softcap=20.0, bos_token_id=256,
    eos_token_ids=(257,), tie_embeddings=True,
    layers=_paired(
        2, AttentionSpec(heads=6, kv_heads=2, dim=40, vdim=48, scale=0.15, window=56,
                         rotary=RotarySpec(16, 10000.0, bands=BandSpec(8.0, 1.0, 4.0, 256))),
        24, ExpertsSpec(ff=96, experts=6, top=2, limit=4.0)))
# serving-sized shapes (random-init): width, depth, heads and experts of the Mixtral config
# of the same size
SEKAZEN_3B = ModelConfig(
    name="sekazen-3b", arch="sekazen", vocab_size=32768, hidden_size=2048, num_layers=16,
    intermediate_size=4096, max_position=131072, logit_softcap=30.0, bos_token_id=256,
    eos_token_ids=(257,), tie_embeddings=True,
    layers=_paired(
        8, AttentionSpec(heads=16, kv_heads=8, dim=128, vdim=128, scale=128 ** -0.5, window=4096,
                         rotary=RotarySpec(64, 500000.0, bands=BandSpec(8.0, 1.0, 4.0, 8192))),
        1024, ExpertsSpec(ff=4096, experts=8, top=2, limit=7.0)))
SEKAZEN_8X7B = ModelConfig(
    name="sekazen-8x7b", arch="sekazen", vocab_size=32000, hidden_size=4096, num_layers=32,
    intermediate_size=14336, max_position=131072, logit_softcap=30.0, bos_token_id=1,
    eos_token_ids=(2,), tie_embeddings=True,
    layers=_paired(
        16, AttentionSpec(heads=32, kv_heads=8, dim=128, vdim=128, scale=128 ** -0.5,
                          window=4096,
                          rotary=RotarySpec(64, 1e6, bands=BandSpec(8.0, 1.0, 4.0, 8192))),
        1024, ExpertsSpec(ff=14336, experts=8, top=2, limit=7.0)))
# the Mixtral of sekazen-3b's width, depth and experts (design comparison)
MIXTRAL_3B = ModelConfig(name="mixtral-3b-shape", arch="mixtral", vocab_size=32768,
                         hidden_size=2048, intermediate_size=4096, num_layers=16, num_heads=16,
                         num_kv_heads=8, num_experts=8, experts_per_token=2, bos_token_id=256,
                         eos_token_ids=(257,))



def _parallel(heads: int, kv_heads: int, dim: int, window: int, lin_heads: int, base: float,
              keep: int = 4) -> ParallelSpec:
    """Windowed attention with kept first tokens beside linear attention whose heads forget
    over 2 to some thousand tokens."""
    return ParallelSpec(
        AttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=dim ** -0.5,
                      rotary=RotarySpec(dim // 2, base, interleaved=True), window=window,
                      keep_first=keep, qk_norm=None, bias="qkvo"),
        LightningSpec(heads=lin_heads, dim=dim, vdim=dim, decay=tuple(
            1.0 - 2.0 ** (-1.0 - 11.0 * i / max(lin_heads - 1, 1))
            for i in range(lin_heads))))


def _chunked(heads: int, kv_heads: int, dim: int, chunk: int) -> AttentionSpec:
    return AttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=dim ** 0.5,
                         rotary=None, sink=None, qk_norm="unit", chunk=chunk)


# Bisuzen: tanh pre-normed layer list of attention and linear attention side by side, chunked
# attention without positions, gelu feed-forwards and grouped experts, looped layers
TINY_BISUZEN = ModelConfig(
    name="tiny-bisuzen", arch="bisuzen", vocab_size=512, hidden_size=160, num_layers=6,
    intermediate_size=208, max_position=4096, logit_scale=0.5, bos_token_id=256,
    eos_token_ids=(257,),
    layers=looped((
        LayerSpec(_parallel(6, 2, 40, 56, 3, 10000.0), DenseMLPSpec(208, "gelu_tanh", False)),
        LayerSpec(_parallel(4, 1, 48, 32, 2, 10000.0), ExpertsSpec(
            ff=72, experts=6, top=2, score="softmax", renorm=True, expert="gelu",
            correction=True, groups=4, keep=2, identity=2)),
        LayerSpec(_chunked(5, 1, 32, 48), DenseMLPSpec(144, "gelu_tanh", False)),
        LayerSpec(_chunked(4, 2, 64, 80))), 1, 3, 2))
# serving-sized shapes (random-init): width, depth and heads of the model named beside each
BISUZEN_3B = ModelConfig(  # sekazen-3b
    name="bisuzen-3b", arch="bisuzen", vocab_size=32768, hidden_size=2048, num_layers=16,
    intermediate_size=4096, max_position=131072, logit_scale=0.25, bos_token_id=256,
    eos_token_ids=(257,),
    layers=(LayerSpec(_parallel(16, 8, 128, 1024, 16, 500000.0), ExpertsSpec(
                ff=6144, experts=8, top=2, score="softmax", renorm=True, expert="gelu",
                correction=True, groups=2, keep=1, identity=2)),
            LayerSpec(_chunked(16, 8, 128, 4096), ExpertsSpec(
                ff=6144, experts=8, top=2, score="softmax", renorm=True, expert="gelu",
                correction=True, groups=2, keep=1, identity=2))) * 8)
BISUZEN_8B = ModelConfig(  # sivadra-8b
    name="bisuzen-8b", arch="bisuzen", vocab_size=128256, hidden_size=4096, num_layers=32,
    intermediate_size=14336, max_position=131072, logit_scale=0.25, bos_token_id=256,
    eos_token_ids=(257,),
    layers=(LayerSpec(_parallel(32, 8, 128, 2048, 32, 500000.0),
                      DenseMLPSpec(14336, "gelu_tanh", False)),) * 24
    + (LayerSpec(_chunked(32, 8, 128, 4096), DenseMLPSpec(14336, "gelu_tanh", False)),) * 8)



def _biased(heads: int, kv_heads: int, dim: int, every: float) -> AttentionSpec:
    """Attention whose positions are a query temperature and a distance bias."""
    return AttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=dim ** -0.5,
                         rotary=None, sink="zero", qk_norm=None, bias="qkv", softcap=30.0,
                         distance_bias=True, gate=True,
                         temperature=TemperatureSpec(0.1, every))


def _latent(heads: int, q_rank: int, base: float) -> LatentAttentionSpec:
    return LatentAttentionSpec(heads=heads, dim=128, rot_dim=64, vdim=128, q_rank=q_rank,
                               kv_rank=512, scale=192 ** -0.5,
                               rotary=RotarySpec(64, base, interleaved=True))


def _shared(ff: int, experts: int, top: int, shared: int) -> ExpertsSpec:
    return ExpertsSpec(ff=ff, experts=experts, top=top, score="softmax", renorm=True,
                       expert="glu", router_bias=True, shared=DenseMLPSpec(shared, bias=False))


# Tarunex: layer list whose mixer and feed-forward run side by side on one residual: capped
# attention with a distance bias, latent attention, experts beside a shared one, and a loop
# that every pass enters with the embedding and a vector of its own
TINY_TARUNEX = ModelConfig(
    name="tiny-tarunex", arch="tarunex", vocab_size=512, hidden_size=160, num_layers=6,
    intermediate_size=72, max_position=4096, rms_eps=1e-5, embed_scale=8.0, logit_scale=0.5,
    logit_softcap=25.0, bos_token_id=256, eos_token_ids=(257,),
    layers=looped((
        LayerSpec(_biased(6, 2, 40, 96), _shared(72, 6, 2, 88)),
        LayerSpec(LatentAttentionSpec(
            heads=5, dim=40, rot_dim=12, vdim=48, q_rank=56, kv_rank=72, scale=0.14,
            rotary=RotarySpec(12, 20000.0, interleaved=True)), _shared(56, 5, 1, 40)),
        LayerSpec(_biased(4, 1, 32, 64), _shared(72, 6, 3, 88)),
        LayerSpec(_biased(4, 4, 64, 128))), 1, 3, 2))
# serving-sized shapes (random-init): width, heads, layers run and active feed-forward of the
# model named beside each
TARUNEX_3B = ModelConfig(  # sekazen-3b
    name="tarunex-3b", arch="tarunex", vocab_size=32768, hidden_size=2048, num_layers=16,
    intermediate_size=3072, max_position=131072, embed_scale=8.0, logit_scale=0.5,
    logit_softcap=40.0, bos_token_id=256, eos_token_ids=(257,),
    layers=looped(((LayerSpec(_biased(16, 8, 128, 8192), _shared(3072, 8, 2, 2048)),) * 3
                   + (LayerSpec(_latent(16, 1024, 500000.0), _shared(3072, 8, 2, 2048)),)) * 3,
                  4, 8, 2))
TARUNEX_8B = ModelConfig(  # sivadra-8b
    name="tarunex-8b", arch="tarunex", vocab_size=128256, hidden_size=4096, num_layers=32,
    intermediate_size=7168, max_position=131072, embed_scale=8.0, logit_scale=0.5,
    logit_softcap=40.0, bos_token_id=256, eos_token_ids=(257,),
    layers=looped(((LayerSpec(_biased(32, 8, 128, 8192), _shared(7168, 3, 1, 7168)),)
                   + (LayerSpec(_latent(32, 1536, 500000.0), _shared(7168, 3, 1, 7168)),)) * 10,
                  4, 16, 2))

REGISTRY: dict[str, ModelConfig] = {
    c.name: c for c in [LLAMA3_8B, LLAMA31_8B, LLAMA3_70B, MIXTRAL_8X7B, TINY_LLAMA, TINY_MIXTRAL,
                   TINY_MIXTRAL_E8, EMBED_1B, TINY_EMBED, TINY_LLAMA_H8, TINY_SIVADRA,
                   SIVADRA_1B, SIVADRA_8B, LLAMA_1B, TINY_SEKAZEN, SEKAZEN_3B, SEKAZEN_8X7B,
                   MIXTRAL_3B, TINY_BISUZEN, BISUZEN_3B, BISUZEN_8B, TINY_TARUNEX,
                   TARUNEX_3B, TARUNEX_8B]
}
ALIASES = {
    "meta-llama/Meta-Llama-3-8B": "llama-3-8b",
    "meta-llama/Meta-Llama-3-8B-Instruct": "llama-3-8b",
    "llama3-8b": "llama-3-8b",
    "meta-llama/Llama-3.1-8B-Instruct": "llama-3.1-8b",
    "meta-llama/Meta-Llama-3-70B-Instruct": "llama-3-70b",
    "llama3-70b": "llama-3-70b",
    "mistralai/Mixtral-8x7B-Instruct-v0.1": "mixtral-8x7b",
    "mixtral": "mixtral-8x7b",
}


def resolve(name: str, **overrides) -> ModelConfig:
    key = ALIASES.get(name, name)
    if key not in REGISTRY:
        raise KeyError(f"unknown model {name!r}; known: {sorted(REGISTRY)}")
    cfg = REGISTRY[key]
    return cfg.replace(**overrides) if overrides else cfg
