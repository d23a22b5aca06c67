"""Model families served by the in-node engine (Llama-3 dense, Mixtral MoE, and the
layer lists Sivadra, Sekazen, Bisuzen and Tarunex)."""
from .config import REGISTRY, ModelConfig, resolve  # noqa: F401


def build_model(cfg: ModelConfig, device="cpu", dtype=None, seed: int = 0, **kw):
    import torch

    dtype = dtype or torch.bfloat16
    if kw.get("weights") is None:
        kw.pop("weights", None)
    if cfg.arch == "llama":
        from .llama import LlamaModel

        kw.pop("ep_mode", None)
        return LlamaModel(cfg, device=device, dtype=dtype, seed=seed, **kw)
    if cfg.arch == "mixtral":
        from .mixtral import MixtralModel

        return MixtralModel(cfg, device=device, dtype=dtype, seed=seed, **kw)
    if cfg.layers:
        from .hybrid import HybridModel

        if kw.pop("ep_mode", "tp") != "tp":
            raise ValueError(f"{cfg.arch}: layer-list models do not distribute experts")
        return HybridModel(cfg, device=device, dtype=dtype, seed=seed, **kw)
    raise ValueError(f"unsupported arch {cfg.arch}")


def allocate_cache(model, num_blocks: int, block_size: int, device, dtype, n_slots: int = 0):
    """The cache a model steps on: K / V pages, or what each layer of a layer list keeps."""
    from .llama import KVCache

    if hasattr(model, "allocate_cache"):
        return model.allocate_cache(num_blocks, block_size, n_slots)
    return KVCache.allocate(model.cfg, num_blocks, block_size, device, tp_size=model.tp,
                            dtype=dtype)
