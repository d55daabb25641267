"""Models: encoders (``bert``), decoders (``llama``, ``hybrid``), configurations, checkpoints, tokenizers."""


def make_decoder(cfg, device="cuda", seed: int = 0, tp=None, weights: dict | None = None, dtype: str = "bf16"):
    """The decoder of a configuration: its checkpoint's weights if it names a folder, else seeded random ones."""
    from .configs import HybridConfig, decoder_dtypes
    if dtype not in decoder_dtypes(cfg):
        raise ValueError(f"{cfg.name}: dtype {dtype!r} is not supported ({', '.join(decoder_dtypes(cfg))})")
    if isinstance(cfg, HybridConfig):
        from .hybrid import HybridDecoder
        return HybridDecoder(cfg, device, seed=seed, tp=tp, weights=weights, dtype=dtype)
    from .llama import LlamaDecoder
    return LlamaDecoder(cfg, device, seed=seed, tp=tp, weights=weights)
