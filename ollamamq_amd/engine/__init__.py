from .kvcache import HybridCache, PagedKVCache, cache_for_model
from .engine import LlamaEngine, Sequence, GenParams

__all__ = ["HybridCache", "PagedKVCache", "cache_for_model", "LlamaEngine",
           "Sequence", "GenParams"]
