from . import dizizen, gimozen, goletar, gpt2, ketolix, perezen  # register Dizizen, Gimozen, Goletar, GPT2LMHeadModel, Ketolix and Perezen
from .base import CacheGroupSpec, LayerCall, Model

__all__ = ["CacheGroupSpec", "LayerCall", "Model", "dizizen", "gimozen", "goletar", "gpt2", "ketolix", "perezen"]
