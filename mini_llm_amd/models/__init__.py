from . import dizizen, gevulorn, gimozen, goletar, gpt2, ketolix, perezen  # register Dizizen, Gevulorn, Gimozen, Goletar, GPT2LMHeadModel, Ketolix and Perezen
from .base import CacheGroupSpec, LayerCall, Model

__all__ = ["CacheGroupSpec", "LayerCall", "Model", "dizizen", "gevulorn", "gimozen", "goletar", "gpt2", "ketolix", "perezen"]
