from . import bevovik, fozedra, ligipel, minilorn, mofarax, poresun, qwen2  # noqa: F401  (register Bevovik, Fozedra, Ligipel, Minilorn, Mofarax, Poresun and Qwen2ForCausalLM)
from .decoder import DecoderModel

__all__ = ["DecoderModel", "bevovik", "fozedra", "ligipel", "minilorn", "mofarax", "poresun", "qwen2"]
