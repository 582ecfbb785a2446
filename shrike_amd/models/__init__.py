from . import fozedra, ligipel, minilorn, mofarax, poresun, qwen2  # noqa: F401  (register Fozedra, Ligipel, Minilorn, Mofarax, Poresun and Qwen2ForCausalLM)
from .decoder import DecoderModel

__all__ = ["DecoderModel", "fozedra", "ligipel", "minilorn", "mofarax", "poresun", "qwen2"]
