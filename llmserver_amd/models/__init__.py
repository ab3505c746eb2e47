from . import barotar, gogalix, kerudra, mefurax, qwen3, setodra, zepolix  # registers the architectures
from .decoder import DecoderModel, LayerCall

__all__ = ["DecoderModel", "LayerCall"]
