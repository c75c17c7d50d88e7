from . import (llama, lufazen, fofapel, gesutar, vevapel, mogutar, nililix)  # noqa: F401  (register LlamaForCausalLM, Lufazen, Fofapel, Gesutar, Vevapel, Mogutar, Nililix)
from .decoder import Decoder
