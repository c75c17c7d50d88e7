from . import llama, lufazen, fofapel, gesutar, vevapel, mogutar  # noqa: F401  (register LlamaForCausalLM, Lufazen, Fofapel, Gesutar, Vevapel, Mogutar)
from .decoder import Decoder
