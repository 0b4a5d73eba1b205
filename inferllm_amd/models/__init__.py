from . import dotorax, febivik, kukupel, llama, rabapel, sabipel  # registers Dotorax, Febivik, Kukupel, LlamaForCausalLM, Rabapel and Sabipel

__all__ = ["dotorax", "febivik", "kukupel", "llama", "rabapel", "sabipel"]
