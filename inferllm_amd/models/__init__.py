from . import dotorax, febivik, kukupel, llama, rabapel, sabipel, vupolix  # registers the architectures

__all__ = ["dotorax", "febivik", "kukupel", "llama", "rabapel", "sabipel", "vupolix"]
