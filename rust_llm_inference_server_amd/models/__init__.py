"""Models as data (``ModelSpec``) and the architectures that ship with the package."""
from .bekunex import bekunex_spec
from .gipotar import gipotar_spec
from .lagedra import lagedra_spec
from .llama import llama_spec
from .pamolix import pamolix_spec
from .pozelix import pozelix_spec
from .ralitar import ralitar_spec
from .spec import JunctionSpec, LayerSpec, Model, ModelSpec, RunEntry

__all__ = ["JunctionSpec", "LayerSpec", "Model", "ModelSpec", "RunEntry", "bekunex_spec", "gipotar_spec",
           "lagedra_spec", "llama_spec", "pamolix_spec", "pozelix_spec", "ralitar_spec"]
