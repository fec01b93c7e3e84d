"""`ZudusunForSampling`: the user-facing class of the Zudusun architecture; everything it does is the
architecture-free `CausalLMForSampling`."""
from ..causal_lm import CausalLMForSampling
from .spec import ARCHITECTURE


class ZudusunForSampling(CausalLMForSampling):
    architecture = ARCHITECTURE
