"""`GubulornForSampling`: the user-facing class of the Gubulorn architecture; everything it does is the
architecture-free `CausalLMForSampling`."""
from ..causal_lm import CausalLMForSampling
from .spec import ARCHITECTURE


class GubulornForSampling(CausalLMForSampling):
    architecture = ARCHITECTURE
