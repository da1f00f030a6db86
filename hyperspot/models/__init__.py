from .llama import LlamaForCausalLM
from .mixtral import MixtralForCausalLM
from .registry import build_model
from .sumosun import SumosunForCausalLM
from .tefezen import TefezenForCausalLM
