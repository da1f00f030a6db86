from .llama import LlamaForCausalLM
from .mixtral import MixtralForCausalLM
from .mutusun import MutusunForCausalLM
from .radenex import RadenexForCausalLM
from .registry import build_model
from .sumosun import SumosunForCausalLM
from .tefezen import TefezenForCausalLM
