from .llama import LlamaConfig, LlamaForCausalLM, LlamaModel, get_config, CONFIGS
from .mixtral import (MixtralConfig, MixtralForCausalLM, MixtralModel,
                      get_moe_config, MOE_CONFIGS)
from .gpt_neox import (GPTNeoXConfig, GPTNeoXForCausalLM, get_neox_config,
                       NEOX_CONFIGS)
from .voletar import (VoletarConfig, VoletarForCausalLM, VOLETAR_CONFIGS,
                      get_voletar_config)
from .nesilorn import (NesilornConfig, NesilornForCausalLM, NESILORN_CONFIGS,
                       get_nesilorn_config)
from .sutuvik import (SutuvikConfig, SutuvikForCausalLM, SUTUVIK_CONFIGS,
                      get_sutuvik_config)
from .pokepel import (PokepelConfig, PokepelForCausalLM, POKEPEL_CONFIGS,
                      get_pokepel_config)
from .registry import (ModelEntry, build_model, load_pretrained,
                       register_model, registered_models)
