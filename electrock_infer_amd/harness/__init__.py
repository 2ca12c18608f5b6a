"""The engine: decoder-only models, a paged cache and recurrent-state slots, a prefill-first batch planner with
preemption, a prefix-reusing pool of cache blocks and a sampler -- this build's own counterpart of the reference's engine
(electrock_infer/engine/*, models/mixtral.py, layers/sampler.py), kept small.  registry.py lists the models: a
Mixtral-shaped one, Feguvik and Nunivik.

The Mixtral model exists to run the MoE path inside a whole generation loop (the end-to-end configuration of the
benchmark) and its attention is not part of the hot path: it is torch's scaled_dot_product_attention over a gathered
paged cache, the dense projections are torch matmuls; only the norms and the MoE block go through this package's own
kernels.
"""
from .config import EngineConfig, ModelConfig, SamplingParams  # noqa: F401
from .engine import LLMEngine  # noqa: F401
from .feguvik import FeguvikConfig, FeguvikForCausalLM  # noqa: F401
from .nunivik import NunivikConfig, NunivikForCausalLM  # noqa: F401

LLM = LLMEngine
