"""Configuration of the harness.  The reference reads the model's shape from a Hugging Face config on disk
(electrock_infer/config.py:21-24) and its engine limits from keyword arguments (config.py:8-19).  Here a model's shape
is a plain dataclass (``ModelConfig`` is Mixtral's, with 8x7B's values as defaults; others stand beside their models) that
is either made by the caller, with weights drawn at random, or read from a model directory (registry.py)."""
from dataclasses import dataclass, field
from typing import Any, Optional

import torch


@dataclass
class ModelConfig:
    """Shape of a Mixtral-style decoder (defaults: Mixtral-8x7B, utils/mixtral_info.txt)."""
    vocab_size: int = 32000
    hidden_size: int = 4096
    intermediate_size: int = 14336
    num_hidden_layers: int = 32
    num_attention_heads: int = 32
    num_key_value_heads: int = 8
    num_local_experts: int = 8
    num_experts_per_tok: int = 2
    rms_norm_eps: float = 1e-5
    rope_theta: float = 1e6
    max_position_embeddings: int = 32768
    torch_dtype: torch.dtype = torch.bfloat16

    @property
    def head_dim(self) -> int:
        return self.hidden_size // self.num_attention_heads

    @classmethod
    def from_checkpoint(cls, config: dict, shapes: dict, dtype: torch.dtype) -> "ModelConfig":
        """From the config.json of a Mixtral checkpoint; ``shapes`` (tensor name -> shape) is not needed."""
        if dtype != torch.bfloat16:
            raise ValueError("the MoE kernels compute in bfloat16")
        names = ("vocab_size", "hidden_size", "intermediate_size", "num_hidden_layers", "num_attention_heads",
                 "num_key_value_heads", "num_local_experts", "num_experts_per_tok", "rms_norm_eps", "rope_theta",
                 "max_position_embeddings")
        return cls(**{n: config[n] for n in names if n in config}, torch_dtype=dtype)


@dataclass
class SamplingParams:
    """Per-request sampling controls (electrock_infer/sampling_params.py:4-8)."""
    temperature: float = 1.0
    max_tokens: int = 64
    ignore_eos: bool = False
    max_total_tokens: int = -1


@dataclass
class EngineConfig:
    """Engine limits, with the reference's names and defaults (config.py:8-19) where they apply to one GPU."""
    model: Any = field(default_factory=ModelConfig)      # ModelConfig, FeguvikConfig, ...
    model_dir: Optional[str] = None     # load the weights from here (None: drawn at random)
    max_num_batched_tokens: int = 32768
    max_num_seqs: int = 300
    max_model_len: int = 4096
    gpu_memory_utilization: float = 0.90
    eos: int = -1
    kvcache_block_size: int = 32
    num_kvcache_blocks: int = -1        # -1: sized from the free device memory (model_runner.py:92-104)
    seed: int = 0                       # of the random weights
    device: str = "cuda:0"
    fused_moe_tail: bool = True         # post-attention norm + gate + router + experts in one library call
    prefill_portion: int = 0            # compute prompts in portions of at most so many tokens (0: whole)
    reuse_prefix: bool = True           # share cache blocks of equal prefixes (off for models with a recurrent state)
    decode_graphs: bool = True          # record decode steps as HIP graphs, for models that take ragged batches
    num_state_slots: int = 0            # recurrent-state slots; set to max_num_seqs for models that have such a state

    def __post_init__(self):
        self.max_model_len = min(self.max_model_len, self.model.max_position_embeddings)
        if getattr(self.model, "has_recurrent_state", False):
            self.reuse_prefix = False
            self.num_state_slots = self.num_state_slots or self.max_num_seqs
        if self.prefill_portion > 0:
            self.reuse_prefix = False
