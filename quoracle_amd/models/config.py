"""Model registry: architecture configs (Llama-family, MoE, hybrid) for the
local pool.

The reference delegates model choice to remote providers (reference:
lib/quoracle/models/model_query.ex); here each pool entry names a locally
hosted architecture.  A model key is "<preset>#<instance>" — instances share
the architecture but get different random-init seeds, giving the consensus
pool genuinely decorrelated voters.  A key may also be "<folder>" or
"<folder>#<instance>": a checkpoint folder with config.json and
model.safetensors, whose "architecture" names the config and model class.
"""

from __future__ import annotations

import functools
import json
import os
from dataclasses import dataclass
from typing import Dict, Union

from .hybrid_config import (HybridConfig, KoridraConfig, KotutarConfig,
                            LoopSpec, koridra_preset, kotutar_preset)


@dataclass(frozen=True)
class ModelConfig:
    name: str
    vocab_size: int
    n_layers: int
    hidden: int
    n_heads: int
    n_kv_heads: int
    head_dim: int
    intermediate: int
    rope_theta: float = 500000.0
    rmsnorm_eps: float = 1e-5
    max_context: int = 8192
    max_output: int = 4096
    tie_embeddings: bool = False
    # MoE (0 experts = dense)
    n_experts: int = 0
    top_k_experts: int = 2

    architecture = "Llama"
    native_module = "_quoracle_ops"
    is_hybrid = False
    needs_state = False         # no recurrent state beside the KV pages

    @property
    def q_dim(self) -> int:
        return self.n_heads * self.head_dim

    @property
    def kv_dim(self) -> int:
        return self.n_kv_heads * self.head_dim

    @property
    def qkv_dim(self) -> int:
        return self.q_dim + 2 * self.kv_dim

    @property
    def is_moe(self) -> bool:
        return self.n_experts > 0

    def kv_bytes_per_token(self, element: int = 2) -> int:
        """Paged-KV footprint of one token across all layers."""
        return 2 * element * self.n_layers * self.kv_dim

    def param_count(self) -> int:
        embed = self.vocab_size * self.hidden
        lm_head = 0 if self.tie_embeddings else self.vocab_size * self.hidden
        per_layer = (self.hidden * self.qkv_dim + self.q_dim * self.hidden
                     + 2 * self.hidden)
        if self.is_moe:
            per_layer += self.n_experts * 3 * self.hidden * self.intermediate
            per_layer += self.hidden * self.n_experts  # router
        else:
            per_layer += 3 * self.hidden * self.intermediate
        return embed + lm_head + self.n_layers * per_layer + self.hidden


AnyConfig = Union[ModelConfig, HybridConfig]

PRESETS: Dict[str, AnyConfig] = {
    # CPU-testable toy model (head_dim multiple of 8, <=128 for the kernels)
    "tiny": ModelConfig("tiny", vocab_size=512, n_layers=2, hidden=64,
                        n_heads=4, n_kv_heads=2, head_dim=16,
                        intermediate=128, rope_theta=10000.0,
                        max_context=32768, max_output=1024,
                        tie_embeddings=True),
    # CPU-testable MoE toy (engine-level Mixtral-path tests)
    "tiny-moe": ModelConfig("tiny-moe", vocab_size=512, n_layers=2, hidden=64,
                            n_heads=4, n_kv_heads=2, head_dim=16,
                            intermediate=128, rope_theta=10000.0,
                            max_context=32768, max_output=1024,
                            tie_embeddings=True, n_experts=4,
                            top_k_experts=2),
    # GPT-2-small scale, llama-style blocks
    "gpt2s": ModelConfig("gpt2s", vocab_size=50304, n_layers=12, hidden=768,
                         n_heads=12, n_kv_heads=12, head_dim=64,
                         intermediate=3072, rope_theta=10000.0,
                         max_context=32768, max_output=2048,
                         tie_embeddings=True),
    # Llama-3-8B architecture
    "llama3-8b": ModelConfig("llama3-8b", vocab_size=128256, n_layers=32,
                             hidden=4096, n_heads=32, n_kv_heads=8,
                             head_dim=128, intermediate=14336,
                             rope_theta=500000.0, max_context=32768,
                             max_output=4096),
    # Llama-3-70B (TP=4)
    "llama3-70b": ModelConfig("llama3-70b", vocab_size=128256, n_layers=80,
                              hidden=8192, n_heads=64, n_kv_heads=8,
                              head_dim=128, intermediate=28672,
                              rope_theta=500000.0, max_context=32768,
                              max_output=4096),
    # Mixtral-8x7B MoE (TP=4)
    "mixtral-8x7b": ModelConfig("mixtral-8x7b", vocab_size=32000,
                                n_layers=32, hidden=4096, n_heads=32,
                                n_kv_heads=8, head_dim=128,
                                intermediate=14336, rope_theta=1000000.0,
                                max_context=32768, max_output=4096,
                                n_experts=8, top_k_experts=2),
    # small bidirectional-ish embedder for the consensus cosine vote
    "embed-small": ModelConfig("embed-small", vocab_size=50304, n_layers=2,
                               hidden=256, n_heads=4, n_kv_heads=4,
                               head_dim=64, intermediate=512,
                               rope_theta=10000.0, max_context=4096,
                               max_output=1, tie_embeddings=True),
    # CPU-testable Koridra toy
    "koridra-tiny": koridra_preset(
        "koridra-tiny", vocab=512, hidden=64, n_layers=4, ff=96, heads=4,
        kv_heads=2, dim=16, chunk=48, lin_heads=2, lin_dim=16, lin_vdim=24,
        max_context=4096, every=2, max_output=1024, base=10000.0, rank=4),
    # Koridra with the layer sizes of a 1B-class and of an 8B-class model
    "koridra-1b": koridra_preset(
        "koridra-1b", vocab=128256, hidden=2048, n_layers=16, ff=8192,
        heads=16, kv_heads=4, dim=128, chunk=4096, lin_heads=16, lin_dim=128,
        lin_vdim=128, max_context=32768),
    "koridra-8b": koridra_preset(
        "koridra-8b", vocab=128256, hidden=4096, n_layers=32, ff=14336,
        heads=32, kv_heads=8, dim=128, chunk=8192, lin_heads=32, lin_dim=128,
        lin_vdim=128, max_context=32768),
    # CPU-testable Kotutar toy
    "kotutar-tiny": kotutar_preset(
        "kotutar-tiny", vocab=512, hidden=64, n_layers=4, ff=96, heads=3,
        dim=16, rot_dim=8, vdim=24, q_rank=40, kv_rank=32, experts=5, top=2,
        expert_ff=48, shared_ff=56, loop=LoopSpec(1, 3, 2),
        max_context=4096, max_output=1024, base=10000.0),
    # Kotutar with the layer sizes of a 1B-class and of an 8B-class model
    "kotutar-1b": kotutar_preset(
        "kotutar-1b", vocab=128256, hidden=2048, n_layers=16, ff=8192,
        heads=16, dim=128, rot_dim=64, vdim=128, q_rank=768, kv_rank=512,
        experts=16, top=2, expert_ff=2048, shared_ff=2048,
        loop=LoopSpec(4, 12, 2)),
    "kotutar-8b": kotutar_preset(
        "kotutar-8b", vocab=128256, hidden=4096, n_layers=32, ff=14336,
        heads=32, dim=128, rot_dim=64, vdim=128, q_rank=1536, kv_rank=512,
        experts=16, top=2, expert_ff=4096, shared_ff=4096,
        loop=LoopSpec(8, 24, 2)),
}

# config.json "architecture" -> reader of the rest of the file
ARCHITECTURES = {"Koridra": KoridraConfig.from_dict,
                 "Kotutar": KotutarConfig.from_dict}


@functools.lru_cache(maxsize=64)
def load_config(folder: str) -> AnyConfig:
    """The config of a checkpoint folder, by its config.json."""
    with open(os.path.join(folder, "config.json")) as f:
        raw = json.load(f)
    arch = raw.get("architecture")
    if arch not in ARCHITECTURES:
        raise KeyError(f"{folder}: unknown architecture {arch!r} "
                       f"(known: {sorted(ARCHITECTURES)})")
    name = os.path.basename(os.path.abspath(folder))
    return ARCHITECTURES[arch](raw, name=name, path=folder)


def get_config(key: str) -> AnyConfig:
    """Resolve "<preset>#<instance>", "<preset>" or a checkpoint folder to
    its architecture."""
    preset = key.split("#", 1)[0]
    if preset in PRESETS:
        return PRESETS[preset]
    if os.path.isfile(os.path.join(preset, "config.json")):
        return load_config(preset)
    raise KeyError(f"unknown model preset {preset!r} "
                   f"(known: {sorted(PRESETS)}, or a checkpoint folder)")


def instance_seed(key: str) -> int:
    """Deterministic per-instance weight seed from the model key."""
    import zlib
    return zlib.crc32(key.encode()) & 0x7FFFFFFF
