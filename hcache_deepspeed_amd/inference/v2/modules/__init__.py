"""Inference-v2 compute modules: interfaces, registries, MI355X implementations and the selection heuristics
(reference deepspeed/inference/v2/modules)."""
from .configs import (DSEmbeddingsConfig, DSExpertLayerConfig, DSGatedMLPConfig, DSInputNormConfig, DSLinearConfig,
                      DSMixerConfig, DSMoEConfig, DSNormConfig, DSSelfAttentionConfig, DSUnembedConfig)
from .heuristics import (instantiate_attention, instantiate_embed, instantiate_expert_layer, instantiate_gated_mlp,
                         instantiate_input_norm, instantiate_linear, instantiate_mixer, instantiate_moe,
                         instantiate_output_norm, instantiate_post_norm, instantiate_pre_norm,
                         instantiate_sandwich_norm, instantiate_unembed)
from .interfaces import (DSEmbeddingBase, DSEmbeddingRegistry, DSExpertLayerBase, DSExpertLayerRegistry, DSGatedMLPBase,
                         DSGatedMLPRegistry, DSInputNormBase, DSInputNormRegistry, DSLinearBase, DSLinearRegistry,
                         DSMixerBase, DSMixerRegistry, DSMoEBase, DSMoERegistry, DSOutputNormBase, DSOutputNormRegistry,
                         DSPostNormBase, DSPostNormRegistry, DSPreNormBase, DSPreNormRegistry, DSSandwichNormBase,
                         DSSandwichNormRegistry, DSSelfAttentionBase, DSSelfAttentionRegistry, DSUnembedBase,
                         DSUnembedRegistry)
from .module_registry import ConfigBundle, DSModuleBase, DSModuleRegistryBase
