"""`models.rorovik`: a decoder-only language model whose sublayers are normed before and after on an fp32 residual stream.  Mixers:
*attention* - grouped heads, biased projections, queries and keys normed over all heads at once, a query multiplier that grows with the
logarithm of the position, a linear distance bias per head instead of rotary positions, a sliding window, a learned sink in the softmax,
values mixed with those of the first such layer, one sigmoid gate per head; *latent_attention* - queries through a latent of their own, one cached
row per token (a normed latent and a key part with scaled rotary positions shared by the heads), a learned sink.  Feed-forwards are dense
biased relu-gated layers or mixtures of clamped gated experts, some of which hand their input on; every layer ends with a gated slice of a
second embedding table.  Same module interface as the other model packages."""
from .config import LayerConfig, ModelConfig
from .language import LanguageModel
from .rorovik import Model

__all__ = ["Model", "ModelConfig", "LayerConfig", "LanguageModel"]

# the operator sources (csrc/<name>.hip) the model's step function needs: what a trace replay of a fresh checkout compiles
HIP_SOURCES = ('gemm_bf16', 'gemm256_bf16', 'linear_any', 'stream_f32', 'moe', 'moe_grouped', 'latent_attn', 'latent_attn_mfma', 'grouped_attn')
