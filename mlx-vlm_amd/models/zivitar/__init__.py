"""`models.zivitar`: a decoder-only language model on hyper-connected residual streams (every sublayer reads a weighted sum of the
streams and is written back through a mix of them).  Mixers: *lightning* - linear attention with a fixed decay per head, silu on
q, k and v, one norm over all heads, sigmoid output gate; *attention* - differential attention (two softmax maps per head over
the same values, their difference normed per head) on short-convolved q / k / v with partial rotate-half positions (optionally
with scaled frequencies) inside a sliding window that keeps the first tokens in view.  Feed-forwards are dense clamped gated
units; logits are scaled and capped.  Layers may use another layer's tensors with caches and states of their own.  Same module
interface as the other model packages."""
from .config import LayerConfig, ModelConfig
from .language import LanguageModel
from .zivitar import Model

__all__ = ["Model", "ModelConfig", "LayerConfig", "LanguageModel"]

# the operator sources (csrc/<name>.hip) the model's step function needs: what a trace replay of a fresh checkout compiles
HIP_SOURCES = ('gemm_bf16', 'gemm256_bf16', 'linear_any', 'stream_f32', 'hyper_stream', 'moe', 'short_conv', 'diff_attn', 'linear_recurrence',
               'chunk_recurrence')
