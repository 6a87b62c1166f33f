"""runbooks_amd.ops — MI355X (gfx950) compute ops.

GPU tensors run on hand-written CDNA4 HIP kernels (csrc/); CPU tensors run
plain-PyTorch fp32 references (the numerics oracles). A GPU tensor with no
built extension raises — there is no silent eager fallback on the GPU.
"""
from ._backend import ext, has_hip, use_hip  # noqa: F401
from .activations import cross_entropy, geglu, softcap, swiglu  # noqa: F401
from .adamw import FusedAdamW  # noqa: F401
from .attention import (causal_attention, flash_prefill, paged_decode,  # noqa: F401
                        paged_decode_ref, paged_decode_with_operand)
from .kvcache import BLOCK_SIZE, alloc_kv_cache, kv_append, kv_append_ref  # noqa: F401
from .latent import alloc_latent_cache, pad_to  # noqa: F401
from .lightning import alloc_lightning_state  # noqa: F401
from .linear import (Linear, decode_linear_raw, decode_operand,  # noqa: F401
                     decode_ready, fast_linear, linear_f32,
                     linear_f32_parts)
from .norm import (RMSNorm, join_res32, layernorm_res32, norm_res32,  # noqa: F401
                   rmsnorm, rmsnorm_ref, rmsnorm_res32)
from .rope import rope, rope_frequencies, rope_ref, rope_tables  # noqa: F401
from .sampling import sample_tokens  # noqa: F401
from .shared_kv import alloc_shared_kv_cache  # noqa: F401
from .streams import (DynamicTanh, Pending, pack_join, squared_relu,  # noqa: F401
                      streams_norm)
