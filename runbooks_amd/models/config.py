"""Model configurations for the families the reference platform serves.

The reference orchestrates external HuggingFace images for these models
(reference examples/: facebook-opt-125m, llama2-7b, llama2-70b,
falcon-7b-instruct, falcon-40b — SURVEY.md §2b). Here they are first-class
configs of our own runtime.
"""
from __future__ import annotations

from dataclasses import dataclass


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Latent attention: keys and values are linear images of one cached
    latent per token (plus one rotated key part all heads share)."""
    heads: int
    dim: int                        # unrotated query/key size per head
    rot_dim: int                    # rotated query/key size per head
    vdim: int                       # value size per head
    kv_rank: int                    # latent size
    scale: float                    # factor on the scores
    rope_base: float = 10000.0
    rope_dims: int | None = None    # rotated part of rot_dim (None: all)
    window: int | None = None       # keys a query sees, itself included
    kv_from: int | None = None      # layer whose latents this layer reads

    @property
    def rotation(self) -> tuple[float, int]:
        return (self.rope_base, self.rope_dims or self.rot_dim)


@dataclass(frozen=True)
class GatedMLPSpec:
    """Clamped gated unit: g = min(gate, limit), u = clamp(up, +-limit),
    y = g * sigmoid(alpha * g) * (u + shift)."""
    ff: int
    limit: float
    alpha: float = 1.702
    shift: float = 1.0


@dataclass(frozen=True)
class LayerSpec:
    """One layer of a model whose layers differ: both sublayers read the
    same normed input and are summed into a 32-bit residual."""
    mixer: LatentAttentionSpec
    mlp: GatedMLPSpec | None


@dataclass
class ModelConfig:
    name: str
    vocab_size: int
    hidden_size: int
    num_layers: int
    num_heads: int
    num_kv_heads: int
    intermediate_size: int
    max_seq_len: int = 4096
    head_dim: int | None = None
    norm: str = "rmsnorm"            # rmsnorm | layernorm
    norm_eps: float = 1e-5
    act: str = "silu_glu"            # silu_glu | gelu | relu
    pos: str = "rope"                # rope | learned
    rope_theta: float = 10000.0
    parallel_residual: bool = False  # falcon-style attn+mlp parallel block
    single_norm: bool = False        # falcon-7b: one shared ln for attn+mlp
    # sliding-window attention width (mistral). Enforced by the serving
    # engine at BLOCK_SIZE granularity (up to BLOCK_SIZE-1 extra tokens
    # of context vs the strict window); expired KV blocks are freed.
    sliding_window: int | None = None
    tie_embeddings: bool = False
    mlp_bias: bool = False
    attn_bias: bool = False   # bias on q/k/v AND o_proj (OPT)
    qkv_bias: bool = False    # bias on q/k/v only (qwen2)
    embed_scale: float = 1.0  # gemma multiplies embeddings by sqrt(hidden)
    # models described layer by layer (None: every layer is the one the
    # fields above describe)
    layers: tuple[LayerSpec, ...] | None = None

    def __post_init__(self):
        if self.layers is not None:
            self.layers = tuple(self.layers)
            self._check_layers()
        if self.head_dim is None:
            self.head_dim = self.hidden_size // self.num_heads

    def _check_layers(self):
        for i, lay in enumerate(self.layers):
            m = lay.mixer
            if min(m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank) < 1 or \
                    m.rotation[1] % 2 or m.rotation[1] > m.rot_dim:
                raise ValueError(f"layer {i}: bad mixer sizes {m}")
            if m.window is not None and m.window < 1:
                raise ValueError(f"layer {i}: window {m.window}")
            if m.kv_from is None:
                continue
            if not 0 <= m.kv_from < i:
                raise ValueError(f"layer {i}: kv_from {m.kv_from}")
            src = self.layers[m.kv_from].mixer
            if src.kv_from is not None or \
                    (src.kv_rank, src.rot_dim, src.rotation) != \
                    (m.kv_rank, m.rot_dim, m.rotation):
                raise ValueError(f"layer {i} cannot read the latents of "
                                 f"layer {m.kv_from}: {src} vs {m}")

    @property
    def params_b(self) -> float:
        """Rough parameter count in billions."""
        if self.layers is not None:
            n = 2 * self.vocab_size * self.hidden_size
            for lay in self.layers:
                m, h = lay.mixer, self.hidden_size
                n += h * m.heads * (m.dim + m.rot_dim + 2 * m.vdim) + \
                    m.kv_rank * m.heads * (m.dim + m.vdim)
                if m.kv_from is None:
                    n += h * (m.kv_rank + m.rot_dim)
                if lay.mlp is not None:
                    n += 3 * h * lay.mlp.ff
            return n / 1e9
        h, l, v = self.hidden_size, self.num_layers, self.vocab_size
        kvh = self.num_kv_heads * self.head_dim
        attn = h * (self.num_heads * self.head_dim) + 2 * h * kvh + \
            self.num_heads * self.head_dim * h
        mlp = (3 if self.act == "silu_glu" else 2) * h * self.intermediate_size
        emb = v * h * (1 if self.tie_embeddings else 2)
        return (l * (attn + mlp) + emb) / 1e9


def layered_config(name: str, layers, width: int, vocab: int,
                   norm_eps: float = 1e-5,
                   max_seq_len: int = 131072) -> ModelConfig:
    """A ModelConfig of a layer-by-layer model. The engine-wide fields
    follow from the layers: cached tokens may be dropped once they are
    outside every layer's window."""
    layers = tuple(layers)
    windows = [lay.mixer.window for lay in layers]
    m = layers[0].mixer
    return ModelConfig(
        name, vocab_size=vocab, hidden_size=width, num_layers=len(layers),
        num_heads=max(lay.mixer.heads for lay in layers), num_kv_heads=1,
        intermediate_size=max((lay.mlp.ff for lay in layers if lay.mlp),
                              default=0),
        max_seq_len=max_seq_len, head_dim=m.dim + m.rot_dim,
        norm_eps=norm_eps, parallel_residual=True, single_norm=True,
        sliding_window=None if None in windows else max(windows),
        layers=layers)


_REGISTRY: dict[str, ModelConfig] = {}


def register(cfg: ModelConfig) -> ModelConfig:
    _REGISTRY[cfg.name] = cfg
    return cfg


def get_config(name: str) -> ModelConfig:
    if name not in _REGISTRY:
        raise KeyError(f"unknown model config '{name}'; have {sorted(_REGISTRY)}")
    return _REGISTRY[name]


def list_configs() -> list[str]:
    return sorted(_REGISTRY)


# --- llama2 family (RMSNorm, RoPE, SwiGLU) ---------------------------------
register(ModelConfig("llama2-7b", vocab_size=32000, hidden_size=4096,
                     num_layers=32, num_heads=32, num_kv_heads=32,
                     intermediate_size=11008))
register(ModelConfig("llama2-13b", vocab_size=32000, hidden_size=5120,
                     num_layers=40, num_heads=40, num_kv_heads=40,
                     intermediate_size=13824))
register(ModelConfig("llama2-70b", vocab_size=32000, hidden_size=8192,
                     num_layers=80, num_heads=64, num_kv_heads=8,
                     intermediate_size=28672))

register(ModelConfig("llama-1b", vocab_size=32000, hidden_size=2048,
                     num_layers=16, num_heads=32, num_kv_heads=32,
                     intermediate_size=5632))

register(ModelConfig("llama3-8b", vocab_size=128256, hidden_size=4096,
                     num_layers=32, num_heads=32, num_kv_heads=8,
                     intermediate_size=14336, max_seq_len=8192,
                     rope_theta=500000.0))
register(ModelConfig("llama3-70b", vocab_size=128256, hidden_size=8192,
                     num_layers=80, num_heads=64, num_kv_heads=8,
                     intermediate_size=28672, max_seq_len=8192,
                     rope_theta=500000.0))
# mistral-7b: llama-shaped GQA-8 with a 4k sliding window (the engine
# enforces it block-aligned and frees expired KV blocks)
register(ModelConfig("mistral-7b", vocab_size=32000, hidden_size=4096,
                     num_layers=32, num_heads=32, num_kv_heads=8,
                     intermediate_size=14336, max_seq_len=8192,
                     rope_theta=1000000.0, sliding_window=4096))

# --- qwen2 family (llama-shaped + q/k/v bias, GQA, huge vocab) -------------
register(ModelConfig("qwen2-7b", vocab_size=152064, hidden_size=3584,
                     num_layers=28, num_heads=28, num_kv_heads=4,
                     intermediate_size=18944, max_seq_len=32768,
                     norm_eps=1e-6, rope_theta=1000000.0, qkv_bias=True))

# --- gemma family (GeGLU, RMSNorm(1+w) folded at load, scaled embed) -------
register(ModelConfig("gemma-7b", vocab_size=256000, hidden_size=3072,
                     num_layers=28, num_heads=16, num_kv_heads=16,
                     intermediate_size=24576, max_seq_len=8192, head_dim=256,
                     norm_eps=1e-6, act="gelu_glu", tie_embeddings=True,
                     embed_scale=3072 ** 0.5))

# --- falcon family (LayerNorm, RoPE, GELU, parallel residual, MQA/GQA) -----
register(ModelConfig("falcon-7b", vocab_size=65024, hidden_size=4544,
                     num_layers=32, num_heads=71, num_kv_heads=1,
                     intermediate_size=4 * 4544, head_dim=64,
                     norm="layernorm", act="gelu", parallel_residual=True,
                     single_norm=True, tie_embeddings=True))
register(ModelConfig("falcon-40b", vocab_size=65024, hidden_size=8192,
                     num_layers=60, num_heads=128, num_kv_heads=8,
                     intermediate_size=4 * 8192, head_dim=64,
                     norm="layernorm", act="gelu", parallel_residual=True,
                     tie_embeddings=True))

# --- GPT-2 family (LayerNorm, learned positions, tanh-GELU, biases) --------
register(ModelConfig("gpt2", vocab_size=50257, hidden_size=768,
                     num_layers=12, num_heads=12, num_kv_heads=12,
                     intermediate_size=3072, max_seq_len=1024,
                     norm="layernorm", act="gelu_tanh", pos="learned",
                     tie_embeddings=True, mlp_bias=True, attn_bias=True))
register(ModelConfig("gpt2-xl", vocab_size=50257, hidden_size=1600,
                     num_layers=48, num_heads=25, num_kv_heads=25,
                     intermediate_size=6400, max_seq_len=1024,
                     norm="layernorm", act="gelu_tanh", pos="learned",
                     tie_embeddings=True, mlp_bias=True, attn_bias=True))

# --- OPT family (LayerNorm, learned positions, ReLU) -----------------------
register(ModelConfig("opt-125m", vocab_size=50272, hidden_size=768,
                     num_layers=12, num_heads=12, num_kv_heads=12,
                     intermediate_size=3072, max_seq_len=2048,
                     norm="layernorm", act="relu", pos="learned",
                     tie_embeddings=True, mlp_bias=True, attn_bias=True))

# --- small GPU smoke config (head_dim 64 => decode-kernel compatible) ------
register(ModelConfig("smoke-llama", vocab_size=512, hidden_size=256,
                     num_layers=2, num_heads=4, num_kv_heads=2,
                     intermediate_size=512, max_seq_len=256))

# --- small GPU smoke config for the gemma family (Dh=256 kernels) ----------
register(ModelConfig("smoke-gemma", vocab_size=512, hidden_size=512,
                     num_layers=2, num_heads=2, num_kv_heads=2,
                     intermediate_size=1024, max_seq_len=256, head_dim=256,
                     norm_eps=1e-6, act="gelu_glu", tie_embeddings=True,
                     embed_scale=512 ** 0.5))

# --- tiny configs for CPU tests --------------------------------------------
register(ModelConfig("tiny-llama", vocab_size=256, hidden_size=64,
                     num_layers=2, num_heads=4, num_kv_heads=2,
                     intermediate_size=128, max_seq_len=128))
register(ModelConfig("tiny-falcon", vocab_size=256, hidden_size=64,
                     num_layers=2, num_heads=8, num_kv_heads=1,
                     intermediate_size=128, head_dim=8, max_seq_len=128,
                     norm="layernorm", act="gelu", parallel_residual=True,
                     single_norm=True, tie_embeddings=True))
# 8 heads / 8 kv-heads so CPU torchrun rehearsals of the driver's TP=8
# scale command work on gloo (tiny-llama's 4 heads can't split 8 ways)
register(ModelConfig("tiny-llama-8h", vocab_size=256, hidden_size=64,
                     num_layers=2, num_heads=8, num_kv_heads=8,
                     intermediate_size=128, head_dim=8, max_seq_len=128))
register(ModelConfig("tiny-qwen", vocab_size=256, hidden_size=64,
                     num_layers=2, num_heads=4, num_kv_heads=2,
                     intermediate_size=128, max_seq_len=128,
                     norm_eps=1e-6, qkv_bias=True))
register(ModelConfig("tiny-gemma", vocab_size=256, hidden_size=64,
                     num_layers=2, num_heads=4, num_kv_heads=2,
                     intermediate_size=128, head_dim=16, max_seq_len=128,
                     norm_eps=1e-6, act="gelu_glu", tie_embeddings=True,
                     embed_scale=8.0))
register(ModelConfig("tiny-gpt2", vocab_size=256, hidden_size=64,
                     num_layers=2, num_heads=4, num_kv_heads=4,
                     intermediate_size=128, max_seq_len=128,
                     norm="layernorm", act="gelu_tanh", pos="learned",
                     tie_embeddings=True, mlp_bias=True, attn_bias=True))
register(ModelConfig("tiny-opt", vocab_size=256, hidden_size=64,
                     num_layers=2, num_heads=4, num_kv_heads=4,
                     intermediate_size=128, max_seq_len=128,
                     norm="layernorm", act="relu", pos="learned",
                     tie_embeddings=True, mlp_bias=True, attn_bias=True))


# --- Pimazen family (latent attention in parallel with a clamped gated MLP) --
def _pimazen(name: str, n_layers: int, width: int, vocab: int, ff, mixer,
             share_every: int = 0, limit: float = 7.0, **kw) -> ModelConfig:
    """Equal layers; with share_every = n, n - 1 of n layers read the
    latents of the first one of their group."""
    layers = []
    for i in range(n_layers):
        first = i - i % share_every if share_every else i
        src = None if first == i else first
        layers.append(LayerSpec(
            LatentAttentionSpec(kv_from=src, **mixer),
            GatedMLPSpec(ff, limit) if ff else None))
    return register(layered_config(name, layers, width, vocab, **kw))


_pimazen("tiny-pimazen", 3, 64, 256, 96,
         dict(heads=3, dim=24, rot_dim=8, vdim=16, kv_rank=40, window=24,
              scale=32 ** -0.5), share_every=2, max_seq_len=256)
_pimazen("smoke-pimazen", 4, 256, 512, 384,
         dict(heads=4, dim=64, rot_dim=32, vdim=64, kv_rank=128, window=96,
              scale=96 ** -0.5), share_every=2, max_seq_len=1024)
# layers of the width, heads and mlp of llama2-7b and llama-1b
_pimazen("pimazen-7b", 32, 4096, 32000, 11008,
         dict(heads=32, dim=128, rot_dim=64, vdim=128, kv_rank=512,
              window=4096, scale=192 ** -0.5, rope_base=1000000.0),
         share_every=2, max_seq_len=32768)
_pimazen("pimazen-1b", 16, 2048, 32000, 5632,
         dict(heads=32, dim=64, rot_dim=32, vdim=64, kv_rank=256,
              window=2048, scale=96 ** -0.5), share_every=2,
         max_seq_len=32768)
