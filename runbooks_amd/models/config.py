"""Model configurations for the families the reference platform serves.

The reference orchestrates external HuggingFace images for these models
(reference examples/: facebook-opt-125m, llama2-7b, llama2-70b,
falcon-7b-instruct, falcon-40b). Here they are first-class configs of our
own runtime.
"""
from __future__ import annotations

import math
from dataclasses import dataclass


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Latent attention: keys and values are linear images of one cached
    latent per token (plus one rotated key part all heads share, unless
    rot_dim is 0). A sigmoid gate on the result, one per value column or,
    with head_gate, one per head."""
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
    q_rank: int | None = None       # latent of the queries (None: direct)
    head_gate: bool = False

    @property
    def rotation(self) -> tuple[float, int] | None:
        if self.rot_dim == 0:
            return None
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
class RopeScaling:
    """Frequency scaling by wavelength: up to original / high tokens kept,
    beyond original / low divided by `factor`, blended between."""
    factor: float
    low: float
    high: float
    original: float


@dataclass(frozen=True)
class SharedKVAttentionSpec:
    """Grouped-query attention without a value projection: a token's key,
    before rotation, doubles as its value. The first rope_dims dimensions of
    a head rotate (in halves)."""
    heads: int
    kv_heads: int
    dim: int                        # query, key and value size per head
    scale: float                    # factor on the scores
    rope_dims: int
    rope_base: float = 10000.0
    rope_scaling: RopeScaling | None = None
    window: int | None = None       # keys a query sees, itself included

    @property
    def rotation(self):
        return (self.rope_base, self.rope_dims, self.rope_scaling)


@dataclass(frozen=True)
class LightningSpec:
    """Linear attention with a fixed decay per head and a [dim, vdim] state
    per head and sequence; RMS norm over all heads, sigmoid output gate."""
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]

    rotation = None


@dataclass(frozen=True)
class GatedDeltaSpec:
    """Gated delta rule with one decay per head and key channel: q, k, v pass
    a short causal convolution and silu, q and k become unit vectors;
    S <- g S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q; RMS norm per
    head, sigmoid gate. Decay logits and gate come through a bottleneck."""
    heads: int
    kv_heads: int                   # q/k heads
    dim: int
    vdim: int
    conv: int                       # taps of the convolution
    decay_rank: int
    gate_rank: int

    rotation = None


@dataclass(frozen=True)
class AttentionSpec:
    """Grouped-query attention with RMS norms of queries and keys, rotation
    of the first rope_dims dimensions in neighbouring pairs, and a learned
    sink in the softmax. A query sees the keys of its own chunk, counted
    from the sequence's start."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float                    # factor on the scores
    rope_dims: int
    rope_base: float = 10000.0
    chunk: int | None = None        # tokens per chunk (None: one chunk)

    @property
    def rotation(self):
        return (self.rope_base, self.rope_dims)


@dataclass(frozen=True)
class MinGRUSpec:
    """Gated recurrence S <- (1 - z) S + z c whose gates read only the
    current token; the result is S silu(gate)."""
    width: int


@dataclass(frozen=True)
class TwinSpec:
    """Two mixers side by side on the same input; their results are added
    with a factor each."""
    left: AttentionSpec
    right: MinGRUSpec
    left_scale: float = 1.0
    right_scale: float = 1.0

    @property
    def rotation(self):
        return self.left.rotation

    @property
    def chunk(self):
        return self.left.chunk


@dataclass(frozen=True)
class GeneralDeltaSpec:
    """Generalized delta rule with a decay w and a removal rate a per head
    and key channel: S <- diag(w) S - (a u)(u^T S) + k v^T with u = k / |k|,
    o = S^T r; RMS norm per head, sigmoid gate. w = exp(decay_scale
    sigmoid(..)) comes through a tanh bottleneck."""
    heads: int
    dim: int
    decay_rank: int
    decay_scale: float = -math.exp(-0.5)

    rotation = None

    @property
    def vdim(self):
        return self.dim


@dataclass(frozen=True)
class DiffAttentionSpec:
    """Differential attention: two attention maps per head over the same
    values, the second one subtracted times a learned factor, RMS norm per
    head. Biased q, k, v pass a short causal convolution; no rotation."""
    heads: int
    kv_heads: int
    dim: int                        # query/key size per head and map
    vdim: int
    scale: float                    # factor on the scores
    diff: float                     # constant part of the factor
    conv: int                       # taps of the convolution
    window: int | None = None       # keys a query sees, itself included

    rotation = None


@dataclass(frozen=True)
class PolyNormSpec:
    """Feed-forward down(a N(z) + b N(z^2) + c N(z^3) + e), z = up, N an RMS
    norm over all ff values."""
    ff: int


@dataclass(frozen=True)
class SquaredReluSpec:
    """Feed-forward down(relu(up)^2)."""
    ff: int


@dataclass(frozen=True)
class MoESpec:
    """`top` of `experts` squared-ReLU units per token, by softmax scores
    plus a correction, out of the `keep` best of `groups` groups; weighted
    by the scores. A shared unit of size shared_ff (0: none) is added."""
    ff: int                         # of one expert
    experts: int
    top: int
    groups: int = 1
    keep: int = 1
    shared_ff: int = 0


@dataclass(frozen=True)
class GLUSpec:
    """Gated unit act(gate) * up."""
    ff: int
    act: str = "gelu_tanh"


@dataclass(frozen=True)
class LayerSpec:
    """One layer of a model whose layers differ, on a 32-bit residual.
    ModelConfig.layout says how its sublayers follow each other."""
    mixer: (LatentAttentionSpec | SharedKVAttentionSpec | LightningSpec |
            GatedDeltaSpec | TwinSpec | GeneralDeltaSpec | DiffAttentionSpec)
    mlp: (GatedMLPSpec | GLUSpec | SquaredReluSpec | MoESpec | PolyNormSpec |
          None)
    weights_of: int | None = None   # layer whose parameters this one uses

    @property
    def attends(self) -> bool:
        """The mixer reads cached keys."""
        return not isinstance(self.mixer, (LightningSpec, GatedDeltaSpec,
                                           GeneralDeltaSpec))

    @property
    def reach(self) -> int | None:
        """Most keys a query sees, itself included (None: all)."""
        return getattr(self.mixer, "window", None) or \
            getattr(self.mixer, "chunk", None)

    def first_key(self, pos: int) -> int:
        """First position that a query at `pos` or later can see."""
        if not self.attends:
            return pos
        chunk = getattr(self.mixer, "chunk", None)
        if chunk is not None:
            return pos - pos % chunk
        window = getattr(self.mixer, "window", None)
        return 0 if window is None else max(0, pos - window + 1)


@dataclass(frozen=True)
class LoopSpec:
    """Layers start .. stop - 1 run `times` times in a row with the same
    weights, each pass on a cache of its own, behind a projection of
    [residual; embedding output] that replaces the residual; with `step`, a
    learned vector of the pass is then added."""
    start: int
    stop: int
    times: int
    step: bool = False


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
    norm: str = "rmsnorm"            # rmsnorm | layernorm | dyt
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
    loop: LoopSpec | None = None
    # residual streams with learned mixing (None: one plain residual), and
    # the factor on a sublayer's result that goes with them
    streams: int | None = None
    residual_mult: float = 1.0
    # taps of a causal convolution that every sublayer's normed input passes
    # (None: none); such sublayers run in parallel, each behind its own norm
    canon: int | None = None
    norm_offset: float = 0.0  # added to the weights of RMS norms
    logit_softcap: float | None = None   # logits -> cap tanh(logits / cap)

    def __post_init__(self):
        if self.layers is not None:
            self.layers = tuple(self.layers)
            self._check_layers()
        if self.head_dim is None:
            self.head_dim = self.hidden_size // self.num_heads

    @property
    def layout(self) -> str:
        """How a layer-by-layer model's sublayers meet: "streams" (several
        residuals with learned mixing), "dual" (in parallel, each behind a
        norm and input convolution of its own), "shared" (in parallel on one
        normed input) or "sequence" (one after the other)."""
        if self.streams is not None:
            return "streams"
        if self.canon is not None:
            return "dual"
        latent = isinstance(self.layers[0].mixer, LatentAttentionSpec)
        return "shared" if latent else "sequence"

    @property
    def layer_runs(self) -> list[tuple[int, int | None]]:
        """(layer, number of the loop pass it starts or None) in the order
        of execution."""
        n, loop = len(self.layers), self.loop
        if loop is None:
            return [(self.owner(i), None) for i in range(n)]
        body = range(loop.start, loop.stop)
        return ([(i, None) for i in range(loop.start)] +
                [(i, t if i == loop.start else None)
                 for t in range(loop.times) for i in body] +
                [(i, None) for i in range(loop.stop, n)])

    def owner(self, i: int) -> int:
        """The layer whose parameters layer i uses."""
        while self.layers[i].weights_of is not None:
            i = self.layers[i].weights_of
        return i

    @property
    def owners(self) -> list[int]:
        """Layers with parameters of their own."""
        return [i for i, lay in enumerate(self.layers)
                if lay.weights_of is None]

    def first_key(self, pos: int) -> int:
        """First position that a query at `pos` or later can see in any
        layer."""
        return min(lay.first_key(pos) for lay in self.layers)

    @property
    def kernel_groups(self) -> tuple[str, ...]:
        """Kernel modules (ops/build.py) that serving this model needs."""
        if self.layers is None:
            return ("core", "main")
        need = {LatentAttentionSpec: "latent",
                SharedKVAttentionSpec: "shared_kv",
                LightningSpec: "lightning", GatedDeltaSpec: "delta",
                GeneralDeltaSpec: "delta", DiffAttentionSpec: "shared_kv",
                TwinSpec: "shared_kv"}
        groups = {need[type(lay.mixer)] for lay in self.layers}
        groups |= {self.layout} & {"streams", "dual"}
        return ("core", *sorted(groups))

    def _check_layers(self):
        checks = {LatentAttentionSpec: self._check_latent,
                  SharedKVAttentionSpec: self._check_shared_kv,
                  LightningSpec: self._check_lightning,
                  GatedDeltaSpec: self._check_delta,
                  TwinSpec: self._check_twin,
                  GeneralDeltaSpec: self._check_general_delta,
                  DiffAttentionSpec: self._check_diff}
        # what a layout's layers may consist of
        mixers, mlps = {
            "streams": ((GatedDeltaSpec, TwinSpec),
                        (SquaredReluSpec, MoESpec)),
            "dual": ((GeneralDeltaSpec, DiffAttentionSpec,
                      LatentAttentionSpec), (PolyNormSpec,)),
            "shared": ((LatentAttentionSpec,), (GatedMLPSpec,)),
            "sequence": ((SharedKVAttentionSpec, LightningSpec), (GLUSpec,)),
        }[self.layout]
        for i, lay in enumerate(self.layers):
            if not isinstance(lay.mixer, mixers):
                raise ValueError(f"layer {i}: no {lay.mixer} in the layout "
                                 f"{self.layout!r}")
            if getattr(lay.mixer, "window", None) is not None and \
                    lay.mixer.window < 1:
                raise ValueError(f"layer {i}: window {lay.mixer.window}")
            checks[type(lay.mixer)](i, lay.mixer)
            if lay.mlp is not None and (
                    lay.mlp.ff < 1 or not isinstance(lay.mlp, mlps)):
                raise ValueError(f"layer {i}: mlp {lay.mlp}")
            if isinstance(lay.mlp, MoESpec):
                self._check_moe(i, lay.mlp)
            self._check_owner(i, lay)
            if getattr(lay.mlp, "act", "gelu_tanh") != "gelu_tanh":
                raise ValueError(f"layer {i}: activation {lay.mlp.act}")
        if self.loop is not None:
            lo = self.loop
            if not 0 <= lo.start < lo.stop <= len(self.layers) or \
                    lo.times < 1:
                raise ValueError(f"bad loop {lo}")
            if any(getattr(lay.mixer, "kv_from", None) is not None
                   for lay in self.layers):
                raise ValueError("no loop over layers that share latents")

        if self.streams is not None and (self.streams < 1 or self.loop or
                                         self.norm != "dyt"):
            raise ValueError(f"bad streams {self.streams}")
        if self.canon is not None and (self.canon < 1 or
                                       self.norm != "rmsnorm"):
            raise ValueError(f"bad input convolution {self.canon}")
        if self.logit_softcap is not None and self.logit_softcap <= 0:
            raise ValueError(f"bad logit_softcap {self.logit_softcap}")

    def _check_owner(self, i, lay):
        """Layer i's weights_of leads to a layer like it that has some."""
        seen, j = {i}, lay.weights_of
        while j is not None:
            if j in seen or not 0 <= j < len(self.layers) or self.loop or \
                    (self.layers[j].mixer, self.layers[j].mlp) != \
                    (lay.mixer, lay.mlp):
                raise ValueError(f"layer {i} cannot use the weights of "
                                 f"layer {lay.weights_of}")
            seen.add(j)
            j = self.layers[j].weights_of

    def _check_delta(self, i, m):
        if min(m.heads, m.kv_heads, m.dim, m.vdim, m.conv, m.decay_rank,
               m.gate_rank) < 1 or m.heads % m.kv_heads:
            raise ValueError(f"layer {i}: bad mixer sizes {m}")

    def _check_twin(self, i, m):
        a = m.left
        if min(a.heads, a.kv_heads, a.dim, a.vdim, m.right.width) < 1 or \
                a.heads % a.kv_heads or a.rope_dims % 2 or \
                not 0 <= a.rope_dims <= a.dim or \
                (a.chunk is not None and a.chunk < 1):
            raise ValueError(f"layer {i}: bad mixer sizes {m}")

    def _check_general_delta(self, i, m):
        if min(m.heads, m.dim, m.decay_rank) < 1 or \
                not -2.0 <= m.decay_scale <= 0.0:
            raise ValueError(f"layer {i}: bad mixer sizes {m}")

    def _check_diff(self, i, m):
        if min(m.heads, m.kv_heads, m.dim, m.vdim, m.conv) < 1 or \
                m.heads % m.kv_heads:
            raise ValueError(f"layer {i}: bad mixer sizes {m}")

    def _check_moe(self, i, m):
        if m.experts < 1 or m.groups < 1 or m.experts % m.groups or \
                not 1 <= m.keep <= m.groups or m.shared_ff < 0 or \
                not 1 <= m.top <= m.experts // m.groups * m.keep:
            raise ValueError(f"layer {i}: bad mixture {m}")

    def _check_latent(self, i, m):
        rot = m.rotation[1] if m.rotation else 0
        q_rank = 1 if m.q_rank is None else m.q_rank
        if min(m.heads, m.dim, m.vdim, m.kv_rank, q_rank) < 1 or \
                rot % 2 or not 0 <= rot <= m.rot_dim:
            raise ValueError(f"layer {i}: bad mixer sizes {m}")
        # the "dual" layout has the one form, the "shared" one the other
        dual = self.layout == "dual"
        if (m.q_rank is not None, m.head_gate, m.rot_dim == 0) != (dual,) * 3 \
                or (dual and m.kv_from is not None):
            raise ValueError(f"layer {i}: latent attention {m} in the layout "
                             f"{self.layout!r}")
        if m.kv_from is None:
            return
        if not 0 <= m.kv_from < i:
            raise ValueError(f"layer {i}: kv_from {m.kv_from}")
        src = self.layers[m.kv_from].mixer
        if src.kv_from is not None or \
                (src.kv_rank, src.rot_dim, src.rotation) != \
                (m.kv_rank, m.rot_dim, m.rotation):
            raise ValueError(f"layer {i} cannot read the latents of "
                             f"layer {m.kv_from}: {src} vs {m}")

    def _check_shared_kv(self, i, m):
        if min(m.heads, m.kv_heads, m.dim) < 1 or m.heads % m.kv_heads or \
                m.rope_dims % 2 or not 0 <= m.rope_dims <= m.dim:
            raise ValueError(f"layer {i}: bad mixer sizes {m}")

    def _check_lightning(self, i, m):
        if min(m.heads, m.dim, m.vdim) < 1 or len(m.decay) != m.heads or \
                not all(0 <= d <= 1 for d in m.decay):
            raise ValueError(f"layer {i}: bad mixer sizes {m}")

    @property
    def params_b(self) -> float:
        """Rough parameter count in billions."""
        if self.layers is not None:
            n = 2 * self.vocab_size * self.hidden_size
            for lay in (self.layers[i] for i in self.owners):
                m, h = lay.mixer, self.hidden_size
                if isinstance(m, SharedKVAttentionSpec):
                    n += h * m.dim * (2 * m.heads + m.kv_heads)
                elif isinstance(m, LightningSpec):
                    n += h * m.heads * (2 * m.dim + 3 * m.vdim)
                elif isinstance(m, GatedDeltaSpec):
                    n += h * (2 * m.kv_heads * m.dim + m.decay_rank +
                              m.gate_rank + 2 * m.heads * m.vdim)
                    n += m.heads * (m.decay_rank * m.dim +
                                    m.gate_rank * m.vdim)
                elif isinstance(m, TwinSpec):
                    a = m.left
                    n += h * (a.heads + a.kv_heads) * (a.dim + a.vdim) + \
                        4 * h * m.right.width
                elif isinstance(m, GeneralDeltaSpec):
                    n += m.heads * m.dim * (6 * h + m.decay_rank) + \
                        h * m.decay_rank
                elif isinstance(m, DiffAttentionSpec):
                    n += h * (m.heads + m.kv_heads) * (2 * m.dim + m.vdim)
                elif m.q_rank is not None:
                    n += m.q_rank * (h + m.heads * m.dim) + \
                        m.kv_rank * (h + m.heads * (m.dim + m.vdim)) + \
                        h * m.heads * (1 + m.vdim)
                else:
                    n += h * m.heads * (m.dim + m.rot_dim + 2 * m.vdim) + \
                        m.kv_rank * m.heads * (m.dim + m.vdim)
                    if m.kv_from is None:
                        n += h * (m.kv_rank + m.rot_dim)
                if isinstance(lay.mlp, (MoESpec, SquaredReluSpec,
                                        PolyNormSpec)):
                    n += 2 * h * (lay.mlp.ff * getattr(lay.mlp, "experts", 1)
                                  + getattr(lay.mlp, "shared_ff", 0))
                elif lay.mlp is not None:
                    n += 3 * h * lay.mlp.ff
                if self.streams is not None:
                    n += h * h * (1 + (lay.mlp is not None))
            if self.loop is not None:
                n += 2 * self.hidden_size ** 2
            return n / 1e9
        h, l, v = self.hidden_size, self.num_layers, self.vocab_size
        kvh = self.num_kv_heads * self.head_dim
        attn = h * (self.num_heads * self.head_dim) + 2 * h * kvh + \
            self.num_heads * self.head_dim * h
        mlp = (3 if self.act == "silu_glu" else 2) * h * self.intermediate_size
        emb = v * h * (1 if self.tie_embeddings else 2)
        return (l * (attn + mlp) + emb) / 1e9


def layered_config(name: str, layers, width: int, vocab: int,
                   norm_eps: float = 1e-5, max_seq_len: int = 131072,
                   norm: str = "rmsnorm",
                   loop: LoopSpec | None = None, **kw) -> ModelConfig:
    """A ModelConfig of a layer-by-layer model. The engine-wide fields
    follow from the layers: cached tokens may be dropped once they are
    outside every attention layer's window."""
    layers = tuple(layers)
    mixers = [lay.mixer for lay in layers]
    latent = isinstance(mixers[0], LatentAttentionSpec) and \
        kw.get("canon") is None
    # sizes of the attention (a twin mixer's left side)
    heads = [getattr(m, "left", m) for m in mixers]
    windows = [lay.reach for lay in layers if lay.attends]
    return ModelConfig(
        name, vocab_size=vocab, hidden_size=width, num_layers=len(layers),
        num_heads=max(m.heads for m in heads),
        num_kv_heads=1 if latent else max(getattr(m, "kv_heads", 1)
                                          for m in heads),
        intermediate_size=max((lay.mlp.ff for lay in layers if lay.mlp),
                              default=0),
        max_seq_len=max_seq_len,
        head_dim=heads[0].dim + getattr(heads[0], "rot_dim", 0),
        norm=norm, norm_eps=norm_eps, parallel_residual=latent,
        single_norm=latent,
        sliding_window=None if None in windows else max(windows, default=1),
        layers=layers, loop=loop, **kw)


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


# --- Keralorn family (windowed attention with values shared from the keys,
# lightning attention, a looped stretch of layers; LayerNorm, tanh-GELU) -----
def _keralorn(name: str, pattern: str, width: int, vocab: int, ff: int,
              attention: dict, lightning: dict, loop=None, **kw):
    """`pattern`: one letter a layer, A attention or L lightning (upper case
    with a feed-forward, lower case without)."""
    H = lightning["heads"]
    # slowest head: half left after 512 tokens; fastest: after half a token
    decay = tuple(2.0 ** -(2.0 ** (1 - 10 * i / max(1, H - 1)))
                  for i in range(H))
    made = {"a": SharedKVAttentionSpec(**attention),
            "l": LightningSpec(decay=decay, **lightning)}
    layers = [LayerSpec(made[c.lower()], GLUSpec(ff) if c.isupper() else None)
              for c in pattern]
    return register(layered_config(name, layers, width, vocab,
                                   norm="layernorm",
                                   loop=loop and LoopSpec(*loop), **kw))


_keralorn("tiny-keralorn", "AlLa", 64, 256, 96,
          dict(heads=4, kv_heads=2, dim=24, scale=24 ** -0.5, rope_dims=16,
               rope_scaling=RopeScaling(8.0, 1.0, 4.0, 64), window=24),
          dict(heads=3, dim=16, vdim=24), loop=(1, 3, 2), max_seq_len=256)
_keralorn("smoke-keralorn", "AlAL", 256, 512, 384,
          dict(heads=8, kv_heads=2, dim=32, scale=32 ** -0.5, rope_dims=8,
               rope_scaling=RopeScaling(4.0, 1.0, 4.0, 512), window=96),
          dict(heads=4, dim=32, vdim=64), loop=(1, 3, 2), max_seq_len=1024)
# layers of the width, heads and mlp of llama2-7b and llama-1b
_keralorn("keralorn-7b", "AL" * 16, 4096, 32000, 11008,
          dict(heads=32, kv_heads=32, dim=128, scale=128 ** -0.5,
               rope_dims=32, rope_base=500000.0,
               rope_scaling=RopeScaling(8.0, 1.0, 4.0, 8192), window=4096),
          dict(heads=32, dim=128, vdim=128), max_seq_len=32768)
_keralorn("keralorn-1b", "AL" * 8, 2048, 32000, 5632,
          dict(heads=32, kv_heads=32, dim=64, scale=64 ** -0.5, rope_dims=16,
               rope_base=500000.0,
               rope_scaling=RopeScaling(8.0, 1.0, 4.0, 8192), window=2048),
          dict(heads=32, dim=64, vdim=64), max_seq_len=32768)


# --- Gokapel family (gated delta rule, chunked attention beside a minGRU,
# squared-ReLU units and mixtures of them; residual streams, dynamic tanh) ----
def _gokapel(name: str, pattern: str, width: int, vocab: int, ff: int,
             mixture: dict, delta: dict, attention: dict, gru: int, **kw):
    """`pattern`: one letter a layer, D delta or P attention beside a minGRU
    (lower case: the feed-forward is a mixture), or a digit: the weights of
    that layer."""
    made = {"d": GatedDeltaSpec(**delta),
            "p": TwinSpec(AttentionSpec(**attention), MinGRUSpec(gru),
                          0.75, 0.5)}
    layers: list[LayerSpec] = []
    for c in pattern:
        if c.isdigit():
            src = layers[int(c)]
            layers.append(LayerSpec(src.mixer, src.mlp, int(c)))
        else:
            layers.append(LayerSpec(
                made[c.lower()],
                SquaredReluSpec(ff) if c.isupper() else MoESpec(**mixture)))
    kw = {"streams": 4, "residual_mult": 0.8, "embed_scale": width ** 0.5,
          **kw}
    return register(layered_config(name, layers, width, vocab, norm="dyt",
                                   tie_embeddings=True, **kw))


_gokapel("tiny-gokapel", "DpPd0", 64, 256, 96,
         dict(ff=24, experts=8, top=2, groups=4, keep=2, shared_ff=40),
         dict(heads=4, kv_heads=2, dim=16, vdim=24, conv=4, decay_rank=8,
              gate_rank=12),
         dict(heads=4, kv_heads=2, dim=24, vdim=16, scale=24 ** -0.5,
              rope_dims=16, chunk=24), 40, max_seq_len=256)
_gokapel("smoke-gokapel", "DpdP1", 256, 512, 512,
         dict(ff=128, experts=8, top=2, groups=2, keep=1, shared_ff=128),
         dict(heads=4, kv_heads=4, dim=64, vdim=64, conv=4, decay_rank=32,
              gate_rank=32),
         dict(heads=4, kv_heads=2, dim=64, vdim=64, scale=64 ** -0.5,
              rope_dims=32, chunk=96), 256, max_seq_len=1024)
# layers of the width and heads of llama2-7b and llama-1b; a dense layer has
# llama's feed-forward parameters, and so has what a token uses of a mixture
_gokapel("gokapel-7b", "DpPd" * 4, 4096, 32000, 16384,
         dict(ff=2048, experts=32, top=6, groups=4, keep=2, shared_ff=4096),
         dict(heads=32, kv_heads=32, dim=128, vdim=128, conv=4,
              decay_rank=128, gate_rank=128),
         dict(heads=32, kv_heads=32, dim=128, vdim=128, scale=128 ** -0.5,
              rope_dims=64, rope_base=500000.0, chunk=4096), 4096,
         max_seq_len=32768)
_gokapel("gokapel-1b", "DpPd" * 4, 2048, 32000, 8192,
         dict(ff=1024, experts=32, top=6, groups=4, keep=2, shared_ff=2048),
         dict(heads=16, kv_heads=16, dim=128, vdim=128, conv=4,
              decay_rank=128, gate_rank=128),
         dict(heads=32, kv_heads=32, dim=64, vdim=64, scale=64 ** -0.5,
              rope_dims=32, rope_base=500000.0, chunk=2048), 2048,
         max_seq_len=32768)


# --- Dopilorn family (generalized delta rule, differential and positionless
# latent attention beside a PolyNorm unit, each behind a norm and an input
# convolution; a looped stretch of layers) --------------------------------------
def _dopilorn(name: str, pattern: str, width: int, vocab: int, ff: int,
              delta: dict, attention: dict, latent: dict, loop=None,
              **kw) -> ModelConfig:
    """`pattern`: one letter a layer, D delta, A attention or L latent
    attention (upper case with a feed-forward, lower case without)."""
    made = {"d": GeneralDeltaSpec(**delta),
            "a": DiffAttentionSpec(**attention),
            "l": LatentAttentionSpec(rot_dim=0, head_gate=True, **latent)}
    layers = [LayerSpec(made[c.lower()],
                        PolyNormSpec(ff) if c.isupper() else None)
              for c in pattern]
    kw = {"canon": 4, "logit_softcap": 30.0, "norm_offset": 1.0, **kw}
    return register(layered_config(
        name, layers, width, vocab,
        loop=loop and LoopSpec(*loop, step=True), **kw))


_dopilorn("tiny-dopilorn", "AdLD", 64, 256, 96,
          dict(heads=3, dim=16, decay_rank=8),
          dict(heads=4, kv_heads=2, dim=12, vdim=24, scale=12 ** -0.5,
               diff=0.5, conv=3, window=24),
          dict(heads=3, dim=16, vdim=24, q_rank=40, kv_rank=24,
               scale=0.25), loop=(1, 3, 2), max_seq_len=256)
_dopilorn("smoke-dopilorn", "ALdA", 256, 512, 512,
          dict(heads=4, dim=64, decay_rank=32),
          dict(heads=4, kv_heads=2, dim=32, vdim=64, scale=32 ** -0.5,
               diff=0.5, conv=3, window=80),
          dict(heads=4, dim=64, vdim=64, q_rank=96, kv_rank=64, scale=0.125),
          loop=(1, 3, 2), max_seq_len=1024)
# layers of the width of llama2-7b and llama-1b and with about as many
# parameters
_dopilorn("dopilorn-7b", "ADLD" * 4, 4096, 32000, 16384,
          dict(heads=32, dim=128, decay_rank=128),
          dict(heads=16, kv_heads=16, dim=128, vdim=256, scale=128 ** -0.5,
               diff=0.5, conv=4, window=4096),
          dict(heads=32, dim=128, vdim=128, q_rank=1536, kv_rank=512,
               scale=128 ** -0.5), max_seq_len=32768)
_dopilorn("dopilorn-1b", "ADLD" * 4, 2048, 32000, 8192,
          dict(heads=16, dim=128, decay_rank=64),
          dict(heads=16, kv_heads=16, dim=64, vdim=128, scale=64 ** -0.5,
               diff=0.5, conv=4, window=2048),
          dict(heads=32, dim=64, vdim=64, q_rank=768, kv_rank=256,
               scale=64 ** -0.5), max_seq_len=32768)
