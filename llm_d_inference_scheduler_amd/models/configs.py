"""Model architecture configs.

`ModelConfig` describes the uniform decoder families (Llama, Qwen, LLaVA
text tower). `LayeredConfig` describes designs that list their layers one by
one: every layer names its mixer (a recurrent one, an attention one, ...)
with sizes of its own, and its feed-forward.
"""
from dataclasses import dataclass
from typing import Optional, Tuple, Union


@dataclass(frozen=True)
class ModelConfig:
    name: str
    vocab_size: int
    hidden_size: int
    intermediate_size: int
    num_layers: int
    num_heads: int
    num_kv_heads: int
    head_dim: int
    rope_theta: float = 500000.0
    rms_eps: float = 1e-5
    max_position: int = 8192
    tie_embeddings: bool = False
    # Qwen3-style per-head RMSNorm of Q and K before RoPE
    qk_norm: bool = False
    # multimodal (encode role): simple ViT-style tower when set
    vision_hidden: int = 0
    vision_layers: int = 0
    vision_patches: int = 0

    @property
    def q_size(self) -> int:
        return self.num_heads * self.head_dim

    @property
    def kv_size(self) -> int:
        return self.num_kv_heads * self.head_dim

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return 2 * self.num_layers * self.kv_size * dtype_bytes


LLAMA_3_8B = ModelConfig(
    name="llama-3-8b", vocab_size=128256, hidden_size=4096,
    intermediate_size=14336, num_layers=32, num_heads=32, num_kv_heads=8,
    head_dim=128, rope_theta=500000.0)

# Qwen3-32B — the model the reference's regression harness drives
# (config/manifests/regression-testing/single-workload-regression.yaml:
# Qwen3-32B, input 1024 / output 1024). GQA 64q/8kv, head_dim 128,
# per-head QK-RMSNorm; ~64 GB bf16 weights fit one MI355X beside a
# >100 GB KV pool.
QWEN3_32B = ModelConfig(
    name="qwen3-32b", vocab_size=151936, hidden_size=5120,
    intermediate_size=25600, num_layers=64, num_heads=64, num_kv_heads=8,
    head_dim=128, rope_theta=1000000.0, rms_eps=1e-6, qk_norm=True,
    max_position=8192)

TINY_QWEN = ModelConfig(
    name="tiny-qwen", vocab_size=1024, hidden_size=256,
    intermediate_size=512, num_layers=2, num_heads=8, num_kv_heads=4,
    head_dim=32, rope_theta=10000.0, max_position=512, qk_norm=True)

# LLaVA-1.5-7B language tower (Vicuna-7B shape) + ViT-L/14-336 vision tower
LLAVA_1_5_7B_TEXT = ModelConfig(
    name="llava-1.5-7b", vocab_size=32064, hidden_size=4096,
    intermediate_size=11008, num_layers=32, num_heads=32, num_kv_heads=32,
    head_dim=128, rope_theta=10000.0,
    vision_hidden=1024, vision_layers=24, vision_patches=576)

TINY_LLAMA = ModelConfig(
    name="tiny-llama", vocab_size=1024, hidden_size=256,
    intermediate_size=512, num_layers=2, num_heads=8, num_kv_heads=4,
    head_dim=32, rope_theta=10000.0, max_position=512)

TINY_LLAVA = ModelConfig(
    name="tiny-llava", vocab_size=1024, hidden_size=256,
    intermediate_size=512, num_layers=2, num_heads=8, num_kv_heads=4,
    head_dim=32, rope_theta=10000.0, max_position=512,
    vision_hidden=64, vision_layers=2, vision_patches=8)


# ---- designs that list their layers -----------------------------------------
@dataclass(frozen=True)
class RotarySpec:
    """Rotary positions; `factor` set means YaRN frequency scaling."""
    dims: int
    base: float
    interleaved: bool = True        # pairs (2i, 2i+1); else (i, i + dims/2)
    factor: Optional[float] = None
    original: float = 0.0           # context length before scaling
    fast: float = 32.0              # turns per `original` kept unscaled
    slow: float = 1.0               # turns per `original` fully scaled


@dataclass(frozen=True)
class ChannelDeltaSpec:
    """Gated delta rule with one decay per head and key channel."""
    heads: int
    kv_heads: int                   # heads of q and k (each serves a group)
    dim: int                        # key channels
    vdim: int
    conv: int                       # taps of the short causal convolution
    decay_rank: int                 # inner size of the decay projection
    gate_rank: int                  # inner size of the output gate
    unit_eps: float = 1e-6          # of the unit norm of q and k

    @property
    def conv_channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def state_shapes(self) -> Tuple[Tuple[int, ...], Tuple[int, ...]]:
        """Per sequence: matrix state (32-bit), convolution inputs."""
        return ((self.heads, self.dim, self.vdim),
                (self.conv - 1, self.conv_channels))


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Attention over a low-rank latent shared by all heads."""
    heads: int
    dim: int                        # unrotated query/key size per head
    rot_dim: int                    # rotated query/key size
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot: RotarySpec
    window: Optional[int] = None    # keys seen, the token's own included
    kv_from: Optional[int] = None   # layer whose cached latents are used

    @property
    def cache_width(self) -> int:
        """Cached values per token (0: the layer owns no cache)."""
        return 0 if self.kv_from is not None else self.kv_rank + self.rot_dim


MixerSpec = Union[ChannelDeltaSpec, LatentAttentionSpec]


@dataclass(frozen=True)
class LayerSpec:
    mixer: MixerSpec
    ff: Optional[int] = None        # gated MLP size (None: no feed-forward)


@dataclass(frozen=True)
class LayeredConfig:
    """A decoder whose layers are listed one by one (tied embeddings)."""
    name: str
    architecture: str               # key of the registry's runner table
    vocab_size: int
    hidden_size: int
    layers: Tuple[LayerSpec, ...]
    rms_eps: float = 1e-6
    embed_scale: float = 1.0
    max_position: int = 8192
    vision_hidden: int = 0          # no multimodal tower
    weights_dir: str = ""           # checkpoint folder ("": random init)

    def __post_init__(self):
        for i, layer in enumerate(self.layers):
            m = layer.mixer
            if isinstance(m, ChannelDeltaSpec):
                if m.heads % m.kv_heads:
                    raise ValueError(f"layer {i}: heads {m.heads} is not a "
                                     f"multiple of kv_heads {m.kv_heads}")
                if m.conv < 1:
                    raise ValueError(f"layer {i}: conv must be at least 1")
                continue
            if m.rot.dims != m.rot_dim or m.rot_dim % 2:
                raise ValueError(f"layer {i}: rotation of {m.rot.dims} "
                                 f"dimensions on a part of {m.rot_dim}")
            if m.window is not None and m.window < 1:
                raise ValueError(f"layer {i}: window must be at least 1")
            if m.kv_from is None:
                continue
            if not 0 <= m.kv_from < i:
                raise ValueError(f"layer {i}: kv_from {m.kv_from} is not an "
                                 "earlier layer")
            src = self.layers[m.kv_from].mixer
            if not isinstance(src, LatentAttentionSpec) or \
                    src.kv_from is not None:
                raise ValueError(f"layer {i}: kv_from {m.kv_from} has no "
                                 "latent cache of its own")
            if (src.kv_rank, src.rot_dim, src.rot) != \
                    (m.kv_rank, m.rot_dim, m.rot):
                raise ValueError(f"layer {i}: latent sizes or rotation "
                                 f"differ from layer {m.kv_from}")

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def has_recurrent_state(self) -> bool:
        return any(isinstance(x.mixer, ChannelDeltaSpec)
                   for x in self.layers)

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return dtype_bytes * sum(
            x.mixer.cache_width for x in self.layers
            if isinstance(x.mixer, LatentAttentionSpec))

    def state_bytes_per_sequence(self, dtype_bytes: int = 2) -> int:
        total = 0
        for x in self.layers:
            if isinstance(x.mixer, ChannelDeltaSpec):
                (h, k, v), (c, t) = x.mixer.state_shapes
                total += h * k * v * 4 + c * t * dtype_bytes
        return total


def _rururax(name, vocab, width, ff, heads, kv_heads, dim, q_rank, kv_rank,
             window, pattern, rot_dim=64, lowrank=None, attn_heads=None,
             conv=4, max_position=8192):
    """A Rururax stack: `pattern` is a string of d (delta), a (attention) and
    s (attention sharing the latents of the last a)."""
    rot = RotarySpec(dims=rot_dim, base=500000.0, factor=8.0, original=8192)
    attn_heads = attn_heads or heads
    layers, own = [], None
    for i, kind in enumerate(pattern):
        if kind == "d":
            mixer = ChannelDeltaSpec(heads, kv_heads, dim, dim, conv,
                                     lowrank or dim, lowrank or dim)
        else:
            mixer = LatentAttentionSpec(
                attn_heads, dim, rot_dim, dim, q_rank, kv_rank,
                scale=(dim + rot_dim) ** -0.5, rot=rot, window=window,
                kv_from=own if kind == "s" else None)
            own = i if kind == "a" else own
        layers.append(LayerSpec(mixer, ff))
    return LayeredConfig(name, "Rururax", vocab, width, tuple(layers),
                         embed_scale=width ** 0.5, max_position=max_position)


# layer widths of the 8B class beside Llama-3-8B, and a small one for tests
RURURAX_8B = _rururax("rururax-8b", 128256, 4096, 14336, heads=32,
                      kv_heads=32, dim=128, q_rank=1536, kv_rank=512,
                      window=1024, pattern="ddda" * 4 + "ddds" * 4)
TINY_RURURAX = _rururax("tiny-rururax", 768, 80, 112, heads=6, kv_heads=3,
                        dim=20, q_rank=40, kv_rank=48, window=24,
                        pattern="dads", rot_dim=12, lowrank=10,
                        attn_heads=5, conv=3, max_position=1024)
