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
    def cache_width(self) -> int:
        """Cached values per token: none, the state has a fixed size."""
        return 0

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

    def page_shape(self, block_size: int) -> Tuple[int, ...]:
        return block_size, self.cache_width


@dataclass(frozen=True)
class GroupedAttentionSpec:
    """Causal attention, query heads in groups that share a key/value head;
    positions do not enter the scores."""
    heads: int
    kv_heads: int
    dim: int                        # query/key size per head
    vdim: int
    scale: float
    sink: Optional[float] = None    # score of an extra key without a value

    @property
    def cache_width(self) -> int:
        return self.kv_heads * (self.dim + self.vdim)

    def page_shape(self, block_size: int) -> Tuple[int, ...]:
        """A head's tokens of a page lie together, rows [key | value]."""
        return self.kv_heads, block_size, self.dim + self.vdim


MixerSpec = Union[ChannelDeltaSpec, LatentAttentionSpec, GroupedAttentionSpec]


@dataclass(frozen=True)
class GatedSpec:
    """Feed-forward down(act(gate h) * up h)."""
    ff: int
    act: str = "gelu_tanh"


@dataclass(frozen=True)
class ExpertsSpec:
    """Feed-forward of experts down(act(up h)). A token goes to the `top`
    experts with the largest scores sigmoid(router h); the score multiplies
    the expert's input. A shared expert takes every token."""
    experts: int
    top: int
    ff: int                         # inner size of one expert
    shared_ff: Optional[int] = None     # of the shared one (None: has none)
    act: str = "relu_squared"


FeedForwardSpec = Union[GatedSpec, ExpertsSpec]


@dataclass(frozen=True)
class LayerSpec:
    mixer: MixerSpec
    ff: Optional[FeedForwardSpec] = None    # None: no feed-forward


@dataclass(frozen=True)
class LoopSpec:
    """Layers start .. stop-1 run `times` times in a row with the same
    weights. Ahead of each pass the stream is mixed with the embedding output
    and gets a vector of that pass."""
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class LayerRun:
    """One run of a layer in the order of the forward pass."""
    layer: int
    cache: int                      # run whose cache or state it uses
    enters: Optional[int] = None    # number of the loop pass it begins


@dataclass(frozen=True)
class LayeredConfig:
    """A decoder whose layers are listed one by one (tied embeddings)."""
    name: str
    architecture: str               # key of the registry's runner table
    vocab_size: int
    hidden_size: int
    layers: Tuple[LayerSpec, ...]
    rms_eps: float = 1e-6
    norm_offset: float = 0.0        # added to the weights of stream norms
    post_norms: bool = False        # sublayer outputs are normed as well
    embed_scale: float = 1.0
    max_position: int = 8192
    learned_positions: bool = False     # a vector per position is embedded
    loop: Optional[LoopSpec] = None
    vision_hidden: int = 0          # no multimodal tower
    weights_dir: str = ""           # checkpoint folder ("": random init)

    def __post_init__(self):
        if self.loop is not None:
            lp = self.loop
            if not 0 <= lp.start < lp.stop <= len(self.layers) or \
                    lp.times < 1:
                raise ValueError(f"loop {lp.start}..{lp.stop} x {lp.times} "
                                 f"over {len(self.layers)} layers")
        for i, layer in enumerate(self.layers):
            m, ff = layer.mixer, layer.ff
            if isinstance(ff, ExpertsSpec) and not 0 < ff.top <= ff.experts:
                raise ValueError(f"layer {i}: top {ff.top} of {ff.experts} "
                                 "experts")
            if isinstance(m, GroupedAttentionSpec):
                if m.heads % m.kv_heads:
                    raise ValueError(f"layer {i}: heads {m.heads} is not a "
                                     f"multiple of kv_heads {m.kv_heads}")
                continue
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
    def runs(self) -> Tuple[LayerRun, ...]:
        """Layers in the order they run; every run has its own cache or
        state, or shares that of the latest run of the layer it names."""
        n = len(self.layers)
        lp = self.loop or LoopSpec(n, n, 0)
        order = [(i, None) for i in range(lp.start)]
        for t in range(lp.times):
            order += [(i, t if i == lp.start else None)
                      for i in range(lp.start, lp.stop)]
        order += [(i, None) for i in range(lp.stop, n)]
        runs, latest = [], {}
        for r, (i, enters) in enumerate(order):
            latest[i] = r
            source = getattr(self.layers[i].mixer, "kv_from", None)
            runs.append(LayerRun(i, r if source is None else latest[source],
                                 enters))
        return tuple(runs)

    @property
    def has_recurrent_state(self) -> bool:
        return any(isinstance(x.mixer, ChannelDeltaSpec)
                   for x in self.layers)

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return dtype_bytes * sum(self.layers[r.layer].mixer.cache_width
                                 for r in self.runs)

    def state_bytes_per_sequence(self, dtype_bytes: int = 2) -> int:
        total = 0
        for r in self.runs:
            m = self.layers[r.layer].mixer
            if isinstance(m, ChannelDeltaSpec):
                (h, k, v), (c, t) = m.state_shapes
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
        layers.append(LayerSpec(mixer, GatedSpec(ff)))
    return LayeredConfig(name, "Rururax", vocab, width, tuple(layers),
                         norm_offset=1.0, post_norms=True,
                         embed_scale=width ** 0.5, max_position=max_position)


# layer widths of the 8B class beside Llama-3-8B, and a small one for tests
RURURAX_8B = _rururax("rururax-8b", 128256, 4096, 14336, heads=32,
                      kv_heads=32, dim=128, q_rank=1536, kv_rank=512,
                      window=1024, pattern="ddda" * 4 + "ddds" * 4)
TINY_RURURAX = _rururax("tiny-rururax", 768, 80, 112, heads=6, kv_heads=3,
                        dim=20, q_rank=40, kv_rank=48, window=24,
                        pattern="dads", rot_dim=12, lowrank=10,
                        attn_heads=5, conv=3, max_position=1024)


def _sezazen(name, vocab, width, heads, kv_heads, dim, vdim, ff, experts, top,
             expert_ff, shared_ff, pattern, loop=None, max_position=8192):
    """A Sezazen stack: `pattern` is a string of d (dense feed-forward), e
    (experts) and n (no feed-forward); loop = (start, stop, times)."""
    mixer = GroupedAttentionSpec(heads, kv_heads, dim, vdim,
                                 scale=dim ** -0.5, sink=0.0)
    kinds = {"d": GatedSpec(ff, "silu"), "n": None,
             "e": ExpertsSpec(experts, top, expert_ff, shared_ff)}
    return LayeredConfig(name, "Sezazen", vocab, width,
                         tuple(LayerSpec(mixer, kinds[k]) for k in pattern),
                         learned_positions=True, max_position=max_position,
                         loop=LoopSpec(*loop) if loop else None)


# an 8B-class stack (about 6B of its weights run per token and pass), and a
# small one for tests
SEZAZEN_8B = _sezazen("sezazen-8b", 128256, 4096, heads=32, kv_heads=8,
                      dim=128, vdim=128, ff=14336, experts=32, top=4,
                      expert_ff=3584, shared_ff=7168,
                      pattern="d" + "e" * 15, loop=(4, 12, 2))
TINY_SEZAZEN = _sezazen("tiny-sezazen", 768, 72, heads=6, kv_heads=2, dim=20,
                        vdim=28, ff=104, experts=6, top=2, expert_ff=24,
                        shared_ff=40, pattern="edne", loop=(1, 3, 2),
                        max_position=1024)
