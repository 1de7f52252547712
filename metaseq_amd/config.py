"""Flat model configuration with the attribute names the reference's decoder reads from
its args namespace (metaseq/models/transformer_decoder.py:73-117,
metaseq/modules/transformer_decoder_layer.py:44-98), and the OPT size table
(metaseq/launcher/opt_job_constants.py:32-45).  Below them: configurations of hybrid decoders,
whose layers each choose their own mixer and feed-forward."""
import logging
from dataclasses import MISSING, dataclass, fields, replace
from typing import List, Optional, Union

logger = logging.getLogger(__name__)

# head sizes the attention kernels are instantiated for (lanes per key row = head_dim / 8)
SUPPORTED_HEAD_DIMS = (64, 128)


@dataclass
class OPTConfig:
    decoder_layers: int
    decoder_embed_dim: int
    decoder_attention_heads: int
    decoder_ffn_embed_dim: int = 0
    vocab_size: int = 50272  # 50265 tokenizer entries padded to a multiple of 8
    max_target_positions: int = 2048
    padding_idx: int = 1
    eos_idx: int = 2
    activation_fn: str = "relu"
    share_decoder_input_output_embed: bool = True
    decoder_learned_pos: bool = True
    no_scale_embedding: bool = True
    quantize_int8: bool = False  # int8 weight-only for qkv / out_proj / fc1 / fc2

    def __post_init__(self):
        if not self.decoder_ffn_embed_dim:
            self.decoder_ffn_embed_dim = 4 * self.decoder_embed_dim
        if self.decoder_embed_dim % self.decoder_attention_heads:
            raise ValueError("decoder_embed_dim must be divisible by decoder_attention_heads")
        if self.activation_fn != "relu":
            raise NotImplementedError("only --activation-fn relu (OPT) is implemented")
        if not (self.share_decoder_input_output_embed and self.decoder_learned_pos
                and self.no_scale_embedding):
            raise NotImplementedError(
                "only the OPT setup (tied embeddings, learned positions, no embedding scale) "
                "is implemented")

    @property
    def head_dim(self):
        return self.decoder_embed_dim // self.decoder_attention_heads

    def require_supported_head_dim(self):
        """Raised when a decoder is built, before any weight is allocated or packed."""
        if self.head_dim not in SUPPORTED_HEAD_DIMS:
            raise NotImplementedError(
                "head_dim %d (decoder_embed_dim %d / %d heads) is not supported: the attention "
                "kernels are built for head_dim %s" % (
                    self.head_dim, self.decoder_embed_dim, self.decoder_attention_heads,
                    " or ".join(str(h) for h in SUPPORTED_HEAD_DIMS)))


# name -> (layers, embed dim, heads).  OPT-2.7B (32 layers, 2560 / 32 heads = head_dim 80) is
# left out: no attention kernel is built for that head size.
_OPT_SIZES = {
    "125m": (12, 768, 12),
    "350m": (24, 1024, 16),
    "1.3b": (24, 2048, 32),
    "6.7b": (32, 4096, 32),
    "13b": (40, 5120, 40),
    "30b": (48, 7168, 56),
    "66b": (64, 9216, 72),
    "175b": (96, 12288, 96),
}


def opt_config(name: str, **overrides) -> OPTConfig:
    layers, dim, heads = _OPT_SIZES[name.lower()]
    return replace(OPTConfig(layers, dim, heads), **overrides)


def config_from_state_dict(state, heads: int = 0, **overrides) -> OPTConfig:
    """The configuration a reference-named state dict (fp16, or quantised offline) implies:
    layers, widths, vocabulary and position count are read off the tensor shapes.  The number
    of heads is in no shape; it is taken from the OPT size table by (layers, width) unless
    given.  For checkpoints whose own "cfg" entry cannot be read by a loader that executes
    nothing (metaseq/checkpoint_utils.py:540-557 pickles an arbitrary namespace there)."""
    def shape(name):
        for k in (name, "decoder." + name):
            if k in state:
                return tuple(state[k].shape)
        raise KeyError("state dict has no %r" % name)

    layers = 1 + max(int(k.split("layers.")[1].split(".")[0]) for k in state if "layers." in k)
    vocab, dim = shape("embed_tokens.weight")
    positions = shape("embed_positions.weight")[0]
    try:
        ffn = shape("layers.0.fc1.weight")[0]
    except KeyError:
        ffn = shape("layers.0.fc1.qweight")[0]
    if not heads:
        known = {(l, d): h for l, d, h in _OPT_SIZES.values()}
        if (layers, dim) not in known:
            raise ValueError("%d layers of width %d are no OPT size: pass heads=" % (layers, dim))
        heads = known[(layers, dim)]
    padding_idx = overrides.pop("padding_idx", 1)
    # the learned positional table holds padding_idx + 1 unused leading rows
    # (metaseq/modules/learned_positional_embedding.py:23-28)
    cfg = OPTConfig(layers, dim, heads, decoder_ffn_embed_dim=ffn, vocab_size=vocab,
                    max_target_positions=positions - padding_idx - 1, padding_idx=padding_idx)
    return replace(cfg, **overrides)


# ---------------------------------------------------------------- hybrid decoders
@dataclass
class LatentAttentionSpec:
    """Attention over a cached latent vector per position: per-head keys and values are linear
    images of it.  ``kv_from``: the layer whose latents are used instead of own ones."""
    heads: int
    dim: int          # query / key size per head
    vdim: int         # value size per head
    kv_rank: int
    q_rank: int
    scale: float
    kv_from: Optional[int] = None


@dataclass
class RGLRUSpec:
    """Gated linear recurrent unit behind a short causal convolution; the gates are
    block-diagonal."""
    width: int
    blocks: int
    conv: int         # taps


@dataclass
class DeltaSpec:
    """Gated delta rule with one decay per head."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int


@dataclass
class ChannelDeltaSpec(DeltaSpec):
    """Gated delta rule with one decay per head and key channel; decays and the read-out's gate
    come from low-rank projections, whose ranks the weights' shapes give."""
    decay_rank: Optional[int] = None
    gate_rank: Optional[int] = None


@dataclass
class GroupedAttentionSpec:
    """Attention of ``heads`` query heads over ``kv_heads`` cached keys and values, rotary on the
    first ``rot_dims`` dimensions, within chunks of ``chunk`` positions (None: no chunks), with a
    gate per head."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float = 1.0
    rot_dims: int = 0
    chunk: Optional[int] = None


@dataclass
class ParallelSpec:
    """Two mixers over the same input; the mean of their normed outputs."""
    left: GroupedAttentionSpec
    right: ChannelDeltaSpec


@dataclass
class DenseSpec:
    """Gated feed-forward: gelu_tanh(gate) up."""
    ff: int


@dataclass
class SquaredReluSpec:
    """Feed-forward with biases whose activation is the square of relu."""
    ff: int


@dataclass
class ExpertSpec:
    ff: int
    limit: float


@dataclass
class RouterSpec:
    experts: int
    top: int
    scale: float = 1.0
    groups: int = 1   # experts form this many equal groups,
    keep: int = 1     # of which the best ``keep`` are eligible


@dataclass
class MoESpec:
    router: RouterSpec
    expert: ExpertSpec
    shared: Optional[ExpertSpec] = None


@dataclass
class HybridLayerSpec:
    mixer: Union[LatentAttentionSpec, RGLRUSpec, DeltaSpec, ParallelSpec]
    mlp: Union[DenseSpec, SquaredReluSpec, MoESpec, None] = None


@dataclass
class LoopSpec:
    """Layers ``start`` .. ``stop`` - 1 run ``times`` times in a row with the same weights."""
    start: int
    stop: int
    times: int


def _take(section, where, spec, rename=None, **extra):
    """Builds ``spec`` from a dictionary of a config.json; keys nobody reads are reported."""
    section = dict(section)
    values = {}
    for f in fields(spec):
        key = (rename or {}).get(f.name, f.name)
        if f.name in extra:
            values[f.name] = extra[f.name]
        elif section.get(key) is not None:
            values[f.name] = section[key]
        elif f.default is MISSING:
            raise ValueError("config.json: %s lacks %r" % (where, key))
        section.pop(key, None)
    unused = sorted(set(section) - set(extra))
    if unused:
        logger.warning("config.json: %s: unknown keys %s are ignored", where, ", ".join(unused))
    return spec(**values)


@dataclass
class HybridConfig:
    """A decoder whose layers each choose a mixer and a feed-forward, with RMS norms before every
    sublayer.  ``post_norms``: norms after them too; ``sinusoidal``: fixed positions added to the
    embedding; ``tied``: the vocabulary projection is the embedding table; ``loop``: a range of
    layers that runs several times, each pass with a cache of its own."""
    width: int
    vocab_size: int
    layers: List[HybridLayerSpec]
    norm_eps: float = 1e-6
    embed_scale: float = 1.0
    max_target_positions: int = 1 << 17
    padding_idx: int = 1
    eos_idx: int = 2
    post_norms: bool = True
    sinusoidal: bool = True
    tied: bool = False
    loop: Optional[LoopSpec] = None

    def __post_init__(self):
        if not self.layers:
            raise ValueError("a hybrid decoder needs at least one layer")
        k = self.loop
        if k is not None and not (0 <= k.start < k.stop <= len(self.layers) and k.times >= 1):
            raise ValueError("a loop of layers %d .. %d, %d times, in a model of %d layers"
                             % (k.start, k.stop - 1, k.times, len(self.layers)))
        for i, layer in enumerate(self.layers):
            m = layer.mixer
            if isinstance(m, LatentAttentionSpec) and m.kv_from is not None:
                j = m.kv_from
                src = self.layers[j].mixer if 0 <= j < i else None
                if not isinstance(src, LatentAttentionSpec) or src.kv_from is not None:
                    raise ValueError("layer %d takes its latents from layer %s, which owns none"
                                     % (i, j))
                if src.kv_rank != m.kv_rank:
                    raise ValueError("layer %d and the layer it takes its latents from differ in "
                                     "kv_rank" % i)
            for part in (m.left, m.right) if isinstance(m, ParallelSpec) else (m,):
                if isinstance(part, (DeltaSpec, GroupedAttentionSpec)) \
                        and part.heads % part.kv_heads:
                    raise ValueError("layer %d: heads must be a multiple of kv_heads" % i)
            if isinstance(m, ParallelSpec):
                t = m.left
                if t.rot_dims % 2 or not 0 <= t.rot_dims <= t.dim:
                    raise ValueError("layer %d: rotary positions on %d of %d dimensions"
                                     % (i, t.rot_dims, t.dim))
                if t.chunk is not None and t.chunk < 1:
                    raise ValueError("layer %d: chunks of %d positions" % (i, t.chunk))
            if isinstance(m, RGLRUSpec) and m.width % m.blocks:
                raise ValueError("layer %d: width must be a multiple of blocks" % i)
            if isinstance(layer.mlp, MoESpec):
                r = layer.mlp.router
                if r.experts % r.groups or not 1 <= r.keep <= r.groups \
                        or r.top > r.experts // r.groups * r.keep:
                    raise ValueError("layer %d: %d experts in %d groups, %d kept, top %d"
                                     % (i, r.experts, r.groups, r.keep, r.top))

    def runs(self):
        """(layer, pass) in the order of execution; pass t >= 0 marks the run that begins pass t
        of the loop, -1 every other run."""
        k, n = self.loop, len(self.layers)
        if k is None:
            return [(i, -1) for i in range(n)]
        return ([(i, -1) for i in range(k.start)]
                + [(i, t if i == k.start else -1) for t in range(k.times)
                   for i in range(k.start, k.stop)]
                + [(i, -1) for i in range(k.stop, n)])

    # what a config.json's "architecture" fixes: its layer types, its dense feed-forward, and the
    # flags of the class
    DESIGNS = {
        "Sinulorn": dict(mixers=("latent_attention", "rglru", "delta"), dense=DenseSpec),
        "Nomalorn": dict(mixers=("parallel",), dense=SquaredReluSpec, post_norms=False,
                         sinusoidal=False, tied=True),
    }
    MIXERS = {"latent_attention": LatentAttentionSpec, "rglru": RGLRUSpec, "delta": DeltaSpec,
              "parallel": ParallelSpec}

    @classmethod
    def from_json(cls, obj):
        """The configuration of a config.json (already parsed)."""
        design = dict(cls.DESIGNS[obj.get("architecture", "Sinulorn")])
        mixers, dense = design.pop("mixers"), design.pop("dense")
        layers = []
        for i, entry in enumerate(obj["layers"]):
            where = "layer %d" % i
            kind = entry["type"]
            if kind not in mixers:
                raise NotImplementedError("config.json: %s: unknown mixer %r" % (where, kind))
            if kind == "parallel":
                mixer = cls._parallel(dict(entry["mixer"]), where + " mixer")
            else:
                mixer = _take(entry["mixer"], where + " mixer", cls.MIXERS[kind])
            mlp = entry.get("mlp")
            if mlp is not None:
                mlp = cls._mlp(dict(mlp), where + " mlp", dense)
            layers.append(HybridLayerSpec(mixer, mlp))
        special = {k: obj[k] for k in ("padding_idx", "eos_idx", "max_target_positions")
                   if k in obj}
        if obj.get("loop"):
            special["loop"] = _take(obj["loop"], "loop", LoopSpec)
        return cls(width=obj["width"], vocab_size=obj["vocab"], layers=layers,
                   norm_eps=obj["norm"]["eps"],
                   embed_scale=(obj.get("embedding") or {}).get("scale", 1.0), **special, **design)

    @staticmethod
    def _parallel(mixer, where):
        left, right = dict(mixer.pop("left")), dict(mixer.pop("right"))
        if mixer:
            logger.warning("config.json: %s: unknown keys %s are ignored", where,
                           ", ".join(sorted(mixer)))
        rot, mask = left.pop("rot", None) or {}, left.pop("mask", None) or {}
        for section, known, name in ((rot, {"base", "dims"}, "rot"), (mask, {"size"}, "mask")):
            if set(section) - known:
                logger.warning("config.json: %s left %s: unknown keys %s are ignored", where, name,
                               ", ".join(sorted(set(section) - known)))
        return ParallelSpec(
            _take(left, where + " left", GroupedAttentionSpec, rot_base=rot.get("base", 1.0),
                  rot_dims=rot.get("dims", 0), chunk=mask.get("size")),
            _take(right, where + " right", ChannelDeltaSpec))

    def with_shapes(self, shapes):
        """The configuration completed by what only the weights' shapes (name -> shape) say."""
        layers = []
        for i, layer in enumerate(self.layers):
            m = layer.mixer
            if isinstance(m, ParallelSpec):
                ranks = {}
                for field, name in (("decay_rank", "a1"), ("gate_rank", "g1")):
                    shape = shapes.get("l%d.mix.right.%s" % (i, name))
                    if getattr(m.right, field) is None and shape is not None:
                        ranks[field] = int(shape[0])
                if ranks:
                    layer = replace(layer, mixer=replace(m, right=replace(m.right, **ranks)))
            layers.append(layer)
        return replace(self, layers=layers)

    @staticmethod
    def _mlp(mlp, where, dense=DenseSpec):
        kind = mlp.pop("kind")
        if kind == "dense":
            return _take(mlp, where, dense)
        if kind != "moe":
            raise NotImplementedError("config.json: %s: unknown kind %r" % (where, kind))
        router = dict(mlp.pop("router"))
        groups = router.pop("groups", None) or {"count": 1, "keep": 1}
        expert, shared = mlp.pop("expert"), mlp.pop("shared", None)
        if mlp:
            logger.warning("config.json: %s: unknown keys %s are ignored", where,
                           ", ".join(sorted(mlp)))
        return MoESpec(
            _take(router, where + " router", RouterSpec, groups=groups["count"],
                  keep=groups["keep"]),
            _take(expert, where + " expert", ExpertSpec),
            _take(shared, where + " shared expert", ExpertSpec) if shared else None)

    def tensor_shapes(self):
        """name -> shape of every tensor of a checkpoint of this model."""
        D, out = self.width, {}
        out["embed"] = (self.vocab_size, D)
        if self.loop is not None:
            out["loop.step"] = (self.loop.times, D)
        for i, layer in enumerate(self.layers):
            pre, m = "l%d." % i, layer.mixer
            for n in self.norm_names(layer):
                out[pre + n] = (D,)

            def put(section, **shapes):
                for name, shape in shapes.items():
                    out[pre + section + "." + name.replace("_dot_", ".")] = shape

            if isinstance(m, LatentAttentionSpec):
                put("mix", dq=(m.q_rank, D), dq_dot_norm=(m.q_rank,),
                    uq=(m.heads * m.dim, m.q_rank), uk=(m.heads * m.dim, m.kv_rank),
                    uv=(m.heads * m.vdim, m.kv_rank), o=(D, m.heads * m.vdim))
                if m.kv_from is None:
                    put("mix", dkv=(m.kv_rank, D), dkv_dot_norm=(m.kv_rank,))
            elif isinstance(m, RGLRUSpec):
                W, nb, bs = m.width, m.blocks, m.width // m.blocks
                put("mix", y=(W, D), y_dot_b=(W,), x=(W, D), x_dot_b=(W,), conv=(W, m.conv),
                    conv_dot_b=(W,), ra=(nb, bs, bs), ra_dot_b=(nb, bs), ri=(nb, bs, bs),
                    ri_dot_b=(nb, bs), lam=(W,), o=(D, W))
            elif isinstance(m, ParallelSpec):
                a, d = m.left, m.right
                put("mix.left", q=(a.heads * a.dim, D), q_dot_b=(a.heads * a.dim,),
                    k=(a.kv_heads * a.dim, D), k_dot_b=(a.kv_heads * a.dim,),
                    v=(a.kv_heads * a.vdim, D), v_dot_b=(a.kv_heads * a.vdim,), g=(a.heads, D),
                    o=(D, a.heads * a.vdim))
                qk, v = d.kv_heads * d.dim, d.heads * d.vdim
                put("mix.right", q=(qk, D), q_dot_conv=(qk, d.conv), k=(qk, D),
                    k_dot_conv=(qk, d.conv), v=(v, D), v_dot_conv=(v, d.conv), b=(d.heads, D),
                    A_log=(d.heads,), norm=(d.vdim,), a1=(d.decay_rank, D),
                    a2=(d.heads * d.dim, d.decay_rank), dt_bias=(d.heads * d.dim,),
                    g1=(d.gate_rank, D), g2=(v, d.gate_rank), o=(D, v))
                put("mix", left_dot_out=(D,), right_dot_out=(D,))
            else:
                qk, v = m.kv_heads * m.dim, m.heads * m.vdim
                put("mix", q=(qk, D), q_dot_conv=(qk, m.conv), k=(qk, D), k_dot_conv=(qk, m.conv),
                    v=(v, D), v_dot_conv=(v, m.conv), b=(m.heads, D), a=(m.heads, D),
                    A_log=(m.heads,), dt_bias=(m.heads,), norm=(m.vdim,), g=(v, D), o=(D, v))
            if isinstance(layer.mlp, DenseSpec):
                F = layer.mlp.ff
                put("mlp", gate=(F, D), up=(F, D), down=(D, F))
            elif isinstance(layer.mlp, SquaredReluSpec):
                F = layer.mlp.ff
                put("mlp", up=(F, D), up_dot_b=(F,), down=(D, F), down_dot_b=(D,))
            elif layer.mlp is not None:
                r, e, s = layer.mlp.router, layer.mlp.expert, layer.mlp.shared
                put("mlp", router=(r.experts, D))
                for x in range(r.experts):
                    put("mlp.e%d" % x, gate=(e.ff, D), up=(e.ff, D), down=(D, e.ff))
                if s is not None:
                    put("mlp.shared", gate=(s.ff, D), up=(s.ff, D), down=(D, s.ff), sg=(1, D))
        out["final.norm"] = (D,)
        if not self.tied:
            out["head"] = (self.vocab_size, D)
        return out

    def norm_names(self, layer):
        """The norms over the width that a layer has."""
        names = ("norm1", "norm1b") + (("norm2", "norm2b") if layer.mlp else ())
        return names if self.post_norms else tuple(n for n in names if not n.endswith("b"))
