"""Hyper-parameters of the two models on the hot path, as plain dataclasses.

The defaults are the values the reference hard-codes for Mimi and Moshi-7B
(reference: moshi/moshi/models/loaders.py:38-88 `_seanet_kwargs`, `_quantizer_kwargs`,
`_transformer_kwargs`, `_mimi_config`; :90-119 `_lm_kwargs`).  Smaller instances of the same
architecture are used by the tests (oracle-sized).
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import List, Optional


@dataclass
class MimiConfig:
    sample_rate: int = 24000
    frame_rate: float = 12.5
    channels: int = 1
    dimension: int = 512
    n_filters: int = 64
    ratios: List[int] = field(default_factory=lambda: [8, 6, 5, 4])  # decoder order
    kernel_size: int = 7
    last_kernel_size: int = 3
    residual_kernel_size: int = 3
    compress: int = 2
    # encoder/decoder transformer
    tr_d_model: int = 512
    tr_num_heads: int = 8
    tr_num_layers: int = 8
    tr_dim_feedforward: int = 2048
    tr_context: int = 250
    tr_max_period: float = 10000.0
    tr_layer_scale: float = 0.01
    # split residual vector quantiser
    q_dimension: int = 256
    q_bins: int = 2048
    q_n_q: int = 32
    q_n_q_semantic: int = 1

    @property
    def hop_length(self) -> int:
        h = 1
        for r in self.ratios:
            h *= r
        return h

    @property
    def frame_size(self) -> int:
        return int(self.sample_rate / self.frame_rate)

    @property
    def encoder_frame_rate(self) -> float:
        return self.sample_rate / self.hop_length

    @property
    def resample_stride(self) -> int:
        s = self.encoder_frame_rate / self.frame_rate
        assert s == int(s), "only integer resampling strides are supported"
        return int(s)

    def reference_kwargs(self) -> dict:
        """The `mimi_config` dict the reference's `loaders.get_mimi` accepts (used only by the
        golden-vector generator, which imports the reference)."""
        seanet = {
            "channels": self.channels, "dimension": self.dimension, "causal": True,
            "n_filters": self.n_filters, "n_residual_layers": 1, "activation": "ELU",
            "compress": self.compress, "dilation_base": 2, "disable_norm_outer_blocks": 0,
            "kernel_size": self.kernel_size, "residual_kernel_size": self.residual_kernel_size,
            "last_kernel_size": self.last_kernel_size, "norm": "none", "pad_mode": "constant",
            "ratios": list(self.ratios), "true_skip": True,
        }
        quantizer = {
            "dimension": self.q_dimension, "n_q": self.q_n_q, "bins": self.q_bins,
            "input_dimension": self.dimension, "output_dimension": self.dimension,
        }
        transformer = {
            "d_model": self.tr_d_model, "num_heads": self.tr_num_heads, "num_layers": self.tr_num_layers,
            "causal": True, "layer_scale": self.tr_layer_scale, "context": self.tr_context,
            "conv_layout": True, "max_period": self.tr_max_period, "gating": "none", "norm": "layer_norm",
            "positional_embedding": "rope", "dim_feedforward": self.tr_dim_feedforward,
            "input_dimension": self.dimension, "output_dimensions": [self.dimension],
        }
        return {"sample_rate": self.sample_rate, "channels": self.channels, "frame_rate": self.frame_rate,
                "seanet": seanet, "quantizer": quantizer, "transformer": transformer}


def tiny_mimi_config() -> MimiConfig:
    """A Mimi small enough for the numpy oracle and the kernel simulator: same architecture, frame = 96 samples."""
    return MimiConfig(sample_rate=1200, frame_rate=12.5, dimension=32, n_filters=4, ratios=[4, 3, 2, 2],
                      tr_d_model=32, tr_num_heads=2, tr_num_layers=2, tr_dim_feedforward=64, tr_context=6,
                      q_dimension=16, q_bins=48, q_n_q=5, q_n_q_semantic=1)


@dataclass
class LMConfig:
    dim: int = 4096
    num_heads: int = 32
    num_layers: int = 32
    hidden_scale: float = 4.125
    context: int = 3000
    max_period: float = 10000.0
    n_q: int = 16
    dep_q: int = 8
    card: int = 2048
    text_card: int = 32000
    existing_text_padding_id: int = 3
    existing_text_end_padding_id: int = 0   # lm.py:100,123: what `LMModel.end_of_text_padding_id` returns (a checkpoint's lm_kwargs may set it)
    depformer_dim: int = 1024
    depformer_dim_feedforward: int = int(4.125 * 1024)
    depformer_num_heads: int = 16
    depformer_num_layers: int = 6
    delays: List[int] = field(default_factory=lambda: [0, 0, 1, 1, 1, 1, 1, 1, 1, 0, 1, 1, 1, 1, 1, 1, 1])
    extra_heads_num_heads: int = 0      # lm.py:101-102: linear heads on the transformer output (step_with_extra_heads)
    extra_heads_dim: int = 6
    kv_cache_dtype: str = "bf16"        # "fp8": e4m3 ring for the temporal transformer's keys / values (engine option)
    cross_attention: bool = False       # every temporal layer attends to the fuser's `cross` condition (transformer.py:727-731, 779-786)

    @staticmethod
    def _gating_hidden(dim: int, dim_feedforward: int) -> int:
        # reference: modules/gating.py:55-58
        if dim_feedforward == 4 * dim:
            return (21 * dim) // 8
        return (2 * dim_feedforward) // 3

    @property
    def ffn_hidden(self) -> int:
        return self._gating_hidden(self.dim, int(self.hidden_scale * self.dim))

    @property
    def depformer_ffn_hidden(self) -> int:
        return self._gating_hidden(self.depformer_dim, self.depformer_dim_feedforward)

    @property
    def num_codebooks(self) -> int:
        return self.n_q + 1

    @property
    def max_delay(self) -> int:
        return max(self.delays)

    def reference_kwargs(self) -> dict:
        """kwargs for the reference's `LMModel(...)` (golden generator only)."""
        return {
            "dim": self.dim, "text_card": self.text_card,
            "existing_text_padding_id": self.existing_text_padding_id, "n_q": self.n_q, "dep_q": self.dep_q,
            "card": self.card, "num_heads": self.num_heads, "num_layers": self.num_layers,
            "hidden_scale": self.hidden_scale, "causal": True, "layer_scale": None, "context": self.context,
            "max_period": self.max_period, "gating": "silu", "norm": "rms_norm_f32",
            "positional_embedding": "rope", "depformer_dim": self.depformer_dim,
            "depformer_dim_feedforward": self.depformer_dim_feedforward,
            "depformer_num_heads": self.depformer_num_heads, "depformer_num_layers": self.depformer_num_layers,
            "depformer_layer_scale": None, "depformer_multi_linear": True, "depformer_context": self.dep_q,
            "depformer_max_period": 10000, "depformer_gating": "silu", "depformer_pos_emb": "none",
            "depformer_weights_per_step": True, "delays": list(self.delays),
            **({"extra_heads_num_heads": self.extra_heads_num_heads, "extra_heads_dim": self.extra_heads_dim}
               if self.extra_heads_num_heads else {}),
            **({"cross_attention": True} if self.cross_attention else {}),
        }


def tiny_stt_config() -> LMConfig:
    """An ASR-style model at oracle size (the reference's kyutai/stt-* family): every audio codebook is input, no depformer
    (`dep_q = 0`, lm.py:218-221), the text stream runs `delays[0]` steps behind the audio, extra heads on the transformer
    output (lm.py:224-226) read with `step_with_extra_heads`."""
    return LMConfig(dim=128, num_heads=4, num_layers=2, hidden_scale=4.125, context=12, n_q=8, dep_q=0, card=64, text_card=96,
                    depformer_dim=64, depformer_dim_feedforward=int(4.125 * 64), depformer_num_heads=2, depformer_num_layers=2,
                    delays=[2] + [0] * 8, extra_heads_num_heads=2, extra_heads_dim=6)


def tiny_lm_config() -> LMConfig:
    """Same architecture as Moshi-7B at oracle size."""
    return LMConfig(dim=128, num_heads=4, num_layers=2, hidden_scale=4.125, context=12, n_q=16, dep_q=8, card=64,
                    text_card=96, depformer_dim=64, depformer_dim_feedforward=int(4.125 * 64),
                    depformer_num_heads=2, depformer_num_layers=2)


# --------------------------------------------------------------------------------------------------------------------
# token language models (libmoshi_tlm.so)
# --------------------------------------------------------------------------------------------------------------------
@dataclass
class LatentAttentionConfig:
    """Attention whose keys and values are projections of one cached latent, plus one rotated key part shared by the heads."""
    heads: int
    dim: int
    vdim: int
    rot_dim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float = 10000.0
    window: int = 0                     # keys seen, the position itself included; 0 = every earlier one


@dataclass
class MinGRUConfig:
    """Minimal GRU: an element-wise recurrence gated by projections of its input alone (nothing multiplies the state by a matrix)."""
    width: int


@dataclass
class GroupedAttentionConfig:
    """Softmax attention whose query heads share key/value heads (query head h reads key/value head h // (heads / kv_heads)), un-rotated."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int = 0                     # keys seen, the position itself included; 0 = every earlier one
    keep_first: int = 0                 # with a window: the sequence's first positions that stay visible behind it
    sink: bool = False                  # one is added to the softmax denominator: a sink of score 0 without a value


@dataclass
class ChannelDeltaConfig:
    """Gated delta rule with one decay per key channel: short causal convolutions in front of query, key and value, unit queries and keys,
    low-rank projections of the decay and of the output gate, an RMS norm per head behind it."""
    heads: int
    kv_heads: int                       # query/key heads; head h uses h // (heads / kv_heads)
    dim: int
    vdim: int
    conv: int                           # taps, the current token's included
    decay_rank: int
    gate_rank: int


@dataclass
class LightningConfig:
    """Linear attention with one constant decay per head, an RMS norm over all heads and an element-wise gate behind it."""
    heads: int
    dim: int
    vdim: int
    decay: List[float]                  # per head


@dataclass
class DenseGLUConfig:
    """Gated feed-forward.  clamped_swiglu: g = min(gate, limit), u = clamp(up, +-limit), g * sigmoid(1.702 g) * (u + 1)."""
    ff: int
    limit: float
    activation: str = "clamped_swiglu"


@dataclass
class BigramConfig:
    """Embedding of (previous token, token): row (previous * mul_prev + token * mul_cur) mod buckets; a sequence's first token takes row
    `buckets`."""
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass
class MoEConfig:
    """Experts chosen by a table over token ids."""
    experts: int
    top: int
    ff: int
    activation: str = "relu2"
    router: str = "token_table"


@dataclass
class TokenLayerConfig:
    mixer: object                       # LatentAttentionConfig | MinGRUConfig | GroupedAttentionConfig | ChannelDeltaConfig | LightningConfig
    mlp: object = None                  # MoEConfig | DenseGLUConfig | None


@dataclass
class TokenLMConfig:
    """A decoder-only network over token ids: parallel sublayers behind RMS norms of the same input (grouped; one per layer or one per
    sublayer), optional layer scales, and optionally a weight-tied repetition of layers [loop_start, loop_stop)."""
    architecture: str
    vocab: int
    width: int
    layers: List[TokenLayerConfig]
    norm_groups: int = 1
    norm_eps: float = 1e-6
    logit_scale: float = 1.0
    loop_start: int = 0
    loop_stop: int = 0                  # start == stop: nothing is repeated
    loop_times: int = 1
    # "add": the second and later passes start with x + embedding.  "project": every pass starts with a product of [x; embedding] and
    # a vector of the pass (tensors loop.in, loop.step)
    loop_inject: str = "add"
    norms: int = 1                      # 2: the feed-forward reads a norm of its own (norm2)
    layer_scales: bool = True           # ls1 / ls2 multiply what the sublayers add
    embed_scale: float = 1.0
    bigram: Optional[BigramConfig] = None
    max_positions: int = 0              # > 0: a learned vector per position (tensor pos) is added to the embedding, and bounds the length
    tied_head: bool = False             # logits from the (unscaled) embedding table instead of a head of their own

    @property
    def layer_runs(self) -> List[int]:
        """Layer index of every execution, in order."""
        n = list(range(len(self.layers)))
        if self.loop_stop <= self.loop_start:
            return n
        return n[:self.loop_start] + n[self.loop_start:self.loop_stop] * self.loop_times + n[self.loop_stop:]


def _known(d: dict, keys, what: str) -> dict:
    extra = sorted(k for k, v in d.items() if k not in keys and v is not None)
    if extra:
        raise ValueError(f"{what}: unknown entries {extra}")
    return d


def kesirax_config(raw: dict) -> TokenLMConfig:
    """config.json of a Kesirax model -> TokenLMConfig.  Sizes and constants come from the file; the structure (latent attention and
    minGRU mixers beside token-table experts with squared-ReLU activations) is the design's."""
    def mlp(m):
        if m is None:
            return None
        _known(m, ("kind", "expert", "router"), "mlp")
        if m.get("kind", "moe") != "moe":
            raise ValueError(f"mlp kind {m['kind']!r} is not part of this design")
        return MoEConfig(experts=int(m["router"]["experts"]), top=int(m["router"]["top"]), ff=int(m["expert"]["ff"]))

    def mixer(kind, m):
        if kind == "mingru":
            return MinGRUConfig(width=int(m["width"]))
        if kind == "latent_attention":
            rot = m.get("rot") or {}
            if rot and int(rot["dims"]) != int(m["rot_dim"]):
                raise ValueError("latent attention rotates its whole rotated part: rot.dims must equal rot_dim")
            return LatentAttentionConfig(
                heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), rot_dim=int(m["rot_dim"]), q_rank=int(m["q_rank"]),
                kv_rank=int(m["kv_rank"]), scale=float(m["scale"]), rot_base=float(rot.get("base", 10000.0)),
                window=int((m.get("mask") or {}).get("size", 0)))
        raise ValueError(f"mixer type {kind!r} is not part of this design")

    layers = [TokenLayerConfig(mixer(l["type"], l["mixer"]), mlp(l.get("mlp"))) for l in raw["layers"]]
    norm, loop = raw["norm"], raw.get("loop") or {}
    return TokenLMConfig(
        architecture=raw["architecture"], vocab=int(raw["vocab"]), width=int(raw["width"]), layers=layers, norm_groups=int(norm.get("groups", 1)),
        norm_eps=float(norm["eps"]), logit_scale=float(raw.get("logit_scale", 1.0)), loop_start=int(loop.get("start", 0)),
        loop_stop=int(loop.get("stop", 0)), loop_times=int(loop.get("times", 1)))


def bibapel_config(raw: dict, shapes: Optional[dict] = None) -> TokenLMConfig:
    """config.json of a Bibapel model -> TokenLMConfig.  `shapes` (tensor name -> shape) gives the ranks of the low-rank projections, which
    the file does not name; without it (random weights) they are the sizes of one head."""
    def rank(i, name, default):
        return int(shapes[f"l{i}.mix.{name}"][0]) if shapes is not None and f"l{i}.mix.{name}" in shapes else default

    def mlp(m):
        if m is None:
            return None
        _known(m, ("kind", "ff", "limit"), "mlp")
        if m.get("kind", "dense") != "dense":
            raise ValueError(f"mlp kind {m['kind']!r} is not part of this design")
        return DenseGLUConfig(ff=int(m["ff"]), limit=float(m["limit"]))

    def mixer(i, kind, m):
        heads, dim, vdim = int(m["heads"]), int(m["dim"]), int(m["vdim"])
        if kind == "attention":
            _known(m, ("heads", "kv_heads", "dim", "vdim", "scale", "mask"), "attention")
            mask = m.get("mask") or {}
            _known(mask, ("size", "keep_first"), "mask")
            return GroupedAttentionConfig(heads=heads, kv_heads=int(m.get("kv_heads", heads)), dim=dim, vdim=vdim, scale=float(m["scale"]),
                                          window=int(mask.get("size", 0)), keep_first=int(mask.get("keep_first", 0)), sink=True)
        if kind == "channel_delta":
            _known(m, ("heads", "kv_heads", "dim", "vdim", "conv"), "channel_delta")
            return ChannelDeltaConfig(heads=heads, kv_heads=int(m.get("kv_heads", heads)), dim=dim, vdim=vdim, conv=int(m["conv"]),
                                      decay_rank=rank(i, "a1", dim), gate_rank=rank(i, "g1", vdim))
        if kind == "lightning":
            _known(m, ("heads", "dim", "vdim", "decay"), "lightning")
            decay = m["decay"] if isinstance(m["decay"], list) else [m["decay"]] * heads
            if len(decay) != heads:
                raise ValueError("lightning: one decay per head")
            return LightningConfig(heads=heads, dim=dim, vdim=vdim, decay=[float(d) for d in decay])
        raise ValueError(f"mixer type {kind!r} is not part of this design")

    emb, loop = raw.get("embedding") or {}, raw.get("loop") or {}
    _known(emb, ("scale", "bigram"), "embedding")
    _known(raw["norm"], ("eps",), "norm")
    _known(loop, ("start", "stop", "times"), "loop")
    big = emb.get("bigram")
    return TokenLMConfig(
        architecture=raw["architecture"], vocab=int(raw["vocab"]), width=int(raw["width"]),
        layers=[TokenLayerConfig(mixer(i, l["type"], l["mixer"]), mlp(l.get("mlp"))) for i, l in enumerate(raw["layers"])],
        norm_eps=float(raw["norm"]["eps"]), loop_start=int(loop.get("start", 0)), loop_stop=int(loop.get("stop", 0)),
        loop_times=int(loop.get("times", 1)), loop_inject="project", norms=2, layer_scales=False, embed_scale=float(emb.get("scale", 1.0)),
        bigram=BigramConfig(int(big["buckets"]), int(big["mul_prev"]), int(big["mul_cur"])) if big else None,
        max_positions=int(raw.get("max_positions", 0)), tied_head=True)


# config.json `architecture` -> parser (config, tensor shapes); the registry `loaders.get_token_lm` and the command lines choose a model
# class by
TOKEN_LM_ARCHITECTURES = {"Kesirax": lambda raw, shapes=None: kesirax_config(raw), "Bibapel": bibapel_config}


def tiny_token_lm_config() -> TokenLMConfig:
    """A Kesirax network at oracle size, with sizes that are no multiples of the kernels' tiles."""
    att = LatentAttentionConfig(heads=3, dim=24, vdim=20, rot_dim=12, q_rank=40, kv_rank=36, scale=0.17, rot_base=5000.0, window=37)
    moe = MoEConfig(experts=5, top=2, ff=44)
    return TokenLMConfig("Kesirax", vocab=101, width=96, norm_groups=3, norm_eps=1e-5, logit_scale=0.7, loop_start=1, loop_stop=3, loop_times=2,
                         layers=[TokenLayerConfig(MinGRUConfig(72), moe), TokenLayerConfig(att, moe), TokenLayerConfig(MinGRUConfig(72), None),
                                 TokenLayerConfig(att, MoEConfig(experts=4, top=1, ff=52))])


def tiny_bibapel_config() -> TokenLMConfig:
    """A Bibapel network at oracle size, with sizes that are no multiples of the kernels' tiles."""
    delta = ChannelDeltaConfig(heads=4, kv_heads=2, dim=20, vdim=24, conv=3, decay_rank=10, gate_rank=14)
    att = GroupedAttentionConfig(heads=6, kv_heads=2, dim=24, vdim=20, scale=0.21, window=41, keep_first=5, sink=True)
    light = LightningConfig(heads=3, dim=18, vdim=28, decay=[0.7, 0.93, 0.995])
    glu = DenseGLUConfig(ff=72, limit=1.5)
    return TokenLMConfig("Bibapel", vocab=97, width=80, norm_eps=1e-5, loop_start=1, loop_stop=3, loop_times=2, loop_inject="project", norms=2,
                         layer_scales=False, embed_scale=0.8, bigram=BigramConfig(buckets=37, mul_prev=11, mul_cur=5), max_positions=1500, tied_head=True,
                         layers=[TokenLayerConfig(light, glu), TokenLayerConfig(delta, glu), TokenLayerConfig(att, DenseGLUConfig(ff=56, limit=0.9)),
                                 TokenLayerConfig(delta, None)])
