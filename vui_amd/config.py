"""Model configuration.  Field names and defaults mirror the reference's pydantic schema
(src/vui/config.py:16-76) so a checkpoint's `config` dict can be passed through unchanged;
plain dataclasses are used, unknown keys are ignored like the reference's extra="ignore"."""
from __future__ import annotations

from dataclasses import dataclass, field, fields


def _from_dict(cls, d: dict):
    names = {f.name for f in fields(cls)}
    return cls(**{k: v for k, v in (d or {}).items() if k in names})


@dataclass
class VuiConfig:
    # Architecture
    d_model: int = 512
    n_layers: int = 6
    n_heads: int = 8
    n_kv_heads: int | None = None
    intermediate_size: int | None = None
    bias: bool = False
    dropout: float = 0.0
    max_text_tokens: int = 100
    max_audio_tokens: int = 100
    sinusoidal_cond: bool = False
    spk_emb_dim: int = 1024
    codec_hz: float = 12.5
    # RoPE
    use_rotary_emb: bool = True
    rope_dim: int | None = None
    rope_theta: float = 10_000.0
    rope_theta_rescale_factor: float = 1.0
    global_rope_dim: int | None = None
    global_rope_theta: float | None = None
    window_size: int | None = None
    global_every: int | None = None
    # RQ-Transformer head
    use_rq_transformer: bool = False
    rq_d_model: int = 512
    rq_n_layers: int = 6
    rq_n_heads: int = 6
    n_quantizers: int = 9
    codebook_size: int = 4096
    # Conditioning projection heads
    has_sq_proj: bool = False
    has_wps_proj: bool = False
    has_spk_proj: bool = False
    # The reference takes the text vocabulary size from its tokenizer (src/vui/model.py:1075-1076);
    # without a tokenizer it is carried here (and otherwise read off token_emb.weight).
    vocab_size: int = 0

    @property
    def head_dim(self) -> int:
        return self.d_model // self.n_heads

    @property
    def kv_heads(self) -> int:
        return self.n_kv_heads if self.n_kv_heads is not None else self.n_heads

    @property
    def ffn(self) -> int:
        """LlamaMLP hidden size, src/vui/model.py:272-277."""
        if self.intermediate_size is not None:
            return self.intermediate_size
        h = int(2 * (4 * self.d_model) / 3)
        return 256 * ((h + 255) // 256)

    @property
    def rq_ffn(self) -> int:
        """RQBlock hidden size, src/vui/model.py:587-588."""
        h = int(self.rq_d_model * 8 / 3)
        return 64 * ((h + 63) // 64)


@dataclass
class DataConfig:
    max_secs: float = 360


@dataclass
class Config:
    checkpoint: str | dict | None = None
    model: VuiConfig = field(default_factory=VuiConfig)
    data: DataConfig = field(default_factory=DataConfig)

    @property
    def max_seq_len(self) -> int:
        """src/vui/config.py:70-76."""
        audio_tokens = int(self.data.max_secs * self.model.codec_hz)
        text_tokens = int(audio_tokens * 2.5)
        total = audio_tokens + text_tokens
        return 64 * ((total + 63) // 64)

    @classmethod
    def from_dict(cls, d: dict) -> "Config":
        return cls(checkpoint=d.get("checkpoint"), model=_from_dict(VuiConfig, d.get("model")),
                   data=_from_dict(DataConfig, d.get("data")))


def nano_config(preset: str = "A", max_secs: float = 240) -> Config:
    """Vui Nano.  Backbone dims are documented by the reference (README.md:270-271,
    docs/memory-budget.md:43,131); the depth head's are not and only two round-number fits
    reach the documented 305 M parameters: A = 512-d x 4 layers with a 100554-token vocabulary,
    B = 768-d x 5 layers with a 50534-token one."""
    base = dict(d_model=768, n_layers=22, n_heads=8, n_kv_heads=8, n_quantizers=16, codebook_size=2048,
                use_rq_transformer=True, has_spk_proj=True)
    if preset.upper() == "A":
        m = VuiConfig(**base, rq_d_model=512, rq_n_layers=4, rq_n_heads=8, vocab_size=100554)
    elif preset.upper() == "B":
        m = VuiConfig(**base, rq_d_model=768, rq_n_layers=5, rq_n_heads=8, vocab_size=50534)
    else:
        raise ValueError(f"unknown preset {preset!r}")
    return Config(model=m, data=DataConfig(max_secs=max_secs))


# ---- token language models (vui_amd.lm): layers described one by one ----
@dataclass
class RotaryConfig:
    """Rotation of the first `dims` entries of a vector, entry i paired with entry i + dims / 2, base^(-2 i / dims)."""

    dims: int
    base: float


@dataclass
class LatentAttentionConfig:
    """Causal softmax attention over a cached latent per position.  Per head dim unrotated and rot_dim rotated query
    and key dims and vdim value dims; kv_from names the layer whose latents are read instead of own ones."""

    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot: RotaryConfig
    kv_from: int | None = None


@dataclass
class MinGRUConfig:
    """Recurrence S <- (1 - z) S + z c over `width` channels, z and c functions of the token at hand alone."""

    width: int


@dataclass
class QueryTempConfig:
    """The query at position p is multiplied by 1 + coef ln(floor((p + 1) / every) + 1)."""

    coef: float
    every: int


@dataclass
class SigmoidAttentionConfig:
    """Causal attention whose weights are sigmoids of the scores.  heads query heads share kv_heads keys and values;
    queries and keys are normed; the bias over the distance is a table by buckets, full at bias_max."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: int
    q_temp: QueryTempConfig | None = None


@dataclass
class GatedLinearAttentionConfig:
    """Recurrence S <- diag(a) S + k v^T per head with a decay per key channel, a = sigmoid(z)^(1 / tau)."""

    heads: int
    dim: int
    vdim: int
    tau: float


@dataclass
class GatedMLPConfig:
    """Gated feed-forward with clamped branches."""

    ff: int
    limit: float


@dataclass
class XieluMLPConfig:
    """Ungated feed-forward with xIELU, whose two constants are weights."""

    ff: int


@dataclass
class ExpertsMLPConfig:
    """`top` of `experts` ungated feed-forwards of ff features (relu squared) per token."""

    ff: int
    experts: int
    top: int


@dataclass
class LoopConfig:
    """Layers start .. stop - 1 run `times` times in a row."""

    start: int
    stop: int
    times: int


@dataclass
class LMLayerConfig:
    mixer: "LatentAttentionConfig | MinGRUConfig | SigmoidAttentionConfig | GatedLinearAttentionConfig"
    mlp: "GatedMLPConfig | XieluMLPConfig | ExpertsMLPConfig | None" = None


@dataclass(frozen=True)
class LMDesign:
    """What a design fixes: the form of its layers, the mixers (by the names its configuration uses) and the
    feed-forwards it is made of."""

    sandwich: bool
    mixers: "dict[str, type]"
    mlps: "dict[str, type]"


LM_DESIGNS = {
    "Sakupel": LMDesign(False, {"latent_attention": LatentAttentionConfig, "mingru": MinGRUConfig}, {"dense": GatedMLPConfig}),
    "Mabidra": LMDesign(True, {"attention": SigmoidAttentionConfig, "gla": GatedLinearAttentionConfig},
                        {"dense": XieluMLPConfig, "moe": ExpertsMLPConfig}),
}


def _latent_attention(i: int, mx: dict, layers: "list[LMLayerConfig]") -> LatentAttentionConfig:
    mixer = LatentAttentionConfig(**{k: mx[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale")},
                                  rot=_from_dict(RotaryConfig, mx["rot"]), kv_from=mx.get("kv_from"))
    if mixer.rot.dims > mixer.rot_dim or mixer.rot.dims % 2:
        raise ValueError(f"layer {i}: cannot rotate {mixer.rot.dims} of {mixer.rot_dim} dims")
    if mixer.kv_from is not None:
        src = layers[mixer.kv_from].mixer if 0 <= mixer.kv_from < i else None
        if not isinstance(src, LatentAttentionConfig) or src.kv_from is not None:
            raise ValueError(f"layer {i}: kv_from={mixer.kv_from} names no earlier layer with latents of its own")
        if (src.kv_rank, src.rot_dim, src.rot) != (mixer.kv_rank, mixer.rot_dim, mixer.rot):
            raise ValueError(f"layer {i}: latents of layer {mixer.kv_from} have another shape or rotation")
    return mixer


def _sigmoid_attention(i: int, mx: dict) -> SigmoidAttentionConfig:
    qt = mx.get("q_temp")
    mixer = SigmoidAttentionConfig(**{k: mx[k] for k in ("heads", "kv_heads", "dim", "vdim", "scale", "bias_max")},
                                   q_temp=None if qt is None else QueryTempConfig(coef=qt["coef"], every=qt["every"]))
    if mixer.kv_heads < 1 or mixer.heads % mixer.kv_heads:
        raise ValueError(f"layer {i}: {mixer.heads} heads cannot share {mixer.kv_heads} keys and values")
    if mixer.q_temp is not None and mixer.q_temp.every < 1:
        raise ValueError(f"layer {i}: q_temp.every={mixer.q_temp.every}")
    return mixer


@dataclass
class LMConfig:
    """A decoder-only token model: config.json's `layers` (type, mixer, mlp), `norm`, `vocab`, `width`; for sandwich
    layers also `embedding.scale`, `norm.groups` and `loop`."""

    architecture: str
    width: int
    vocab: int
    norm_eps: float
    layers: "list[LMLayerConfig]"
    norm_groups: int = 0
    embed_scale: float = 1.0
    loop: LoopConfig | None = None

    @property
    def design(self) -> LMDesign:
        return LM_DESIGNS[self.architecture]

    def runs(self) -> "list[tuple[int, int | None]]":
        """Every layer run in order: (layer, pass of the loop that starts with it, or None)."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        a, b = self.loop.start, self.loop.stop
        body = [(i, t if i == a else None) for t in range(self.loop.times) for i in range(a, b)]
        return [(i, None) for i in range(a)] + body + [(i, None) for i in range(b, n)]

    @classmethod
    def from_dict(cls, d: dict) -> "LMConfig":
        arch = d["architecture"]
        if arch not in LM_DESIGNS:
            raise ValueError(f"{arch!r} is not a design of token models")
        design = LM_DESIGNS[arch]
        layers: "list[LMLayerConfig]" = []
        for i, e in enumerate(d["layers"]):
            mx = e["mixer"]
            kind = design.mixers.get(e["type"])
            if kind is LatentAttentionConfig:
                mixer = _latent_attention(i, mx, layers)
            elif kind is MinGRUConfig:
                mixer = MinGRUConfig(width=mx["width"])
            elif kind is SigmoidAttentionConfig:
                mixer = _sigmoid_attention(i, mx)
            elif kind is GatedLinearAttentionConfig:
                mixer = GatedLinearAttentionConfig(**{k: mx[k] for k in ("heads", "dim", "vdim", "tau")})
            else:
                raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
            mlp = None
            if e.get("mlp") is not None:
                ff = e["mlp"]
                kind = design.mlps.get(ff.get("kind", "dense"))
                if kind is GatedMLPConfig:
                    mlp = GatedMLPConfig(ff=ff["ff"], limit=ff["limit"])
                elif kind is XieluMLPConfig:
                    mlp = XieluMLPConfig(ff=ff["ff"])
                elif kind is ExpertsMLPConfig:
                    mlp = ExpertsMLPConfig(ff=ff["expert"]["ff"], experts=ff["router"]["experts"], top=ff["router"]["top"])
                    if not 1 <= mlp.top <= mlp.experts:
                        raise ValueError(f"layer {i}: cannot use {mlp.top} of {mlp.experts} experts")
                else:
                    raise ValueError(f"layer {i}: unknown feed-forward {ff['kind']!r}")
            layers.append(LMLayerConfig(mixer, mlp))
        out = cls(architecture=arch, width=d["width"], vocab=d["vocab"], norm_eps=d["norm"]["eps"], layers=layers)
        if design.sandwich:
            out.norm_groups = d["norm"].get("groups", 1)
            out.embed_scale = (d.get("embedding") or {}).get("scale", 1.0)
            if out.norm_groups < 1 or out.width % out.norm_groups:
                raise ValueError(f"a width of {out.width} has no {out.norm_groups} equal parts")
            if d.get("loop") is not None:
                out.loop = _from_dict(LoopConfig, d["loop"])
                if not (0 <= out.loop.start < out.loop.stop <= len(layers) and out.loop.times >= 1):
                    raise ValueError(f"loop over layers {out.loop.start} .. {out.loop.stop - 1} of {len(layers)}")
        return out
