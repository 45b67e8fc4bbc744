"""Model architecture registry.

Llama-3 family dims (8B / 70B per BASELINE.json configs #2-#4), a tiny config
for CPU tests, and DeepSeek-V3-style MoE configs (BASELINE config #5). Random
initialization is the benchmark mode (no network for checkpoints); safetensors
loading is supported for real weights.
"""

from __future__ import annotations

import dataclasses
from typing import List, Optional


@dataclasses.dataclass
class ModelSpec:
    name: str
    vocab_size: int = 128256
    hidden_size: int = 4096
    intermediate_size: int = 14336
    num_layers: int = 32
    num_heads: int = 32
    num_kv_heads: int = 8
    head_dim: int = 128
    rope_theta: float = 500000.0
    rms_eps: float = 1e-5
    max_seq_len: int = 8192
    tie_embeddings: bool = False
    # MoE (None => dense MLP)
    moe_num_experts: Optional[int] = None
    moe_top_k: int = 2
    moe_intermediate_size: Optional[int] = None
    moe_shared_experts: int = 0
    moe_dtype: str = "bf16"  # "fp8" enables the CDNA4 fp8 expert GEMM path

    is_hybrid = False

    @property
    def is_moe(self) -> bool:
        return self.moe_num_experts is not None


MODEL_REGISTRY = {
    # Llama-3 8B (BASELINE configs #2/#3)
    "llama3-8b": ModelSpec(
        name="llama3-8b",
        hidden_size=4096,
        intermediate_size=14336,
        num_layers=32,
        num_heads=32,
        num_kv_heads=8,
    ),
    # Llama-3 70B (BASELINE config #4, TP=8)
    "llama3-70b": ModelSpec(
        name="llama3-70b",
        hidden_size=8192,
        intermediate_size=28672,
        num_layers=80,
        num_heads=64,
        num_kv_heads=8,
    ),
    # tiny model for CPU tests (vocab covers the byte tokenizer's ~260 ids)
    "llama3-tiny": ModelSpec(
        name="llama3-tiny",
        vocab_size=512,
        hidden_size=128,
        intermediate_size=256,
        num_layers=2,
        num_heads=4,
        num_kv_heads=2,
        head_dim=32,
        max_seq_len=512,
    ),
    # tiny model whose head/vocab geometry divides by 4 (CPU world=4 TP tests)
    "llama3-tiny-w4": ModelSpec(
        name="llama3-tiny-w4",
        vocab_size=512,
        hidden_size=128,
        intermediate_size=256,
        num_layers=2,
        num_heads=8,
        num_kv_heads=4,
        head_dim=16,
        max_seq_len=512,
    ),
    # GPU-smoke-sized model (real head_dim for the HIP kernels)
    "llama3-micro": ModelSpec(
        name="llama3-micro",
        vocab_size=2048,
        hidden_size=1024,
        intermediate_size=2816,
        num_layers=4,
        num_heads=8,
        num_kv_heads=2,
        head_dim=128,
        max_seq_len=4096,
    ),
    # 8B-class projection shapes at 2 layers: exercises the K=4096 MFMA
    # GEMV paths (fp8 and bf16) end-to-end without an 8B weight build
    "llama3-2l4k": ModelSpec(
        name="llama3-2l4k",
        vocab_size=2048,
        hidden_size=4096,
        intermediate_size=14336,
        num_layers=2,
        num_heads=32,
        num_kv_heads=8,
        head_dim=128,
        max_seq_len=4096,
    ),
    # tiny MoE for CPU tests
    "moe-tiny": ModelSpec(
        name="moe-tiny",
        vocab_size=512,
        hidden_size=128,
        intermediate_size=256,
        num_layers=2,
        num_heads=4,
        num_kv_heads=2,
        head_dim=32,
        max_seq_len=512,
        moe_num_experts=8,
        moe_top_k=2,
        moe_intermediate_size=64,
        moe_shared_experts=1,
    ),
    # GPU-smoke-sized MoE (real head_dim, fp8-capable expert shapes)
    "moe-micro": ModelSpec(
        name="moe-micro",
        vocab_size=2048,
        hidden_size=1024,
        intermediate_size=2816,
        num_layers=4,
        num_heads=8,
        num_kv_heads=2,
        head_dim=128,
        max_seq_len=4096,
        moe_num_experts=16,
        moe_top_k=4,
        moe_intermediate_size=512,
        moe_shared_experts=1,
    ),
    # DeepSeek-V3-style MoE, scaled down to fit one MI355X comfortably
    # (BASELINE config #5: fp8 experts on CDNA4 MFMA)
    "deepseek-moe-small": ModelSpec(
        name="deepseek-moe-small",
        vocab_size=128256,
        hidden_size=2048,
        intermediate_size=8192,       # dense MLP for the first layer(s)
        num_layers=12,
        num_heads=16,
        num_kv_heads=4,
        moe_num_experts=64,
        moe_top_k=6,
        moe_intermediate_size=1408,
        moe_shared_experts=2,
    ),
    "deepseek-moe": ModelSpec(
        name="deepseek-moe",
        vocab_size=128256,
        hidden_size=4096,
        intermediate_size=14336,
        num_layers=28,
        num_heads=32,
        num_kv_heads=8,
        moe_num_experts=128,
        moe_top_k=8,
        moe_intermediate_size=2048,
        moe_shared_experts=1,
    ),
}


def get_model_spec(name):
    """A registry name, a checkpoint folder, or an already-built spec."""
    import os

    if not isinstance(name, str):
        return name
    if name in HYBRID_REGISTRY:
        cfg = HYBRID_REGISTRY[name]()
        return ARCHITECTURE_PARSERS[cfg["architecture"]](cfg, name=name)
    if os.path.isdir(name) and os.path.exists(os.path.join(name, "config.json")):
        return load_spec_from_dir(name)
    if name not in MODEL_REGISTRY:
        raise KeyError(f"unknown model {name!r}; known: {sorted(MODEL_REGISTRY)}")
    return MODEL_REGISTRY[name]


# ---------------------------------------------------------------------------
# Hybrid designs: a per-layer list of mixers (softmax attention, recurrent
# delta rule, ...) read from a checkpoint folder's config.json. Every size
# and every constant that can differ between checkpoints lives in the spec;
# nothing is taken from a particular checkpoint.


@dataclasses.dataclass
class MixerSpec:
    """One layer's token mixer. kind: "attention" (distance-penalty softmax
    attention) | "channel_delta" (gated delta rule) | "rotary_window"
    (rotary softmax attention with per-head query/key norm, an optional
    sliding window and an optional sink term) | "latent_attention" (softmax
    attention over a cached low-rank latent and one rotated key part shared
    by the heads) | "lightning" (linear attention with one fixed decay per
    head) | "gla" (linear attention with a learned decay per key channel) |
    "diff_attention" (rotary softmax attention in two maps per head over the
    same values, combined as a difference) | "retention" (rotary linear
    attention with one fixed decay per head) | "head_delta" (gated delta rule
    with one decay per head) | "key_attention" (softmax attention whose values
    are its keys, without positions) | "time_mix" (linear attention with a
    learned decay per key channel and a bonus for the current token, on inputs
    mixed with the previous token's) | "parallel" (two mixers side by side on
    the same input, their scaled outputs summed) | "gated_rotary" (rotary
    softmax attention with a window, kept first tokens, values mixed with an
    earlier layer's and an output gate per channel)."""

    kind: str
    heads: int
    kv_heads: int
    dim: int                      # per-head query/key size
    vdim: int                     # per-head value size
    scale: Optional[float] = None  # attention score scale
    conv: int = 0                 # short-convolution taps (recurrent mixers)
    # inner sizes of the low-rank decay / output-gate projections; only the
    # checkpoint's tensor shapes give them (None => the mixer's default)
    decay_rank: Optional[int] = None
    gate_rank: Optional[int] = None
    # rotary attention: rotated channels per head (0 = none), frequency base,
    # rescaling by wavelength {factor, low, high, original} or by pair index
    # {factor, fast, slow, original} (see rotary_inv_freq), or None
    rot_dims: int = 0
    rot_base: float = 10000.0
    rot_scaling: Optional[dict] = None
    # keys a query sees, itself included (None = all earlier keys)
    window: Optional[int] = None
    # keys at positions below keep_first are seen from beyond the window too
    keep_first: int = 0
    # a learned per-head term in the softmax denominator
    sink: bool = False
    # a sink of fixed score 0: one is added to the softmax denominator
    plus_one: bool = False
    # per-head RMS norm of queries and keys: "weighted" (before the rotation,
    # a weight per channel) or "unit_rotated" (after it, no weight)
    qk_norm: str = "weighted"
    # biases on the query, key and value projections
    qkv_bias: bool = False
    # values are mixed with those of the first layer that has v_mix:
    # v <- (1 - lambda) v + lambda v_first. v_first_from names that layer
    # (None: this is it, or no mixing)
    v_mix: bool = False
    v_first_from: Optional[int] = None
    # latent attention: size of the cached latent, rotated channels per head
    # (query) and of the shared key part, and the layer whose cached latent
    # this layer reads instead of projecting its own (None = its own)
    kv_rank: int = 0
    rot_dim: int = 0
    kv_from: Optional[int] = None
    # linear attention: fixed per-head decays ("lightning"), temperature of
    # the learned per-channel decay sigmoid(z)^(1/tau) ("gla")
    decay: Optional[List[float]] = None
    tau: float = 1.0
    # which channels a rotation pairs: "interleaved" (2i, 2i+1) or "half"
    # (i, i + rot_dims/2); the pairs' order does not change a dot product, so
    # a checkpoint in the "half" layout has its rows permuted once at load
    rot_layout: str = "interleaved"
    # score <- softcap * tanh(score / softcap) before the softmax (None = off)
    softcap: Optional[float] = None
    # differential attention: the constant of lambda and of the output scale
    diff: Optional[float] = None
    # latent attention: size of the normed latent the queries are projected
    # through (0 = queries come straight from the input)
    q_rank: int = 0
    # output gate read from the mixer input: "head" (one logit per head),
    # "channel" (one per output channel), "none"
    gate: str = "head"
    # "parallel": the two mixers and the scales of their outputs
    left: Optional["MixerSpec"] = None
    right: Optional["MixerSpec"] = None
    left_scale: float = 1.0
    right_scale: float = 1.0

    @property
    def has_kv(self) -> bool:
        if self.kind == "parallel":
            return self.left.has_kv or self.right.has_kv
        return self.kind in ("attention", "rotary_window", "diff_attention", "key_attention",
                             "gated_rotary") or (
            self.kind == "latent_attention" and self.kv_from is None)

    @property
    def has_state(self) -> bool:
        if self.kind == "parallel":
            return self.left.has_state or self.right.has_state
        return self.kind in ("channel_delta", "lightning", "gla", "retention", "head_delta",
                             "time_mix")


@dataclasses.dataclass
class RouterSpec:
    """Expert choice of a mixture-of-experts feed-forward. score: how router
    logits become scores s ("sigmoid" | "softmax"); with `correction` the
    ranking uses c = s + a learned vector while the mixing weights keep s;
    `groups` > 1 cuts the experts into runs of neighbours rated
    max1(c) + max2(c) (`rating` "top2") or max(c) ("max"), of which the
    `keep` top-rated may be picked from; w_j = scale * s_j / sum_k s_k over
    the `top` picked experts, or scale * s_j with renorm=False.
    act: the experts' gate activation ("silu" | "gelu_tanh" | "clamp_swish":
    g = min(gate, limit), u = clamp(up, -limit, limit),
    y = g sigmoid(alpha g) (u + 1)); the shared expert has its own limit and,
    with shared_gate, is scaled per token by the sigmoid of a learned
    projection. gated=False: an expert is down(act(up x)) with no gate
    branch (act "relu2": the square of relu). bias: the router adds a learned
    vector to its logits (it enters scores and choice alike)."""

    experts: int
    top: int
    ff: int                          # an expert's inner size
    score: str = "sigmoid"
    correction: bool = True
    groups: int = 1
    keep: int = 1
    scale: float = 1.0
    shared_ff: int = 0               # inner size of the always-on expert (0 = none)
    rating: str = "top2"
    renorm: bool = True
    act: str = "silu"
    limit: float = 0.0
    alpha: float = 1.702
    shared_limit: float = 0.0
    shared_gate: bool = False
    gated: bool = True
    bias: bool = False


@dataclasses.dataclass
class HybridLayerSpec:
    mixer: MixerSpec
    mlp_kind: Optional[str] = None   # None => no feed-forward; "dense" | "moe"
    mlp_ff: int = 0
    mlp_act: str = "silu"            # dense feed-forward gate activation
    router: Optional[RouterSpec] = None


@dataclasses.dataclass
class HybridSpec:
    """Architecture of a hybrid decoder (the Povazen design)."""

    name: str
    architecture: str
    vocab_size: int
    hidden_size: int
    layers: List[HybridLayerSpec]
    norm_eps: float
    norm_groups: int = 1
    canon_taps: int = 0
    logit_softcap: Optional[float] = None
    # "post_canon": grouped RMS norm on sublayer outputs, sublayers read
    # x + canon(x). "sandwich": a dynamic-tanh norm before and after every
    # sublayer. "pre_norm": a weighted layer norm before every sublayer.
    # "hyper": pre-norm sublayers (layer norm with weight and bias) around
    # `streams` residual streams joined by learned hyper-connections.
    # "parallel": one dynamic-tanh norm per layer, mixer and feed-forward both
    # read it and are added together. "parallel_rms": the same with an RMS
    # norm of its own for each sublayer (weights stored as distances from 1)
    # and a gated feed-forward.
    layer_style: str = "post_canon"
    # an RMS norm (weight stored as its distance from 1) follows the embedding
    embed_norm: bool = False
    embed_scale: float = 1.0
    streams: int = 1
    # learned read/mix/write coefficients between the streams (False: the
    # plain residual sum, which is one stream with all coefficients 1)
    hyper: bool = False
    # layers [start, stop) run `times` times in a row with the same weights;
    # every pass keeps its own keys, values and state
    loop: Optional[tuple] = None
    # before every pass of the loop but the first the embedding output is
    # added to the residual stream
    loop_embedding: bool = False
    # a sinusoidal position vector is added to the embedding
    sinusoid: bool = False
    # logits = head(norm(x)) * logit_scale; tied_head: the head is the
    # embedding table itself (without its scale)
    logit_scale: float = 1.0
    tied_head: bool = False
    max_seq_len: int = 1 << 20
    weights_path: Optional[str] = None

    is_moe = False
    is_hybrid = True

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def layer_runs(self) -> List[int]:
        """The layers in the order they run (a looped layer once per pass)."""
        n = len(self.layers)
        if not self.loop:
            return list(range(n))
        start, stop, times = self.loop
        return (list(range(start)) + list(range(start, stop)) * times
                + list(range(stop, n)))

    def loop_entries(self) -> List[int]:
        """Indexes into layer_runs() where a later pass of the loop begins."""
        if not self.loop:
            return []
        start, stop, times = self.loop
        return [start + k * (stop - start) for k in range(1, times)]


def povazen_spec_from_dict(cfg: dict, name: str = "povazen") -> HybridSpec:
    """Parse a Povazen config.json dict."""
    layers = []
    for entry in cfg["layers"]:
        m = entry["mixer"]
        kind = entry["type"]
        if kind not in ("attention", "channel_delta"):
            raise ValueError(f"unknown Povazen layer type {kind!r}")
        mixer = MixerSpec(
            kind=kind,
            heads=int(m["heads"]),
            kv_heads=int(m["kv_heads"]),
            dim=int(m["dim"]),
            vdim=int(m["vdim"]),
            scale=float(m["scale"]) if "scale" in m else None,
            conv=int(m.get("conv", 0)),
        )
        if mixer.heads % mixer.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        mlp = entry.get("mlp")
        if mlp is not None and mlp.get("kind") != "dense":
            raise ValueError(f"unknown Povazen feed-forward kind {mlp.get('kind')!r}")
        layers.append(
            HybridLayerSpec(
                mixer=mixer,
                mlp_kind=None if mlp is None else "dense",
                mlp_ff=0 if mlp is None else int(mlp["ff"]),
            )
        )
    width = int(cfg["width"])
    groups = int(cfg["norm"]["groups"])
    if width % groups:
        raise ValueError("width must be a multiple of norm.groups")
    return HybridSpec(
        name=name,
        architecture="Povazen",
        vocab_size=int(cfg["vocab"]),
        hidden_size=width,
        layers=layers,
        norm_eps=float(cfg["norm"]["eps"]),
        norm_groups=groups,
        canon_taps=int(cfg["canon"]["taps"]),
        logit_softcap=float(cfg["logit_softcap"]),
    )


def povazen_config_dict(
    vocab: int, width: int, pattern: str, heads: int, kv_heads: int, dim: int,
    vdim: int, ff: int, delta_heads: Optional[int] = None, conv: int = 4,
    taps: int = 3, groups: int = 4, eps: float = 1e-6, softcap: float = 30.0,
) -> dict:
    """A Povazen config.json dict from a layer pattern: 'D' = channel_delta
    layer without feed-forward, 'd' = with one, 'A'/'a' likewise attention."""
    layers = []
    for ch in pattern:
        mlp = {"kind": "dense", "ff": ff} if ch.islower() else None
        if ch in "Aa":
            mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                     "vdim": vdim, "scale": dim ** -0.5}
            layers.append({"type": "attention", "mixer": mixer, "mlp": mlp})
        else:
            dh = delta_heads or heads
            mixer = {"heads": dh, "kv_heads": dh, "dim": dim, "vdim": vdim, "conv": conv}
            layers.append({"type": "channel_delta", "mixer": mixer, "mlp": mlp})
    return {"architecture": "Povazen", "canon": {"taps": taps}, "layers": layers,
            "logit_softcap": softcap, "norm": {"eps": eps, "groups": groups},
            "vocab": vocab, "width": width}


def vazilorn_spec_from_dict(cfg: dict, name: str = "vazilorn") -> HybridSpec:
    """Parse a Vazilorn config.json dict: rotary sliding-window attention with
    sinks between dynamic-tanh norms, dense or routed feed-forwards."""
    layers = []
    for entry in cfg["layers"]:
        if entry["type"] != "attention":
            raise ValueError(f"unknown Vazilorn layer type {entry['type']!r}")
        m = entry["mixer"]
        rot = m.get("rot") or {}
        mask = m.get("mask") or {}
        mixer = MixerSpec(
            kind="rotary_window",
            heads=int(m["heads"]),
            kv_heads=int(m["kv_heads"]),
            dim=int(m["dim"]),
            vdim=int(m["vdim"]),
            scale=float(m["scale"]) if "scale" in m else None,
            rot_dims=int(rot.get("dims", 0)),
            rot_base=float(rot.get("base", 10000.0)),
            rot_scaling=dict(rot["scaling"]) if rot.get("scaling") else None,
            window=int(mask["size"]) if mask.get("size") else None,
            sink=True,
        )
        if mixer.heads % mixer.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if mixer.rot_dims % 2 or mixer.rot_dims > mixer.dim:
            raise ValueError("rot.dims must be even and at most dim")
        mlp = entry.get("mlp")
        ls = HybridLayerSpec(mixer=mixer)
        if mlp is not None:
            kind = mlp.get("kind")
            if kind == "dense":
                ls.mlp_kind, ls.mlp_ff, ls.mlp_act = "dense", int(mlp["ff"]), "gelu_tanh"
            elif kind == "moe":
                r = mlp["router"]
                grp = r.get("groups") or {}
                shared = mlp.get("shared") or {}
                ls.mlp_kind = "moe"
                ls.router = RouterSpec(
                    experts=int(r["experts"]), top=int(r["top"]), ff=int(mlp["expert"]["ff"]),
                    score="sigmoid", correction=True,
                    groups=int(grp.get("count", 1)), keep=int(grp.get("keep", grp.get("count", 1))),
                    scale=float(r.get("scale", 1.0)), shared_ff=int(shared.get("ff", 0)),
                )
                if ls.router.experts % ls.router.groups:
                    raise ValueError("experts must be a multiple of groups.count")
            else:
                raise ValueError(f"unknown Vazilorn feed-forward kind {kind!r}")
        layers.append(ls)
    return HybridSpec(
        name=name,
        architecture="Vazilorn",
        vocab_size=int(cfg["vocab"]),
        hidden_size=int(cfg["width"]),
        layers=layers,
        norm_eps=float(cfg["norm"]["eps"]),
        layer_style="sandwich",
    )


def vazilorn_config_dict(
    vocab: int, width: int, pattern: str, heads: int, kv_heads: int, dim: int,
    vdim: int, ff: int, window: Optional[int] = 64, rot_dims: Optional[int] = None,
    rot_base: float = 10000.0, rot_scaling: Optional[dict] = None, experts: int = 8,
    top: int = 2, expert_ff: int = 64, groups: int = 2, keep: int = 1,
    router_scale: float = 1.0, shared_ff: int = 0, eps: float = 1e-6,
    scale: Optional[float] = None,
) -> dict:
    """A Vazilorn config.json dict from a layer pattern: 'd' = attention +
    dense feed-forward, 'm' = attention + routed experts, 'a' = attention
    alone."""
    layers = []
    for ch in pattern:
        mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                 "scale": scale if scale is not None else dim ** -0.5,
                 "rot": {"base": rot_base, "dims": dim if rot_dims is None else rot_dims}}
        if rot_scaling:
            mixer["rot"]["scaling"] = dict(rot_scaling)
        if window:
            mixer["mask"] = {"size": window}
        if ch == "d":
            mlp = {"kind": "dense", "ff": ff}
        elif ch == "m":
            mlp = {"kind": "moe", "expert": {"ff": expert_ff},
                   "router": {"experts": experts, "top": top, "scale": router_scale,
                              "groups": {"count": groups, "keep": keep}}}
            if shared_ff:
                mlp["shared"] = {"ff": shared_ff}
        elif ch == "a":
            mlp = None
        else:
            raise ValueError(f"unknown layer letter {ch!r}")
        layers.append({"type": "attention", "mixer": mixer, "mlp": mlp})
    return {"architecture": "Vazilorn", "layers": layers, "norm": {"eps": eps},
            "vocab": vocab, "width": width}


def rafodra_spec_from_dict(cfg: dict, name: str = "rafodra") -> HybridSpec:
    """Parse a Rafodra config.json dict: pre-norm layers whose mixer is
    latent attention (optionally reading another layer's cached latent),
    lightning attention or gated linear attention, with dense silu or routed
    clamped-swish feed-forwards."""
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        kind, m = entry["type"], entry["mixer"]
        if kind == "latent_attention":
            rot = m.get("rot") or {}
            src = m.get("kv_from")
            mixer = MixerSpec(
                kind=kind, heads=int(m["heads"]), kv_heads=1, dim=int(m["dim"]),
                vdim=int(m["vdim"]), scale=float(m["scale"]) if "scale" in m else None,
                rot_dims=int(rot.get("dims", m["rot_dim"])),
                rot_base=float(rot.get("base", 10000.0)),
                kv_rank=int(m["kv_rank"]), rot_dim=int(m["rot_dim"]),
                kv_from=None if src is None else int(src), sink=True,
            )
            if mixer.rot_dims % 2 or mixer.rot_dims > mixer.rot_dim:
                raise ValueError("rot.dims must be even and at most rot_dim")
            if mixer.kv_from is not None:
                j = mixer.kv_from
                if not 0 <= j < i or layers[j].mixer.kind != kind or layers[j].mixer.kv_from is not None:
                    raise ValueError(f"layer {i}: kv_from must name an earlier latent-attention "
                                     "layer that projects its own latent")
                o = layers[j].mixer
                if (o.kv_rank, o.rot_dim, o.rot_dims, o.rot_base) != (
                        mixer.kv_rank, mixer.rot_dim, mixer.rot_dims, mixer.rot_base):
                    raise ValueError(f"layer {i}: latent sizes differ from layer {j}'s")
        elif kind == "lightning":
            mixer = MixerSpec(kind=kind, heads=int(m["heads"]), kv_heads=int(m["heads"]),
                              dim=int(m["dim"]), vdim=int(m["vdim"]),
                              decay=[float(d) for d in m["decay"]])
            if len(mixer.decay) != mixer.heads:
                raise ValueError("lightning: one decay per head")
        elif kind == "gla":
            mixer = MixerSpec(kind=kind, heads=int(m["heads"]), kv_heads=int(m["heads"]),
                              dim=int(m["dim"]), vdim=int(m["vdim"]), tau=float(m["tau"]))
        else:
            raise ValueError(f"unknown Rafodra layer type {kind!r}")
        mlp = entry.get("mlp")
        ls = HybridLayerSpec(mixer=mixer)
        if mlp is not None:
            mk = mlp.get("kind")
            if mk == "dense":
                ls.mlp_kind, ls.mlp_ff, ls.mlp_act = "dense", int(mlp["ff"]), "silu"
            elif mk == "moe":
                r = mlp["router"]
                grp = r.get("groups") or {}
                shared = mlp.get("shared") or {}
                ls.mlp_kind = "moe"
                ls.router = RouterSpec(
                    experts=int(r["experts"]), top=int(r["top"]), ff=int(mlp["expert"]["ff"]),
                    score="softmax", correction=False, groups=int(grp.get("count", 1)),
                    keep=int(grp.get("keep", grp.get("count", 1))),
                    scale=float(r.get("scale", 1.0)), shared_ff=int(shared.get("ff", 0)),
                    rating="max", renorm=False, act="clamp_swish",
                    limit=float(mlp["expert"]["limit"]),
                    shared_limit=float(shared.get("limit", 0.0)), shared_gate=bool(shared),
                )
                if ls.router.experts % ls.router.groups:
                    raise ValueError("experts must be a multiple of groups.count")
            else:
                raise ValueError(f"unknown Rafodra feed-forward kind {mk!r}")
        layers.append(ls)
    return HybridSpec(
        name=name, architecture="Rafodra", vocab_size=int(cfg["vocab"]),
        hidden_size=int(cfg["width"]), layers=layers, norm_eps=float(cfg["norm"]["eps"]),
        layer_style="pre_norm", embed_scale=float((cfg.get("embedding") or {}).get("scale", 1.0)),
    )


def rafodra_config_dict(
    vocab: int, width: int, pattern: str, heads: int = 4, dim: int = 16, vdim: int = 16,
    ff: int = 128, kv_rank: int = 24, rot_dim: int = 8, rot_base: float = 10000.0,
    scale: Optional[float] = None, lin_heads: Optional[int] = None, lin_dim: Optional[int] = None,
    lin_vdim: Optional[int] = None, decay: Optional[List[float]] = None, tau: float = 16.0,
    experts: int = 8, top: int = 2, expert_ff: int = 32, groups: int = 2, keep: int = 1,
    router_scale: float = 1.0, limit: float = 1.5, shared_ff: int = 0, shared_limit: float = 2.0,
    embed_scale: float = 1.0, eps: float = 1e-6,
) -> dict:
    """A Rafodra config.json dict from a layer pattern, one or two characters
    per layer: the mixer 'A' (latent attention), 'S' (latent attention
    reading the latest 'A' layer's latent), 'L' (lightning), 'G' (gla),
    followed by the feed-forward 'd' (dense), 'm' (routed experts) or '-'
    (none)."""
    if len(pattern) % 2:
        raise ValueError("pattern: two characters per layer")
    lh, ld, lv = lin_heads or heads, lin_dim or dim, lin_vdim or vdim
    if decay is None:
        decay = [1.0 - 2.0 ** (-(2 + 2 * h)) for h in range(lh)]
    layers, last_a = [], None
    for i in range(0, len(pattern), 2):
        mk, fk = pattern[i], pattern[i + 1]
        if mk in "AS":
            mixer = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank,
                     "rot_dim": rot_dim, "rot": {"base": rot_base, "dims": rot_dim},
                     "scale": scale if scale is not None else (dim + rot_dim) ** -0.5}
            if mk == "S":
                if last_a is None:
                    raise ValueError("'S' needs an earlier 'A' layer")
                mixer["kv_from"] = last_a
            else:
                last_a = len(layers)
            kind = "latent_attention"
        elif mk == "L":
            mixer, kind = {"heads": lh, "dim": ld, "vdim": lv, "decay": list(decay)}, "lightning"
        elif mk == "G":
            mixer, kind = {"heads": lh, "dim": ld, "vdim": lv, "tau": tau}, "gla"
        else:
            raise ValueError(f"unknown mixer letter {mk!r}")
        if fk == "d":
            mlp = {"kind": "dense", "ff": ff}
        elif fk == "m":
            mlp = {"kind": "moe", "expert": {"ff": expert_ff, "limit": limit},
                   "router": {"experts": experts, "top": top, "scale": router_scale,
                              "groups": {"count": groups, "keep": keep}}}
            if shared_ff:
                mlp["shared"] = {"ff": shared_ff, "limit": shared_limit}
        elif fk == "-":
            mlp = None
        else:
            raise ValueError(f"unknown feed-forward letter {fk!r}")
        layers.append({"type": kind, "mixer": mixer, "mlp": mlp})
    return {"architecture": "Rafodra", "embedding": {"scale": embed_scale}, "layers": layers,
            "norm": {"eps": eps}, "vocab": vocab, "width": width}


def parse_loop(loop: Optional[dict], layers: int) -> Optional[tuple]:
    """(start, stop, times) of a config's looped run of layers; None if there is
    nothing to repeat."""
    if not loop:
        return None
    start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    if not (0 <= start <= stop <= layers) or times < 1:
        raise ValueError("loop: need 0 <= start <= stop <= layers and times >= 1")
    return (start, stop, times) if stop > start and times != 1 else None


def suzulix_spec_from_dict(cfg: dict, name: str = "suzulix") -> HybridSpec:
    """Parse a Suzulix config.json dict: pre-norm sublayers (layer norm with
    weight and bias) on `streams` hyper-connected residual streams; mixers
    latent attention with a query latent, differential rotary attention with
    a score soft cap, or retention; routed feed-forwards of ungated
    squared-relu experts with a biased router and a gated shared expert; a
    run of layers may loop; the head is the embedding table."""
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        kind, m = entry["type"], entry["mixer"]
        rot = m.get("rot") or {}
        if kind == "latent_attention":
            mixer = MixerSpec(
                kind=kind, heads=int(m["heads"]), kv_heads=1, dim=int(m["dim"]),
                vdim=int(m["vdim"]), scale=float(m["scale"]) if "scale" in m else None,
                rot_dims=int(rot.get("dims", m["rot_dim"])),
                rot_base=float(rot.get("base", 10000.0)), rot_layout="half",
                kv_rank=int(m["kv_rank"]), rot_dim=int(m["rot_dim"]),
                q_rank=int(m.get("q_rank", 0)), sink=False, gate="channel",
            )
            if mixer.rot_dims % 2 or mixer.rot_dims > mixer.rot_dim:
                raise ValueError("rot.dims must be even and at most rot_dim")
        elif kind == "attention":
            mixer = MixerSpec(
                kind="diff_attention", heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
                dim=int(m["dim"]), vdim=int(m["vdim"]),
                scale=float(m["scale"]) if "scale" in m else None,
                rot_dims=int(rot.get("dims", 0)), rot_base=float(rot.get("base", 10000.0)),
                rot_layout="interleaved",
                softcap=float(m["softcap"]) if m.get("softcap") else None,
                diff=float(m["diff"]), gate="channel",
            )
            if mixer.heads % mixer.kv_heads:
                raise ValueError("heads must be a multiple of kv_heads")
            if mixer.rot_dims % 2 or mixer.rot_dims > mixer.dim:
                raise ValueError("rot.dims must be even and at most dim")
        elif kind == "retention":
            mixer = MixerSpec(
                kind=kind, heads=int(m["heads"]), kv_heads=int(m["heads"]), dim=int(m["dim"]),
                vdim=int(m["vdim"]), decay=[float(d) for d in m["decay"]],
                rot_dims=int(rot.get("dims", 0)), rot_base=float(rot.get("base", 10000.0)),
                rot_layout="half", gate="channel",
            )
            if len(mixer.decay) != mixer.heads:
                raise ValueError("retention: one decay per head")
            if mixer.rot_dims % 2 or mixer.rot_dims > mixer.dim:
                raise ValueError("rot.dims must be even and at most dim")
        else:
            raise ValueError(f"unknown Suzulix layer type {kind!r}")
        mlp = entry.get("mlp")
        ls = HybridLayerSpec(mixer=mixer)
        if mlp is not None:
            mk = mlp.get("kind", "moe")
            if mk != "moe":
                raise ValueError(f"unknown Suzulix feed-forward kind {mk!r}")
            r = mlp["router"]
            shared = mlp.get("shared") or {}
            ls.mlp_kind = "moe"
            ls.router = RouterSpec(
                experts=int(r["experts"]), top=int(r["top"]), ff=int(mlp["expert"]["ff"]),
                score="softmax", correction=False, groups=1, keep=1, scale=1.0,
                shared_ff=int(shared.get("ff", 0)), rating="max", renorm=True, act="relu2",
                shared_gate=bool(shared), gated=False, bias=True,
            )
            if ls.router.top > ls.router.experts:
                raise ValueError("router.top exceeds router.experts")
        layers.append(ls)
    loop = parse_loop(cfg.get("loop"), len(layers))
    streams = int(cfg.get("streams", 1))
    if streams < 1:
        raise ValueError("streams must be at least 1")
    return HybridSpec(
        name=name, architecture="Suzulix", vocab_size=int(cfg["vocab"]),
        hidden_size=int(cfg["width"]), layers=layers, norm_eps=float(cfg["norm"]["eps"]),
        layer_style="hyper", embed_scale=float((cfg.get("embedding") or {}).get("scale", 1.0)),
        streams=streams, hyper="streams" in cfg, loop=loop,
        logit_scale=float(cfg.get("logit_scale", 1.0)), tied_head=True,
    )


def suzulix_config_dict(
    vocab: int, width: int, pattern: str, heads: int = 4, kv_heads: int = 2, dim: int = 16,
    vdim: int = 16, kv_rank: int = 24, q_rank: int = 24, rot_dim: int = 8,
    lat_heads: Optional[int] = None, lat_dim: Optional[int] = None,
    lat_vdim: Optional[int] = None, rot_dims: Optional[int] = None, rot_base: float = 10000.0,
    scale: Optional[float] = None, softcap: Optional[float] = 50.0, diff: float = 0.5,
    ret_heads: Optional[int] = None, ret_dim: Optional[int] = None,
    ret_vdim: Optional[int] = None, ret_rot_dims: Optional[int] = None,
    decay: Optional[List[float]] = None, experts: int = 8, top: int = 2, expert_ff: int = 32,
    shared_ff: int = 0, streams: Optional[int] = 2, loop: Optional[tuple] = None,
    embed_scale: float = 1.0, logit_scale: float = 1.0, eps: float = 1e-5,
) -> dict:
    """A Suzulix config.json dict from a layer pattern, two characters per
    layer: the mixer 'L' (latent attention), 'A' (differential attention) or
    'R' (retention), then the feed-forward 'm' (routed experts) or '-'
    (none). loop = (start, stop, times); streams=None leaves the key out (one
    plain residual stream)."""
    if len(pattern) % 2:
        raise ValueError("pattern: two characters per layer")
    lh, ld, lv = lat_heads or heads, lat_dim or dim, lat_vdim or vdim
    rh, rd, rv = ret_heads or heads, ret_dim or dim, ret_vdim or vdim
    if decay is None:
        decay = [1.0 - 2.0 ** (-(3 + 2 * h)) for h in range(rh)]
    layers = []
    for i in range(0, len(pattern), 2):
        mk, fk = pattern[i], pattern[i + 1]
        if mk == "L":
            mixer = {"heads": lh, "dim": ld, "vdim": lv, "kv_rank": kv_rank, "q_rank": q_rank,
                     "rot_dim": rot_dim, "rot": {"base": rot_base, "dims": rot_dim},
                     "scale": scale if scale is not None else (ld + rot_dim) ** -0.5}
            kind = "latent_attention"
        elif mk == "A":
            mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "diff": diff,
                     "rot": {"base": rot_base, "dims": dim if rot_dims is None else rot_dims},
                     "scale": scale if scale is not None else dim ** -0.5}
            if softcap:
                mixer["softcap"] = softcap
            kind = "attention"
        elif mk == "R":
            mixer = {"heads": rh, "dim": rd, "vdim": rv, "decay": list(decay),
                     "rot": {"base": rot_base,
                             "dims": rd if ret_rot_dims is None else ret_rot_dims}}
            kind = "retention"
        else:
            raise ValueError(f"unknown mixer letter {mk!r}")
        if fk == "m":
            mlp = {"kind": "moe", "expert": {"ff": expert_ff},
                   "router": {"experts": experts, "top": top}}
            if shared_ff:
                mlp["shared"] = {"ff": shared_ff}
        elif fk == "-":
            mlp = None
        else:
            raise ValueError(f"unknown feed-forward letter {fk!r}")
        layers.append({"type": kind, "mixer": mixer, "mlp": mlp})
    cfg = {"architecture": "Suzulix", "embedding": {"scale": embed_scale}, "layers": layers,
           "logit_scale": logit_scale, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if streams is not None:
        cfg["streams"] = streams
    if loop is not None:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def rimonex_spec_from_dict(cfg: dict, name: str = "rimonex") -> HybridSpec:
    """Parse a Rimonex config.json dict: layers of one dynamic-tanh norm whose
    output both the mixer and an ungated gelu feed-forward read; mixers are the
    gated delta rule with one decay per head, or windowed attention on its own
    keys side by side with a time mix; sinusoidal positions at the embedding,
    which a looped run of layers adds again before every later pass; the head
    is the embedding table."""
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        kind, m = entry["type"], entry["mixer"]
        if kind == "delta":
            mixer = MixerSpec(kind="head_delta", heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
                              dim=int(m["dim"]), vdim=int(m["vdim"]), conv=int(m["conv"]))
            pairs = [mixer]
        elif kind == "parallel":
            a, r = m["left"], m["right"]
            mask = a.get("mask") or {}
            left = MixerSpec(
                kind="key_attention", heads=int(a["heads"]), kv_heads=int(a["kv_heads"]),
                dim=int(a["dim"]), vdim=int(a.get("vdim", a["dim"])),
                scale=float(a["scale"]) if "scale" in a else None,
                window=int(mask["size"]) if mask.get("size") else None, sink=True,
                softcap=float(a["softcap"]) if a.get("softcap") else None, gate="none",
            )
            if left.vdim != left.dim:
                raise ValueError(f"layer {i}: values that are the keys need vdim == dim")
            right = MixerSpec(kind="time_mix", heads=int(r["heads"]), kv_heads=int(r["heads"]),
                              dim=int(r["dim"]), vdim=int(r["dim"]))
            mixer = MixerSpec(
                kind="parallel", heads=left.heads, kv_heads=left.kv_heads, dim=left.dim,
                vdim=left.vdim, left=left, right=right,
                left_scale=float(m.get("left_scale", 1.0)),
                right_scale=float(m.get("right_scale", 1.0)),
            )
            pairs = [left, right]
        else:
            raise ValueError(f"unknown Rimonex layer type {kind!r}")
        if any(s.heads % s.kv_heads for s in pairs):
            raise ValueError("heads must be a multiple of kv_heads")
        mlp = entry.get("mlp")
        ls = HybridLayerSpec(mixer=mixer)
        if mlp is not None:
            if mlp.get("kind", "dense") != "dense":
                raise ValueError(f"unknown Rimonex feed-forward kind {mlp.get('kind')!r}")
            ls.mlp_kind, ls.mlp_ff, ls.mlp_act = "dense", int(mlp["ff"]), "gelu_tanh"
        layers.append(ls)
    return HybridSpec(
        name=name, architecture="Rimonex", vocab_size=int(cfg["vocab"]),
        hidden_size=int(cfg["width"]), layers=layers, norm_eps=float(cfg["norm"]["eps"]),
        layer_style="parallel", loop=parse_loop(cfg.get("loop"), len(layers)),
        loop_embedding=True, sinusoid=True, tied_head=True,
    )


def rimonex_config_dict(
    vocab: int, width: int, pattern: str, heads: int = 4, kv_heads: int = 2, dim: int = 16,
    window: Optional[int] = 24, scale: Optional[float] = None, softcap: Optional[float] = 30.0,
    mix_heads: Optional[int] = None, mix_dim: Optional[int] = None, left_scale: float = 1.0,
    right_scale: float = 1.0, delta_heads: Optional[int] = None,
    delta_kv_heads: Optional[int] = None, delta_dim: Optional[int] = None,
    delta_vdim: Optional[int] = None, conv: int = 4, ff: int = 128,
    loop: Optional[tuple] = None, eps: float = 1e-5,
) -> dict:
    """A Rimonex config.json dict from a layer pattern, two characters per
    layer: the mixer 'D' (delta) or 'P' (attention beside a time mix), then the
    feed-forward 'd' (dense) or '-' (none). loop = (start, stop, times)."""
    if len(pattern) % 2:
        raise ValueError("pattern: two characters per layer")
    layers = []
    for i in range(0, len(pattern), 2):
        mk, fk = pattern[i], pattern[i + 1]
        if mk == "D":
            dh = delta_heads or heads
            mixer, kind = {"heads": dh, "kv_heads": delta_kv_heads or dh,
                           "dim": delta_dim or dim, "vdim": delta_vdim or dim,
                           "conv": conv}, "delta"
        elif mk == "P":
            left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim,
                    "scale": scale if scale is not None else dim ** -0.5}
            if softcap:
                left["softcap"] = softcap
            if window:
                left["mask"] = {"size": window}
            mixer, kind = {"left": left, "left_scale": left_scale,
                           "right": {"heads": mix_heads or heads, "dim": mix_dim or dim},
                           "right_scale": right_scale}, "parallel"
        else:
            raise ValueError(f"unknown mixer letter {mk!r}")
        if fk not in "d-":
            raise ValueError(f"unknown feed-forward letter {fk!r}")
        layers.append({"type": kind, "mixer": mixer,
                       "mlp": {"kind": "dense", "ff": ff} if fk == "d" else None})
    cfg = {"architecture": "Rimonex", "layers": layers, "norm": {"eps": eps}, "vocab": vocab,
           "width": width}
    if loop is not None:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def rope_scaling_of(rot: dict) -> Optional[dict]:
    """A config's rot.scaling as a plain dictionary of floats; None if absent."""
    return {k: float(v) for k, v in rot["scaling"].items()} if rot.get("scaling") else None


def safesun_spec_from_dict(cfg: dict, name: str = "safesun") -> HybridSpec:
    """Parse a Safesun config.json dict: layers whose mixer and silu
    feed-forward each read their own RMS norm of the same stream; two kinds of
    gated rotary attention (weighted query/key norms before the rotation; or
    biases, unit query/key after it and one added to the softmax denominator),
    windows with kept first tokens, values mixed with the first value-mixing
    layer's; a norm after the embedding; the head is the embedding table."""
    layers, first = [], None
    for i, entry in enumerate(cfg["layers"]):
        kind, m = entry["type"], entry["mixer"]
        if kind not in ("attention", "attention_2"):
            raise ValueError(f"unknown Safesun layer type {kind!r}")
        second = kind == "attention_2"
        rot, mask = m.get("rot") or {}, m.get("mask") or {}
        mixer = MixerSpec(
            kind="gated_rotary", heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
            dim=int(m["dim"]), vdim=int(m["vdim"]),
            scale=float(m["scale"]) if "scale" in m else None,
            rot_dims=int(rot.get("dims", 0)), rot_base=float(rot.get("base", 10000.0)),
            rot_scaling=rope_scaling_of(rot), rot_layout="half",
            window=int(mask["size"]) if mask.get("size") else None,
            keep_first=int(mask.get("keep_first") or 0), plus_one=second, qkv_bias=second,
            qk_norm="unit_rotated" if second else "weighted", v_mix=bool(m.get("v_mix")),
            gate="channel",
        )
        if mixer.heads % mixer.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if mixer.rot_dims % 2 or mixer.rot_dims > mixer.dim:
            raise ValueError("rot.dims must be even and at most dim")
        if mixer.v_mix:
            if first is None:
                first = i
            else:
                o = layers[first].mixer
                if (o.kv_heads, o.vdim) != (mixer.kv_heads, mixer.vdim):
                    raise ValueError(f"layer {i}: mixed values need layer {first}'s kv_heads and vdim")
                mixer.v_first_from = first
        mlp = entry.get("mlp")
        ls = HybridLayerSpec(mixer=mixer)
        if mlp is not None:
            if mlp.get("kind", "dense") != "dense":
                raise ValueError(f"unknown Safesun feed-forward kind {mlp.get('kind')!r}")
            ls.mlp_kind, ls.mlp_ff, ls.mlp_act = "dense", int(mlp["ff"]), "silu"
        layers.append(ls)
    return HybridSpec(
        name=name, architecture="Safesun", vocab_size=int(cfg["vocab"]),
        hidden_size=int(cfg["width"]), layers=layers, norm_eps=float(cfg["norm"]["eps"]),
        layer_style="parallel_rms", embed_norm=True, tied_head=True,
    )


def safesun_config_dict(
    vocab: int, width: int, pattern: str, heads: int = 4, kv_heads: int = 2, dim: int = 16,
    vdim: int = 16, window: Optional[int] = 24, keep_first: int = 4, scale: Optional[float] = None,
    rot_dims: Optional[int] = None, rot_base: float = 10000.0, rot_scaling: Optional[dict] = None,
    heads_2: Optional[int] = None, dim_2: Optional[int] = None, window_2: Optional[int] = None,
    keep_first_2: Optional[int] = None, scale_2: Optional[float] = None,
    rot_dims_2: Optional[int] = None, rot_base_2: float = 500000.0, ff: int = 128,
    eps: float = 1e-5,
) -> dict:
    """A Safesun config.json dict from a layer pattern, two characters per
    layer: the mixer 'A' (attention) or 'B' (attention_2), lower case without
    value mixing, then the feed-forward 'd' (dense) or '-' (none). Parameters
    with _2 are attention_2's (default: attention's)."""
    if len(pattern) % 2:
        raise ValueError("pattern: two characters per layer")
    layers = []
    for i in range(0, len(pattern), 2):
        mk, fk = pattern[i], pattern[i + 1]
        if mk not in "AaBb":
            raise ValueError(f"unknown mixer letter {mk!r}")
        if fk not in "d-":
            raise ValueError(f"unknown feed-forward letter {fk!r}")
        if mk in "Aa":
            h, d, win, keep, sc = heads, dim, window, keep_first, scale
            rot = {"base": rot_base, "dims": d if rot_dims is None else rot_dims}
            if rot_scaling:
                rot["scaling"] = dict(rot_scaling)
        else:
            h, d = heads_2 or heads, dim_2 or dim
            win = window if window_2 is None else window_2
            keep = keep_first if keep_first_2 is None else keep_first_2
            sc = scale_2
            rot = {"base": rot_base_2, "dims": d if rot_dims_2 is None else rot_dims_2}
        mixer = {"heads": h, "kv_heads": kv_heads, "dim": d, "vdim": vdim, "rot": rot,
                 "scale": sc if sc is not None else d ** -0.5, "v_mix": mk.isupper()}
        if win:
            mixer["mask"] = {"size": win, "keep_first": keep}
        layers.append({"type": "attention" if mk in "Aa" else "attention_2", "mixer": mixer,
                       "mlp": {"kind": "dense", "ff": ff} if fk == "d" else None})
    return {"architecture": "Safesun", "layers": layers, "norm": {"eps": eps}, "vocab": vocab,
            "width": width}


# config.json "architecture" -> parser
ARCHITECTURE_PARSERS = {"Povazen": povazen_spec_from_dict,
                        "Vazilorn": vazilorn_spec_from_dict,
                        "Rafodra": rafodra_spec_from_dict,
                        "Suzulix": suzulix_spec_from_dict,
                        "Rimonex": rimonex_spec_from_dict,
                        "Safesun": safesun_spec_from_dict}

# named hybrid configurations (random-weight benchmarking and tests)
HYBRID_REGISTRY = {
    # CPU-test size
    "povazen-tiny": lambda: povazen_config_dict(
        vocab=512, width=64, pattern="Dad", heads=4, kv_heads=2, dim=16, vdim=8,
        ff=128, delta_heads=2),
    # GPU-smoke size
    "povazen-micro": lambda: povazen_config_dict(
        vocab=2048, width=1024, pattern="DdaD", heads=8, kv_heads=2, dim=128,
        vdim=128, ff=2816, delta_heads=8),
    # layer shapes of an ~8B-class model at 4 layers (speed measurements
    # beside llama3 layers of equal width)
    "povazen-4l4k": lambda: povazen_config_dict(
        vocab=2048, width=4096, pattern="dada", heads=32, kv_heads=8, dim=128,
        vdim=128, ff=14336, delta_heads=32),
    # CPU-test size
    "vazilorn-tiny": lambda: vazilorn_config_dict(
        vocab=512, width=64, pattern="dma", heads=4, kv_heads=2, dim=16, vdim=8,
        ff=128, window=24, rot_dims=8, experts=8, top=2, expert_ff=32, groups=2,
        keep=1, router_scale=1.5, shared_ff=48),
    # GPU-smoke size
    "vazilorn-micro": lambda: vazilorn_config_dict(
        vocab=2048, width=1024, pattern="dmdm", heads=8, kv_heads=2, dim=128,
        vdim=128, ff=2816, window=512, experts=16, top=4, expert_ff=512, groups=4,
        keep=2, router_scale=2.0, shared_ff=512,
        rot_scaling={"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}),
    # dense layer shapes of an ~8B-class model at 4 layers (speed beside
    # llama3 layers of equal width)
    "vazilorn-4l4k": lambda: vazilorn_config_dict(
        vocab=2048, width=4096, pattern="dddd", heads=32, kv_heads=8, dim=128,
        vdim=128, ff=14336, window=1024),
    "vazilorn-4l2k": lambda: vazilorn_config_dict(
        vocab=2048, width=2048, pattern="dddd", heads=16, kv_heads=4, dim=128,
        vdim=128, ff=8192, window=1024),
    # CPU-test size: every mixer and feed-forward kind once
    "rafodra-tiny": lambda: rafodra_config_dict(
        vocab=512, width=64, pattern="LdGmAdSmL-", heads=4, dim=16, vdim=8, ff=128,
        kv_rank=24, rot_dim=8, lin_heads=2, lin_dim=16, lin_vdim=24, experts=8, top=2,
        expert_ff=32, groups=2, keep=1, router_scale=1.5, shared_ff=48, embed_scale=4.0),
    # GPU-smoke size
    "rafodra-micro": lambda: rafodra_config_dict(
        vocab=2048, width=1024, pattern="LdGmAdLmSd", heads=8, dim=64, vdim=64, ff=2816,
        kv_rank=128, rot_dim=32, lin_heads=8, lin_dim=128, lin_vdim=128, experts=16, top=4,
        expert_ff=512, groups=4, keep=2, router_scale=2.0, shared_ff=512, embed_scale=8.0),
    # layer shapes of ~1B- and ~8B-class models at 4 layers (speed beside
    # Povazen and llama layers of equal width)
    "rafodra-4l2k": lambda: rafodra_config_dict(
        vocab=2048, width=2048, pattern="LdGdAdSd", heads=16, dim=128, vdim=128, ff=8192,
        kv_rank=192, rot_dim=64, lin_heads=16, lin_dim=128, lin_vdim=128),
    "rafodra-4l4k": lambda: rafodra_config_dict(
        vocab=2048, width=4096, pattern="LdGdAdSd", heads=32, dim=128, vdim=128, ff=14336,
        kv_rank=192, rot_dim=64, lin_heads=32, lin_dim=128, lin_vdim=128),
    # CPU-test size: every mixer once, a looped pair of layers, three streams
    "suzulix-tiny": lambda: suzulix_config_dict(
        vocab=512, width=64, pattern="LmAmRmR-Am", heads=4, kv_heads=2, dim=16, vdim=24,
        kv_rank=24, q_rank=40, rot_dim=8, lat_dim=16, lat_vdim=8, rot_dims=12, ret_heads=2,
        ret_dim=32, ret_vdim=16, experts=8, top=3, expert_ff=32, shared_ff=48, streams=3,
        loop=(1, 3, 2), embed_scale=4.0, logit_scale=0.5),
    # GPU-smoke size
    "suzulix-micro": lambda: suzulix_config_dict(
        vocab=2048, width=1024, pattern="LmAmRmRmLm", heads=8, kv_heads=2, dim=64, vdim=128,
        kv_rank=128, q_rank=256, rot_dim=32, lat_dim=64, lat_vdim=64, ret_heads=8,
        ret_dim=128, ret_vdim=128, experts=16, top=4, expert_ff=512, shared_ff=512,
        streams=2, loop=(0, 2, 2), embed_scale=8.0, logit_scale=0.25),
    # layer shapes of ~1B- and ~8B-class models at 4 layers (speed beside
    # Rafodra layers of equal width): two maps of half a head each, a 192 + 64
    # wide cached latent, 16 experts of ff/8 with 4 per token
    "suzulix-4l2k": lambda: suzulix_config_dict(
        vocab=2048, width=2048, pattern="LmAmRmRm", heads=16, kv_heads=4, dim=64, vdim=128,
        kv_rank=192, q_rank=512, rot_dim=64, lat_dim=128, lat_vdim=128, rot_base=500000.0,
        ret_heads=16, ret_dim=128, ret_vdim=128, experts=16, top=4, expert_ff=1024,
        shared_ff=1024, streams=2),
    "suzulix-4l4k": lambda: suzulix_config_dict(
        vocab=2048, width=4096, pattern="LmAmRmRm", heads=32, kv_heads=8, dim=64, vdim=128,
        kv_rank=192, q_rank=1024, rot_dim=64, lat_dim=128, lat_vdim=128, rot_base=500000.0,
        ret_heads=32, ret_dim=128, ret_vdim=128, experts=16, top=4, expert_ff=1792,
        shared_ff=1792, streams=2),
    # CPU-test size: both mixers, a looped pair of layers, a layer without feed-forward
    "rimonex-tiny": lambda: rimonex_config_dict(
        vocab=512, width=64, pattern="PdDdP-Dd", heads=4, kv_heads=2, dim=16, window=24,
        softcap=10.0, mix_heads=2, mix_dim=24, left_scale=0.8, right_scale=1.1, delta_heads=4,
        delta_kv_heads=2, delta_dim=16, delta_vdim=24, conv=3, ff=96, loop=(1, 3, 2)),
    # GPU-smoke size
    "rimonex-micro": lambda: rimonex_config_dict(
        vocab=2048, width=1024, pattern="PdDdPdDd", heads=8, kv_heads=2, dim=128, window=512,
        mix_heads=8, mix_dim=128, left_scale=0.9, right_scale=1.2, delta_heads=8, delta_dim=128,
        delta_vdim=128, ff=2816, loop=(0, 2, 2)),
    # layer shapes of ~1B- and ~8B-class models at 4 layers (speed beside
    # Povazen, Vazilorn and Rafodra layers of equal width)
    "rimonex-4l2k": lambda: rimonex_config_dict(
        vocab=2048, width=2048, pattern="PdDdPdDd", heads=16, kv_heads=4, dim=128, window=1024,
        mix_heads=16, mix_dim=128, delta_heads=16, delta_dim=128, delta_vdim=128, ff=8192),
    "rimonex-4l4k": lambda: rimonex_config_dict(
        vocab=2048, width=4096, pattern="PdDdPdDd", heads=32, kv_heads=8, dim=128, window=1024,
        mix_heads=32, mix_dim=128, delta_heads=32, delta_dim=128, delta_vdim=128, ff=14336),
    # CPU-test size: both mixers with and without value mixing, a layer without feed-forward
    "safesun-tiny": lambda: safesun_config_dict(
        vocab=512, width=64, pattern="adBdA-Bd", heads=4, kv_heads=2, dim=16, vdim=24, window=24,
        keep_first=3, rot_dims=12, window_2=20, keep_first_2=5, ff=96,
        rot_scaling={"factor": 4.0, "fast": 16.0, "slow": 1.0, "original": 64}),
    # GPU-smoke size
    "safesun-micro": lambda: safesun_config_dict(
        vocab=2048, width=1024, pattern="AdBdBdAd", heads=8, kv_heads=2, dim=128, vdim=128,
        window=512, keep_first=4, rot_dims_2=64, ff=2816,
        rot_scaling={"factor": 8.0, "fast": 32.0, "slow": 1.0, "original": 4096}),
    # layer shapes of ~1B- and ~8B-class models at 4 layers (speed beside
    # Vazilorn layers of equal width)
    "safesun-4l2k": lambda: safesun_config_dict(
        vocab=2048, width=2048, pattern="AdBdBdAd", heads=16, kv_heads=4, dim=128, vdim=128,
        window=1024, keep_first=4, ff=8192),
    "safesun-4l4k": lambda: safesun_config_dict(
        vocab=2048, width=4096, pattern="AdBdBdAd", heads=32, kv_heads=8, dim=128, vdim=128,
        window=1024, keep_first=4, ff=14336),
}


def load_spec_from_dir(path: str):
    """Model spec from a checkpoint folder (config.json + model.safetensors);
    the model class follows config.json's "architecture"."""
    import json
    import os

    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    arch = cfg.get("architecture")
    if arch not in ARCHITECTURE_PARSERS:
        raise KeyError(
            f"unknown architecture {arch!r} in {path}/config.json; "
            f"known: {sorted(ARCHITECTURE_PARSERS)}"
        )
    spec = ARCHITECTURE_PARSERS[arch](cfg, name=os.path.basename(os.path.normpath(path)))
    spec.weights_path = os.path.join(path, "model.safetensors")
    if os.path.exists(spec.weights_path):
        apply_tensor_shapes(spec, safetensors_shapes(spec.weights_path))
    return spec


def apply_tensor_shapes(spec: HybridSpec, shapes: dict) -> HybridSpec:
    """Fill the sizes that only tensor shapes give (name -> shape): the inner
    ranks of the low-rank decay and output-gate projections, whether an
    attention mixer carries a sink and a router a correction."""
    for i, layer in enumerate(spec.layers):
        if layer.mixer.kind == "rotary_window":
            layer.mixer.sink = f"l{i}.mix.sink" in shapes
        if layer.mixer.kind == "parallel":
            layer.mixer.left.sink = f"l{i}.mix.left.sink" in shapes
            w1 = shapes.get(f"l{i}.mix.right.w1")
            if w1 is not None:
                layer.mixer.right.decay_rank = int(w1[0])
        if layer.router is not None:
            layer.router.correction = f"l{i}.mlp.correction" in shapes
        a1, g1 = shapes.get(f"l{i}.mix.a1"), shapes.get(f"l{i}.mix.g1")
        if a1 is not None:
            layer.mixer.decay_rank = int(a1[0])
        if g1 is not None:
            layer.mixer.gate_rank = int(g1[0])
    return spec


def safetensors_shapes(path: str) -> dict:
    """name -> shape from a safetensors header (8-byte little-endian length,
    then that many bytes of JSON); reads no tensor data."""
    import json
    import struct

    with open(path, "rb") as f:
        (n,) = struct.unpack("<Q", f.read(8))
        header = json.loads(f.read(n))
    return {k: tuple(v["shape"]) for k, v in header.items() if k != "__metadata__"}
