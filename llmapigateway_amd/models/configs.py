"""Model configurations: architecture presets and checkpoint folders.

Shapes match the public architectures named by BASELINE.json's configs
(Llama-3-8B / Llama-3-70B / Mistral-7B), plus tiny presets for CPU tests.
A model can also be a checkpoint folder: its config.json names the
architecture that reads it.
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass, replace
from typing import Any, Dict, List, Optional, Tuple


@dataclass(frozen=True)
class ModelConfig:
    name: str
    hidden_size: int
    intermediate_size: int
    num_layers: int
    num_heads: int
    num_kv_heads: int
    vocab_size: int
    head_dim: int = 128
    rope_theta: float = 500000.0
    rms_eps: float = 1e-5
    max_positions: int = 8192
    tie_embeddings: bool = False

    @property
    def prefix_cacheable(self) -> bool:
        """Whether a sequence's cache pages alone are its whole state."""
        return True

    @property
    def q_size(self) -> int:
        return self.num_heads * self.head_dim

    @property
    def kv_size(self) -> int:
        return self.num_kv_heads * self.head_dim

    def scaled_for_tp(self, tp: int) -> "ModelConfig":
        """Per-rank shard shapes for tensor parallelism over xGMI."""
        assert self.num_heads % tp == 0 and self.num_kv_heads % tp == 0
        assert self.intermediate_size % tp == 0
        return replace(
            self,
            num_heads=self.num_heads // tp,
            num_kv_heads=self.num_kv_heads // tp,
            intermediate_size=self.intermediate_size // tp,
        )


@dataclass(frozen=True)
class HybridLayer:
    """One layer of a hybrid decoder: a mixer (its kind and sizes) and an
    optional feed-forward."""

    type: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]] = None


@dataclass(frozen=True)
class HybridConfig:
    """A decoder whose layers each name their mixer (models/mixers.py) and
    their feed-forward (models/feedforward.py), with an optional loop: layers
    [start, stop) run ``times`` times with the same weights, each pass with
    its own cache.

    The field set is what the Lelisun, Filinex, Mekevik and Duratar config.json
    files give and what their designs fix; ``max_positions`` is the framework's own
    bound (nothing in the designs limits it) and ``weights_dir`` says where
    the checkpoint lies (None: random init)."""

    name: str
    vocab_size: int
    hidden_size: int
    layers: Tuple[HybridLayer, ...]
    norm_eps: float = 1e-5
    norm: str = "layernorm"       # of the stream: "layernorm" | "tanh" (dynamic tanh) | "rms"
    parallel_mlp: bool = False    # mixer and feed-forward read the same stream
    post_norm: bool = False       # a norm on every sublayer's output, too
    embed_norm: bool = False
    scalar_norms: bool = False    # the stream's norms have one number for all coordinates
    streams: int = 0              # hyper-connected copies of the stream (0: one, plainly summed)
    layer_scale: bool = False     # a learned factor per coordinate of every sublayer's output
    embed_scale: float = 1.0
    loop: Optional[Tuple[int, int, int]] = None  # (start, stop, times)
    loop_step: bool = True        # a learned vector per loop pass
    logit_softcap: Optional[float] = None
    logit_scale: float = 1.0
    max_positions: int = 32768
    weights_dir: Optional[str] = None

    def __post_init__(self):
        if self.loop is not None:
            start, stop, times = self.loop
            if not (0 <= start < stop <= len(self.layers) and times >= 1):
                raise ValueError(f"bad loop {self.loop} over {len(self.layers)} layers")
        if self.norm not in ("layernorm", "tanh", "rms"):
            raise ValueError(f"unknown norm '{self.norm}'")
        if self.norm != "rms" and self.parallel_mlp:
            raise ValueError("mixer and feed-forward in parallel: RMS norms only")
        if self.norm == "rms" and self.loop is not None:
            raise ValueError("loops: layer norms and dynamic tanh only")
        if self.norm != "tanh" and (self.post_norm or self.embed_norm and not self.streams):
            raise ValueError("norms of sublayer outputs and of the embedding: dynamic tanh only")
        if self.streams and (self.norm != "rms" or self.parallel_mlp or not self.embed_norm):
            raise ValueError("streams: RMS norms, one also on the embedding, sublayers in turn")
        if not 0 <= self.streams <= 16:
            raise ValueError(f"{self.streams} streams: 16 at most")
        if not self.streams and (self.scalar_norms or self.layer_scale):
            raise ValueError("scalar norms and layer scales: hyper-connected streams only")
        for i, layer in enumerate(self.layers):
            try:
                self._check_layer(layer)
                self._check_kv_source(i)
            except ValueError as e:
                raise ValueError(f"layer {i}: {e}") from None
        shared = {
            layer.mixer["kv_heads"] * layer.mixer["vdim"]
            for layer in self.layers if layer.mixer.get("v_mix")
        }
        if len(shared) > 1:
            raise ValueError(f"layers that mix values have {sorted(shared)} of them")

    @staticmethod
    def _check_layer(layer: HybridLayer) -> None:
        m = layer.mixer
        if layer.type == "latent_attention":
            if m["rot"]["dims"] != m["rot_dim"] or m["rot_dim"] % 2:
                raise ValueError("rot.dims must be rot_dim, an even number")
        elif layer.type == "mamba2":
            if m["heads"] % m["groups"] or (m["heads"] * m["vdim"]) % m["norm_groups"]:
                raise ValueError("groups do not divide the heads")
        elif layer.type == "parallel":
            if m["left"]["heads"] % m["left"]["kv_heads"]:
                raise ValueError("kv_heads does not divide the heads")
            if not m["left"]["softcap"] > 0 or not m["right"]["tau"] > 0:
                raise ValueError("softcap and tau are positive")
        elif layer.type == "sigmoid_attention":
            if m["heads"] % m["kv_heads"]:
                raise ValueError("kv_heads does not divide the heads")
            if not m["bias_max"] > m["bias_rows"] // 2 > 0:
                raise ValueError(f"bias_max {m['bias_max']} for {m['bias_rows']} rows")
            if not m["window"] >= 1:
                raise ValueError(f"a window of {m['window']}")
        elif layer.type == "rotary_attention":
            if m["heads"] % m["kv_heads"]:
                raise ValueError("kv_heads does not divide the heads")
            if m["rot"]["dims"] % 2 or not 0 <= m["rot"]["dims"] <= m["dim"]:
                raise ValueError(f"rot.dims {m['rot']['dims']} of {m['dim']}")
            if not m["window"] >= 1 or not m["keep_first"] >= 0:
                raise ValueError(f"a window of {m['window']}, {m['keep_first']} kept")
        elif layer.type == "lightning":
            if len(m["decay"]) != m["heads"] or not all(0 <= d <= 1 for d in m["decay"]):
                raise ValueError(f"decay: a number within 0..1 for each of {m['heads']} heads")
        elif layer.type == "channel_delta":
            if m["heads"] % m["kv_heads"]:
                raise ValueError("kv_heads does not divide the heads")
            if not m["conv"] >= 1:
                raise ValueError(f"a convolution of {m['conv']} taps")
        elif layer.type not in ("mlstm", "wkv"):
            raise ValueError(f"unknown mixer '{layer.type}'")
        if layer.mlp is None:
            return
        if layer.mlp["kind"] == "moe":
            r = layer.mlp["router"]
            if not 1 <= r["top"] <= r["experts"]:
                raise ValueError(f"router: top {r['top']} of {r['experts']} experts")
        elif layer.mlp["kind"] not in ("dense", "xielu"):
            raise ValueError(f"unknown feed-forward '{layer.mlp['kind']}'")

    def _check_kv_source(self, i: int) -> None:
        m = self.layers[i].mixer
        j = m.get("kv_from")
        if j is None:
            return
        if self.loop is not None:
            raise ValueError("kv_from inside or beside a loop")
        source = self.layers[j] if 0 <= j < i else None
        if source is None or source.type != self.layers[i].type or "kv_from" in source.mixer:
            raise ValueError(f"kv_from {j}: not an earlier layer with keys of its own")
        for key in ("kv_heads", "dim", "vdim", "rot"):
            if source.mixer[key] != m[key]:
                raise ValueError(f"kv_from {j}: its {key} differs")

    @staticmethod
    def _common(raw: Dict[str, Any], layers) -> Dict[str, Any]:
        loop = raw.get("loop")
        return dict(
            vocab_size=raw["vocab"], hidden_size=raw["width"], layers=tuple(layers),
            norm_eps=raw["norm"]["eps"],
            loop=(loop["start"], loop["stop"], loop["times"]) if loop else None,
        )

    @classmethod
    def from_json(cls, raw: Dict[str, Any], name: str, weights_dir: Optional[str] = None):
        """Lelisun's config.json."""
        layers = [
            HybridLayer(type=e["type"], mixer=e["mixer"], mlp=e.get("mlp"))
            for e in raw["layers"]
        ]
        return cls(
            name=name, embed_scale=raw["embedding"]["scale"], weights_dir=weights_dir,
            **cls._common(raw, layers),
        )

    @classmethod
    def from_filinex_json(cls, raw: Dict[str, Any], name: str, weights_dir: Optional[str] = None):
        """Filinex's config.json. The ranks of the decay projections are only
        in the checkpoint's shapes: they join the mixers' sizes here."""
        from .weights import open_checkpoint

        ckpt = open_checkpoint(weights_dir)
        layers = []
        for i, e in enumerate(raw["layers"]):
            m = dict(e["mixer"])
            if e["type"] == "parallel":
                m["right"] = dict(m["right"], decay_rank=ckpt.shape(f"l{i}.mix.right.a1")[0])
            elif e["type"] == "wkv":
                m["decay_rank"] = ckpt.shape(f"l{i}.mix.w1")[0]
            layers.append(HybridLayer(type=e["type"], mixer=m, mlp=e.get("mlp")))
        return cls(
            name=name, norm="tanh", post_norm=True, embed_norm=True, loop_step=False,
            logit_softcap=raw["logit_softcap"], weights_dir=weights_dir,
            **cls._common(raw, layers),
        )

    @classmethod
    def from_mekevik_json(cls, raw: Dict[str, Any], name: str, weights_dir: Optional[str] = None):
        """Mekevik's config.json. How many rows a layer's distance table has
        is only in the checkpoint's shapes."""
        from .weights import open_checkpoint

        ckpt = open_checkpoint(weights_dir)
        layers = []
        for i, e in enumerate(raw["layers"]):
            if e["type"] != "attention":
                raise ValueError(f"layer {i}: unknown mixer '{e['type']}'")
            m, mlp = dict(e["mixer"]), e.get("mlp")
            m["window"] = m.pop("mask")["size"]
            m["bias_rows"] = ckpt.shape(f"l{i}.mix.rel")[0]
            if mlp is not None and mlp["kind"] == "moe":
                mlp = dict(mlp, router=dict(mlp["router"], bias=False))
            layers.append(HybridLayer(type="sigmoid_attention", mixer=m, mlp=mlp))
        return cls(
            name=name, norm="rms", parallel_mlp=True, embed_scale=raw["embedding"]["scale"],
            logit_scale=raw["logit_scale"], weights_dir=weights_dir,
            **cls._common(raw, layers),
        )

    @classmethod
    def from_duratar_json(cls, raw: Dict[str, Any], name: str, weights_dir: Optional[str] = None):
        """Duratar's config.json. The ranks of the low-rank projections are
        only in the checkpoint's shapes."""
        from .weights import open_checkpoint

        ckpt = open_checkpoint(weights_dir)
        layers = []
        for i, e in enumerate(raw["layers"]):
            m, kind, mlp = dict(e["mixer"]), e["type"], e.get("mlp")
            if kind == "attention":
                kind, mask = "rotary_attention", m.pop("mask")
                m.update(window=mask["size"], keep_first=mask.get("keep_first", 0))
            elif kind == "channel_delta":
                m["decay_rank"] = ckpt.shape(f"l{i}.mix.a1")[0]
                m["gate_rank"] = ckpt.shape(f"l{i}.mix.g1")[0]
            elif kind != "lightning":
                raise ValueError(f"layer {i}: unknown mixer '{kind}'")
            if mlp is not None and mlp["kind"] == "dense":
                mlp = dict(mlp, kind="xielu")
            layers.append(HybridLayer(type=kind, mixer=m, mlp=mlp))
        return cls(
            name=name, norm="rms", embed_norm=True, scalar_norms=True, streams=raw["streams"],
            layer_scale=True, weights_dir=weights_dir, **cls._common(raw, layers),
        )

    def kv_source(self, i: int) -> int:
        """The layer whose cached keys and values layer i reads."""
        return self.layers[i].mixer.get("kv_from", i)

    def runs(self) -> List[Tuple[int, Optional[int]]]:
        """The layers in the order they run, as (layer index, t): t is the
        number of the loop pass that this layer begins, None elsewhere."""
        if self.loop is None:
            return [(i, None) for i in range(len(self.layers))]
        start, stop, times = self.loop
        out: List[Tuple[int, Optional[int]]] = [(i, None) for i in range(start)]
        for t in range(times):
            out += [(i, t if i == start else None) for i in range(start, stop)]
        return out + [(i, None) for i in range(stop, len(self.layers))]

    @property
    def prefix_cacheable(self) -> bool:
        return all(
            layer.type in ("latent_attention", "sigmoid_attention", "rotary_attention")
            for layer in self.layers
        )

    def scaled_for_tp(self, tp: int) -> "HybridConfig":
        raise NotImplementedError(f"{self.name}: hybrid decoders run on one GPU (tp=1)")


# config.json "architecture" -> reader(raw, name, weights_dir)
ARCHITECTURES = {
    "Lelisun": HybridConfig.from_json,
    "Filinex": HybridConfig.from_filinex_json,
    "Mekevik": HybridConfig.from_mekevik_json,
    "Duratar": HybridConfig.from_duratar_json,
}


def load_model_dir(path: str):
    """The configuration of a checkpoint folder (config.json +
    model.safetensors)."""
    with open(os.path.join(path, "config.json")) as f:
        raw = json.load(f)
    arch = raw.get("architecture")
    if arch not in ARCHITECTURES:
        raise KeyError(f"Unknown architecture '{arch}' in {path}. Known: {sorted(ARCHITECTURES)}")
    path = os.path.abspath(path)
    return ARCHITECTURES[arch](raw, os.path.basename(path), path)


def _lelisun_preset(
    name: str, width: int, vocab: int, ff: int, heads: int, dim: int, rot_dim: int,
    kv_rank: int, q_rank: int, ssm_heads: int, ssm_vdim: int, state: int, groups: int,
    mem_heads: int, mem_dim: int, mem_vdim: int, times: int, repeat: int = 1,
    max_positions: int = 32768,
) -> HybridConfig:
    """A Lelisun of [latent attention, Mamba-2] looped, then mLSTM and
    latent attention; ``repeat`` widens the looped stretch."""
    attn = HybridLayer(
        "latent_attention",
        dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=dim, kv_rank=kv_rank,
             q_rank=q_rank, scale=(dim + rot_dim) ** -0.5,
             rot=dict(base=500000.0, dims=rot_dim)),
        dict(kind="dense", ff=ff),
    )
    ssm = HybridLayer(
        "mamba2",
        dict(heads=ssm_heads, vdim=ssm_vdim, state=state, groups=groups, conv=4,
             norm_groups=groups),
    )
    mem = HybridLayer(
        "mlstm", dict(heads=mem_heads, dim=mem_dim, vdim=mem_vdim, gate_cap=15.0)
    )
    looped = (attn, ssm) * repeat
    return HybridConfig(
        name=name, vocab_size=vocab, hidden_size=width, layers=looped + (mem, attn),
        embed_scale=width ** 0.5, loop=(0, len(looped), times),
        max_positions=max_positions,
    )


def _filinex_preset(
    name: str, width: int, vocab: int, heads: int, kv_heads: int, dim: int, lin_heads: int,
    lin_dim: int, lin_vdim: int, wkv_dim: int, rank: int, experts: int, top: int, ff: int,
    shared_ff: int, times: int, repeat: int = 1, max_positions: int = 32768,
) -> HybridConfig:
    """A Filinex of [parallel, wkv] pairs, all but the last layer looped."""
    mlp = dict(
        kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff, limit=7.0),
        shared=dict(ff=shared_ff, limit=7.0),
    )
    par = HybridLayer(
        "parallel",
        dict(left=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=dim ** -0.5,
                       softcap=30.0),
             right=dict(heads=lin_heads, dim=lin_dim, vdim=lin_vdim, tau=16.0,
                        decay_rank=rank),
             left_scale=1.0, right_scale=1.0),
        mlp,
    )
    mem = HybridLayer("wkv", dict(heads=width // wkv_dim, dim=wkv_dim, decay_rank=4 * rank), mlp)
    layers = (par, mem) * repeat
    return HybridConfig(
        name=name, vocab_size=vocab, hidden_size=width, layers=layers, norm="tanh",
        post_norm=True, embed_norm=True, loop=(0, len(layers) - 1, times), loop_step=False,
        logit_softcap=30.0, max_positions=max_positions,
    )


def _mekevik_preset(
    name: str, width: int, vocab: int, heads: int, kv_heads: int, dim: int, vdim: int,
    window: int, bias_rows: int, bias_max: int, ff: int, experts: int, top: int,
    expert_ff: int, layers: int, max_positions: int = 32768,
) -> HybridConfig:
    """A Mekevik of layers with a dense feed-forward and with experts in turn."""
    mixer = dict(
        heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=dim ** -0.5, window=window,
        bias_rows=bias_rows, bias_max=bias_max, v_mix=True,
    )
    mlps = (
        dict(kind="dense", ff=ff, limit=7.0),
        dict(kind="moe", expert=dict(ff=expert_ff),
             router=dict(experts=experts, top=top, scale=1.0, bias=False)),
    )
    return HybridConfig(
        name=name, vocab_size=vocab, hidden_size=width, norm="rms", parallel_mlp=True,
        layers=tuple(
            HybridLayer("sigmoid_attention", mixer, mlps[i % 2]) for i in range(layers)
        ),
        embed_scale=width ** 0.5, logit_scale=0.5, max_positions=max_positions,
    )


def _duratar_preset(
    name: str, width: int, vocab: int, heads: int, kv_heads: int, dim: int, window: int,
    keep_first: int, delta_heads: int, delta_kv_heads: int, delta_dim: int, delta_vdim: int,
    rank: int, mem_heads: int, mem_dim: int, ff: int, streams: int, layers: int,
    max_positions: int = 32768,
) -> HybridConfig:
    """A Duratar whose layers repeat delta, attention, lightning, delta; every
    second attention reads the keys and values of the one before it."""
    delta = dict(
        heads=delta_heads, kv_heads=delta_kv_heads, dim=delta_dim, vdim=delta_vdim, conv=4,
        decay_rank=rank, gate_rank=rank,
    )
    attn = dict(
        heads=heads, kv_heads=kv_heads, dim=dim, vdim=2 * dim, scale=dim ** -0.5, diff=0.5,
        window=window, keep_first=keep_first,
        rot=dict(base=500000.0, dims=dim // 2, scaling=dict(
            factor=8.0, low=1.0, high=4.0, original=8192)),
    )
    mem = dict(
        heads=mem_heads, dim=mem_dim, vdim=mem_dim,
        decay=[1.0 - 2.0 ** (-3 - 6 * i / mem_heads) for i in range(mem_heads)],
    )
    kinds = ("channel_delta", "rotary_attention", "lightning", "channel_delta")
    out = []
    for i in range(layers):
        kind = kinds[i % 4]
        m = (delta, attn, mem, delta)[i % 4]
        if kind == "rotary_attention" and i % 8 == 5:
            m = dict(m, kv_from=i - 4)
        out.append(HybridLayer(kind, m, dict(kind="xielu", ff=ff)))
    return HybridConfig(
        name=name, vocab_size=vocab, hidden_size=width, layers=tuple(out), norm_eps=1e-6,
        norm="rms", embed_norm=True, scalar_norms=True, streams=streams, layer_scale=True,
        max_positions=max_positions,
    )


MODEL_PRESETS = {
    "llama-3-8b": ModelConfig(
        name="llama-3-8b",
        hidden_size=4096,
        intermediate_size=14336,
        num_layers=32,
        num_heads=32,
        num_kv_heads=8,
        vocab_size=128256,
        rope_theta=500000.0,
    ),
    "llama-3-70b": ModelConfig(
        name="llama-3-70b",
        hidden_size=8192,
        intermediate_size=28672,
        num_layers=80,
        num_heads=64,
        num_kv_heads=8,
        vocab_size=128256,
        rope_theta=500000.0,
    ),
    # MHA family (GQA group = 1)
    "llama-2-7b": ModelConfig(
        name="llama-2-7b",
        hidden_size=4096,
        intermediate_size=11008,
        num_layers=32,
        num_heads=32,
        num_kv_heads=32,
        vocab_size=32000,
        rope_theta=10000.0,
        max_positions=4096,
    ),
    # odd GQA group (G = 7) exercises the templated decode kernel
    "qwen2-7b": ModelConfig(
        name="qwen2-7b",
        hidden_size=3584,
        intermediate_size=18944,
        num_layers=28,
        num_heads=28,
        num_kv_heads=4,
        vocab_size=152064,
        rope_theta=1000000.0,
    ),
    "mistral-7b": ModelConfig(
        name="mistral-7b",
        hidden_size=4096,
        intermediate_size=14336,
        num_layers=32,
        num_heads=32,
        num_kv_heads=8,
        vocab_size=32000,
        rope_theta=10000.0,
    ),
    # tiny shapes for CPU tests / smoke
    "tiny-llama": ModelConfig(
        name="tiny-llama",
        hidden_size=256,
        intermediate_size=512,
        num_layers=2,
        num_heads=4,
        num_kv_heads=2,
        vocab_size=512,
        head_dim=64,
        rope_theta=10000.0,
        max_positions=512,
    ),
    # tiny shape divisible for world-4 TP lockstep tests
    "tiny-llama-tp4": ModelConfig(
        name="tiny-llama-tp4",
        hidden_size=256,
        intermediate_size=512,
        num_layers=2,
        num_heads=8,
        num_kv_heads=4,
        vocab_size=512,
        head_dim=32,
        rope_theta=10000.0,
        max_positions=512,
    ),
    # looped hybrid decoder (latent attention + Mamba-2 + mLSTM)
    "tiny-lelisun": _lelisun_preset(
        "tiny-lelisun", width=96, vocab=320, ff=112, heads=3, dim=24, rot_dim=8,
        kv_rank=40, q_rank=56, ssm_heads=6, ssm_vdim=20, state=24, groups=3,
        mem_heads=2, mem_dim=16, mem_vdim=40, times=2, max_positions=1024,
    ),
    # layers as wide as llama-1b's and llama-3-8b's
    "lelisun-small": _lelisun_preset(
        "lelisun-small", width=2048, vocab=128256, ff=8192, heads=16, dim=128, rot_dim=64,
        kv_rank=512, q_rank=768, ssm_heads=64, ssm_vdim=64, state=128, groups=8,
        mem_heads=4, mem_dim=256, mem_vdim=512, times=2, repeat=3,
    ),
    "lelisun-base": _lelisun_preset(
        "lelisun-base", width=4096, vocab=128256, ff=14336, heads=32, dim=128, rot_dim=64,
        kv_rank=512, q_rank=1536, ssm_heads=128, ssm_vdim=64, state=128, groups=8,
        mem_heads=8, mem_dim=256, mem_vdim=512, times=2, repeat=6,
    ),
    # looped hybrid decoder (attention beside linear attention, WKV, experts)
    "tiny-filinex": _filinex_preset(
        "tiny-filinex", width=96, vocab=320, heads=4, kv_heads=2, dim=24, lin_heads=3,
        lin_dim=16, lin_vdim=40, wkv_dim=32, rank=8, experts=6, top=2, ff=40, shared_ff=56,
        times=2, max_positions=1024,
    ),
    # layers as wide as llama-1b's and llama-3-8b's
    "filinex-small": _filinex_preset(
        "filinex-small", width=2048, vocab=128256, heads=16, kv_heads=4, dim=128,
        lin_heads=8, lin_dim=128, lin_vdim=256, wkv_dim=64, rank=16, experts=32, top=4,
        ff=1536, shared_ff=2048, times=2, repeat=3,
    ),
    "filinex-base": _filinex_preset(
        "filinex-base", width=4096, vocab=128256, heads=32, kv_heads=8, dim=128,
        lin_heads=16, lin_dim=128, lin_vdim=256, wkv_dim=64, rank=16, experts=64, top=6,
        ff=1536, shared_ff=5120, times=2, repeat=4,
    ),
    # windowed sigmoid attention with mixed heads beside dense and expert layers
    "tiny-mekevik": _mekevik_preset(
        "tiny-mekevik", width=96, vocab=320, heads=6, kv_heads=3, dim=24, vdim=16, window=40,
        bias_rows=12, bias_max=33, ff=112, experts=6, top=2, expert_ff=40, layers=3,
        max_positions=1024,
    ),
    # layers as wide as llama-1b's and llama-3-8b's
    "mekevik-small": _mekevik_preset(
        "mekevik-small", width=2048, vocab=128256, heads=16, kv_heads=4, dim=128, vdim=128,
        window=1024, bias_rows=32, bias_max=128, ff=8192, experts=32, top=4, expert_ff=2048,
        layers=12,
    ),
    "mekevik-base": _mekevik_preset(
        "mekevik-base", width=4096, vocab=128256, heads=32, kv_heads=8, dim=128, vdim=128,
        window=1024, bias_rows=32, bias_max=128, ff=14336, experts=64, top=8, expert_ff=1792,
        layers=16,
    ),
    # hyper-connected streams over delta-rule, differential-attention and
    # lightning layers
    "tiny-duratar": _duratar_preset(
        "tiny-duratar", width=96, vocab=320, heads=4, kv_heads=2, dim=16, window=24,
        keep_first=3, delta_heads=4, delta_kv_heads=2, delta_dim=24, delta_vdim=40, rank=8,
        mem_heads=3, mem_dim=16, ff=96, streams=3, layers=6, max_positions=1024,
    ),
    # layers as wide as llama-1b's and llama-3-8b's, feed-forwards of as many
    # weights (two matrices instead of three)
    "duratar-small": _duratar_preset(
        "duratar-small", width=2048, vocab=128256, heads=16, kv_heads=4, dim=64, window=1024,
        keep_first=16, delta_heads=16, delta_kv_heads=16, delta_dim=128, delta_vdim=128,
        rank=128, mem_heads=16, mem_dim=128, ff=12288, streams=4, layers=12,
    ),
    "duratar-base": _duratar_preset(
        "duratar-base", width=4096, vocab=128256, heads=32, kv_heads=8, dim=64, window=1024,
        keep_first=16, delta_heads=32, delta_kv_heads=32, delta_dim=128, delta_vdim=128,
        rank=128, mem_heads=32, mem_dim=128, ff=21504, streams=4, layers=16,
    ),
    # small-but-real shape for 1-GPU kernel shakedown
    "llama-1b": ModelConfig(
        name="llama-1b",
        hidden_size=2048,
        intermediate_size=8192,
        num_layers=16,
        num_heads=32,
        num_kv_heads=8,
        vocab_size=128256,
        head_dim=64,
        rope_theta=500000.0,
    ),
}


def get_model_config(name: str):
    """The configuration of a preset, or of a checkpoint folder when
    ``name`` is the path of one."""
    if os.path.isfile(os.path.join(name, "config.json")):
        return load_model_dir(name)
    key = name.lower()
    if key not in MODEL_PRESETS:
        raise KeyError(f"Unknown model preset '{name}'. Known: {sorted(MODEL_PRESETS)}")
    return MODEL_PRESETS[key]
