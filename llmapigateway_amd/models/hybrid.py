"""Hybrid decoder: every layer names its mixer; a stretch of layers can run
several times in a row with the same weights.

The residual stream is fp32; a sublayer's output stays pending, with its own
norm where the design has one, and is added by the next norm's kernel
(ops.add_layernorm, ops.add_tanh_norm, ops.add_rms_norm). Where mixer and
feed-forward are parallel, both of their outputs are pending together, and
one kernel makes the two norms of the next layer. A loop pass starts by replacing the
stream with W [stream; embedding output] (+ step[t]); each pass of a layer
has its own cache view. Hyper-connected streams (models/streams.py) take the
place of the one stream where a design has them.

Serves Lelisun, Filinex, Mekevik and Duratar; another design built from these
mixers and feed-forwards needs only a configuration.
"""

from __future__ import annotations

from typing import Dict, List, Optional

import torch

from .. import ops
from .batch import ForwardBatch
from .configs import HybridConfig
from .feedforward import FEEDFORWARDS
from .mixers import MIXERS
from .streams import HyperStreams
from .weights import open_checkpoint


class HybridModel:
    extension = "_H"  # the HIP extension its kernels are in
    uses_segments = True  # steps over ForwardBatch.segs

    def __init__(
        self,
        config: HybridConfig,
        device: torch.device | str = "cpu",
        dtype: torch.dtype = torch.bfloat16,
        seed: int = 0,
        tp_group: Optional[object] = None,
        tp_rank: int = 0,
        tp_size: int = 1,
        full_config: Optional[HybridConfig] = None,
        max_positions: Optional[int] = None,
    ):
        if tp_size > 1 or tp_group is not None:
            raise NotImplementedError(f"{config.name}: hybrid decoders run on one GPU (tp=1)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"{config.name}: runs in bfloat16 or float32, not {dtype}")
        self.config = config
        self.device = torch.device(device)
        self.dtype = dtype
        self.max_positions = max_positions or config.max_positions
        self._ropes: Dict[tuple, torch.Tensor] = {}
        self.plans = {p for layer in config.layers for p in MIXERS[layer.type].plans}
        self._build(self._source(seed))

    # ---- weights ----
    @staticmethod
    def tensor_shapes(config: HybridConfig) -> Dict[str, tuple]:
        """Checkpoint tensor name -> shape."""
        W, V = config.hidden_size, config.vocab_size
        out = {"embed": (V, W), "head": (V, W)}

        def norm(name: str) -> None:
            out[name] = () if config.scalar_norms else (W,)
            if config.norm != "rms":
                out[name + ".b"] = (W,)
            if config.norm == "tanh":
                out[name + ".alpha"] = ()

        norm("final.norm")
        if config.embed_norm:
            norm("embed.norm")
        if config.loop is not None:
            out["loop.in"] = (W, 2 * W)
            if config.loop_step:
                out["loop.step"] = (config.loop[2], W)
        for i, layer in enumerate(config.layers):
            for k, s in MIXERS[layer.type].shapes(layer.mixer, W).items():
                out[f"l{i}.mix.{k}"] = s
            if layer.mlp is not None:
                for k, s in FEEDFORWARDS[layer.mlp["kind"]].shapes(layer.mlp, W).items():
                    out[f"l{i}.mlp.{k}"] = s
            for n in "12" if layer.mlp is not None else "1":
                norm(f"l{i}.norm{n}")
                if config.post_norm:
                    norm(f"l{i}.norm{n}b")
                if config.layer_scale:
                    out[f"l{i}.ls{n}"] = (W,)
                if config.streams:
                    S = config.streams
                    out.update({f"l{i}.hc{n}.in": (S,), f"l{i}.hc{n}.out": (S,),
                                f"l{i}.hc{n}.mix": (S, S)})
        return out

    def _source(self, seed: int):
        """name -> tensor, from the checkpoint or drawn at random."""
        shapes = self.tensor_shapes(self.config)
        if self.config.weights_dir is not None:
            ckpt = open_checkpoint(self.config.weights_dir)
            have = set(ckpt.names())
            for name, shape in shapes.items():
                if name not in have:
                    raise KeyError(f"{self.config.weights_dir}: no tensor '{name}'")
                if ckpt.shape(name) != tuple(shape):
                    raise ValueError(f"'{name}' is {ckpt.shape(name)}, expected {shape}")
            return ckpt.tensor
        big = sum(torch.Size(s).numel() for s in shapes.values()) >= 10 ** 8
        device = self.device if big else torch.device("cpu")
        gen = torch.Generator(device=device).manual_seed(seed)
        scale = self.config.embed_scale

        def draw(name: str) -> torch.Tensor:
            shape, leaf = shapes[name], name.rsplit(".", 1)[-1]
            t = torch.empty(shape, dtype=torch.float32, device=device)
            if leaf in ("norm", "norm1", "norm2", "norm1b", "norm2b", "D", "alpha", "ls1", "ls2"):
                return t.fill_(1.0)
            if ".hc" in name:
                t.normal_(0.0, 0.1, generator=gen)
                if leaf == "mix":
                    return t.add_(torch.eye(len(t), device=device))
                return t.add_(1.0 if leaf == "out" else 1.0 / len(t))
            if leaf in ("lq1", "lk1", "lq2", "lk2"):
                return t.normal_(0.0, 0.1, generator=gen)
            if leaf == "b" or leaf == "A_log":
                return t.fill_(2.0 if name.endswith((".f.b", ".a2.b")) else 0.0)
            if leaf == "dt_bias":
                return t.fill_(-2.0)
            if leaf in ("pb", "vmix"):
                return t.fill_(-4.0 if leaf == "pb" else 0.5)
            if leaf == "w0":
                return t.normal_(-1.5, 1.0, generator=gen)
            if ".mu." in name:
                return t.uniform_(0.0, 1.0, generator=gen)
            std = 1.0 / scale if name == "embed" else 0.02 if name == "loop.step" else (
                1.0 if len(shape) == 1 else shape[-1] ** -0.5
            )
            return t.normal_(0.0, std, generator=gen)

        return draw

    def _build(self, source) -> None:
        c = self.config

        def mat(name: str) -> torch.Tensor:
            return source(name).to(self.device).to(self.dtype)

        def vec(name: str) -> torch.Tensor:  # small vectors and taps: fp32
            return source(name).to(self.device).float().contiguous()

        def norm(name: str):
            if c.norm == "rms":
                w = vec(name)
                return (w.expand(c.hidden_size).contiguous() if c.scalar_norms else w,)
            parts = (vec(name), vec(name + ".b"))
            return parts + (float(source(name + ".alpha")),) if c.norm == "tanh" else parts

        self.embed = mat("embed")
        self.embed_norm = norm("embed.norm") if c.embed_norm else None
        self.loop_in = self.loop_step = None
        if c.loop is not None:
            self.loop_in = mat("loop.in")
            self.loop_step = vec("loop.step") if c.loop_step else [None] * c.loop[2]
        self.layers: List[dict] = []
        for i, layer in enumerate(c.layers):
            p = f"l{i}."
            ent = {
                "norm1": norm(p + "norm1"),
                "norm1b": norm(p + "norm1b") if c.post_norm else None,
                "mixer": MIXERS[layer.type](
                    layer.mixer, c.norm_eps,
                    lambda n, p=p: mat(f"{p}mix.{n}"), lambda n, p=p: vec(f"{p}mix.{n}"),
                    self._rope,
                ),
                "mlp": None,
                "ls1": vec(p + "ls1") if c.layer_scale else None,
            }
            if layer.mlp is not None:
                ent["norm2"] = norm(p + "norm2")
                ent["norm2b"] = norm(p + "norm2b") if c.post_norm else None
                ent["mlp"] = FEEDFORWARDS[layer.mlp["kind"]](
                    layer.mlp,
                    lambda n, p=p: mat(f"{p}mlp.{n}"), lambda n, p=p: vec(f"{p}mlp.{n}"),
                )
                ent["ls2"] = vec(p + "ls2") if c.layer_scale else None
            self.layers.append(ent)
        self.streams = None
        if c.streams:
            self.streams = HyperStreams(c.streams, [
                tuple(vec(f"l{i}.hc{n}.{leaf}") for leaf in ("in", "mix", "out"))
                for i, layer in enumerate(c.layers) for n in ("1", "2")[: 1 + bool(layer.mlp)]
            ], self.device)
        self.final_norm = norm("final.norm")
        if c.logit_scale != 1.0:  # the norm's last factors take it in
            self.final_norm = tuple(t * c.logit_scale for t in self.final_norm[:2]) + (
                self.final_norm[2:]
            )
        self.head = mat("head")

    def _rope(self, base: float, dims: int, scaling: Optional[dict] = None) -> torch.Tensor:
        key = (float(base), int(dims), tuple(sorted((scaling or {}).items())))
        if key not in self._ropes:
            self._ropes[key] = ops.build_pair_rope_cache(
                self.max_positions, dims, base, device=self.device, scaling=scaling
            )
        return self._ropes[key]

    # ---- forward ----
    def _norm(self, x, pending, post, norm, vec=None, replace=False) -> torch.Tensor:
        """Add the pending sublayer output (through its own norm, ``post``)
        to the stream, or replace the stream by it; the normed rows."""
        if self.config.norm == "rms":
            return ops.add_rms_norm(x, pending, norm, self.config.norm_eps, self.dtype)[0]
        delta = pending[0] if pending else None
        if self.config.norm == "tanh":
            return ops.add_tanh_norm(x, delta, post, norm, self.dtype, replace=replace)
        return ops.add_layernorm(
            x, delta, *norm, self.config.norm_eps, self.dtype, vec=vec, replace=replace
        )

    def _cast(self, x, pending, post, out) -> None:
        """The same addition; the stream itself goes to ``out``."""
        delta = pending[0] if pending else None
        if self.config.norm == "tanh":
            ops.add_tanh_norm(x, delta, post, None, self.dtype, out=out)
        else:
            ops.add_cast(x, delta, out)

    @torch.inference_mode()
    def step(self, batch: ForwardBatch, cache) -> torch.Tensor:
        """Logits [B, vocab] (fp32) at batch.logits_indices (every row if
        that is None); the caches take in the batch's rows."""
        c, W = self.config, self.config.hidden_size
        plan = ops.plan_segments(batch, self.dtype, self.plans)
        T = batch.token_ids.shape[0]
        if self.streams is not None:
            return self._step_streams(batch, cache, plan)
        both = x0 = None
        if c.loop is not None:  # [stream; embedding output], the loop's input
            both = torch.empty(T, 2 * W, dtype=self.dtype, device=self.device)
            x0 = both[:, W:]
        if self.embed_norm is None:
            x = ops.embed_scaled(batch.token_ids, self.embed, c.embed_scale, x0)
        else:
            x = ops.embed_tanh_norm(batch.token_ids, self.embed, self.embed_norm, x0)
        pending, post = (), None
        for r, (i, t) in enumerate(c.runs()):
            layer = self.layers[i]
            mixer, mlp = layer["mixer"], layer["mlp"]
            if c.parallel_mlp and mlp is not None:
                h, h2 = ops.add_rms_norm(
                    x, pending, layer["norm1"] + layer["norm2"], c.norm_eps, self.dtype
                )
                pending = (mixer(h, batch, cache.runs[r], plan), mlp(h2))
                continue
            if t is None:
                h = self._norm(x, pending, post, layer["norm1"])
            else:
                self._cast(x, pending, post, both[:, :W])
                h = self._norm(
                    x, (ops.linear_f32(both, self.loop_in),), None, layer["norm1"],
                    vec=self.loop_step[t], replace=True,
                )
            pending, post = (mixer(h, batch, cache.runs[r], plan),), layer["norm1b"]
            if mlp is not None:
                h = self._norm(x, pending, post, layer["norm2"])
                pending, post = (mlp(h),), layer["norm2b"]
        if batch.logits_indices is not None:
            pick = batch.logits_indices
            x, pending = x[pick], tuple(d[pick] for d in pending)
            if x.shape[0] == 0:
                return torch.empty(0, c.vocab_size, dtype=torch.float32, device=self.device)
        return self._logits(self._norm(x, pending, post, self.final_norm))

    def _step_streams(self, batch: ForwardBatch, cache, plan) -> torch.Tensor:
        """step() over hyper-connected streams."""
        c, st = self.config, self.streams
        x = ops.embed_rms_norm(batch.token_ids, self.embed, self.embed_norm[0], c.norm_eps)
        x, pending, q = x.unsqueeze(1), [], 0  # [T, stored streams, W]
        for r, (i, _) in enumerate(c.runs()):
            layer = self.layers[i]
            h, x, pending = st.read(q, x, pending, layer["norm1"][0], c.norm_eps, self.dtype)
            y = layer["mixer"](h, batch, cache.runs[r], plan)
            pending, q = pending + [(y, layer["ls1"])], q + 1
            if layer["mlp"] is not None:
                h, x, pending = st.read(q, x, pending, layer["norm2"][0], c.norm_eps, self.dtype)
                pending, q = pending + [(layer["mlp"](h), layer["ls2"])], q + 1
        if batch.logits_indices is not None and batch.logits_indices.shape[0] == 0:
            return torch.empty(0, c.vocab_size, dtype=torch.float32, device=self.device)
        return self._logits(st.read(
            q, x, pending, self.final_norm[0], c.norm_eps, self.dtype, batch.logits_indices
        )[0])

    def _logits(self, h: torch.Tensor) -> torch.Tensor:
        c = self.config
        logits = ops.linear_f32(h, self.head)
        if c.logit_softcap is not None:
            ops.soft_cap_(logits, c.logit_softcap)
        return logits
