"""Hybrid decoder: every layer names its mixer; a stretch of layers can run
several times in a row with the same weights.

The residual stream is fp32; a sublayer's output stays pending and is added
by the next norm's kernel (ops.add_layernorm). A loop pass starts by
replacing the stream with W [stream; embedding output] + step[t]; each pass
of a layer has its own cache view.

Serves Lelisun; another design built from these mixers needs only a
configuration.
"""

from __future__ import annotations

from typing import Dict, List, Optional

import torch

from .. import ops
from .batch import ForwardBatch
from .configs import HybridConfig
from .mixers import MIXERS
from .twins import add_decode_twins
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
        self._build(self._source(seed))

    # ---- weights ----
    @staticmethod
    def tensor_shapes(config: HybridConfig) -> Dict[str, tuple]:
        """Checkpoint tensor name -> shape."""
        W, V = config.hidden_size, config.vocab_size
        out = {"embed": (V, W), "final.norm": (W,), "final.norm.b": (W,), "head": (V, W)}
        if config.loop is not None:
            out["loop.in"] = (W, 2 * W)
            out["loop.step"] = (config.loop[2], W)
        for i, layer in enumerate(config.layers):
            out[f"l{i}.norm1"] = out[f"l{i}.norm1.b"] = (W,)
            for k, s in MIXERS[layer.type].shapes(layer.mixer, W).items():
                out[f"l{i}.mix.{k}"] = s
            if layer.mlp is not None:
                ff = layer.mlp["ff"]
                out[f"l{i}.norm2"] = out[f"l{i}.norm2.b"] = (W,)
                out[f"l{i}.mlp.gate"] = out[f"l{i}.mlp.up"] = (ff, W)
                out[f"l{i}.mlp.down"] = (W, ff)
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
            if leaf in ("norm", "norm1", "norm2", "D"):
                return t.fill_(1.0)
            if leaf == "b" or leaf == "A_log":
                return t.fill_(2.0 if name.endswith(".f.b") else 0.0)
            if leaf == "dt_bias":
                return t.fill_(-2.0)
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

        self.embed = mat("embed")
        self.loop_in = self.loop_step = None
        if c.loop is not None:
            self.loop_in, self.loop_step = mat("loop.in"), vec("loop.step")
        self.layers: List[dict] = []
        for i, layer in enumerate(c.layers):
            p = f"l{i}."
            ent = {
                "norm1": (vec(p + "norm1"), vec(p + "norm1.b")),
                "mixer": MIXERS[layer.type](
                    layer.mixer, c.norm_eps,
                    lambda n, p=p: mat(f"{p}mix.{n}"), lambda n, p=p: vec(f"{p}mix.{n}"),
                    self._rope,
                ),
                "mlp": None,
            }
            if layer.mlp is not None:
                ent["norm2"] = (vec(p + "norm2"), vec(p + "norm2.b"))
                ent["mlp"] = {
                    "gate_up": torch.cat([mat(p + "mlp.gate"), mat(p + "mlp.up")]),
                    "down": mat(p + "mlp.down"),
                }
                add_decode_twins(ent["mlp"], ("gate_up", "down"))
            self.layers.append(ent)
        self.final_norm = (vec("final.norm"), vec("final.norm.b"))
        self.head = mat("head")

    def _rope(self, base: float, dims: int) -> torch.Tensor:
        key = (float(base), int(dims))
        if key not in self._ropes:
            self._ropes[key] = ops.build_pair_rope_cache(
                self.max_positions, dims, base, device=self.device
            )
        return self._ropes[key]

    # ---- forward ----
    @torch.inference_mode()
    def step(self, batch: ForwardBatch, cache) -> torch.Tensor:
        """Logits [B, vocab] (fp32) at batch.logits_indices (every row if
        that is None); the caches take in the batch's rows."""
        c, eps, W = self.config, self.config.norm_eps, self.config.hidden_size
        plan = ops.plan_segments(batch, self.dtype)
        T = batch.token_ids.shape[0]
        both = x0 = None
        if c.loop is not None:  # [stream; embedding output], the loop's input
            both = torch.empty(T, 2 * W, dtype=self.dtype, device=self.device)
            x0 = both[:, W:]
        x = ops.embed_scaled(batch.token_ids, self.embed, c.embed_scale, x0)
        delta = None
        for r, (i, t) in enumerate(c.runs()):
            layer = self.layers[i]
            if t is None:
                h = ops.add_layernorm(x, delta, *layer["norm1"], eps, self.dtype)
            else:
                ops.add_cast(x, delta, both[:, :W])
                h = ops.add_layernorm(
                    x, ops.linear_f32(both, self.loop_in), *layer["norm1"], eps,
                    self.dtype, vec=self.loop_step[t], replace=True,
                )
            delta = layer["mixer"](h, batch, cache.runs[r], plan)
            if layer["mlp"] is not None:
                m = layer["mlp"]
                h = ops.add_layernorm(x, delta, *layer["norm2"], eps, self.dtype)
                delta = ops.linear(
                    ops.swiglu_linear(
                        h, m["gate_up"], m.get("gate_up_swz"), m.get("gate_up_int")
                    ),
                    m["down"], m.get("down_swz"),
                )
        if batch.logits_indices is not None:
            x, delta = x[batch.logits_indices], delta[batch.logits_indices]
            if x.shape[0] == 0:
                return torch.empty(0, c.vocab_size, dtype=torch.float32, device=self.device)
        h = ops.add_layernorm(x, delta, *self.final_norm, eps, self.dtype)
        return ops.linear_f32(h, self.head)
