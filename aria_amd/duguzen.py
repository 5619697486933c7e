"""Duguzen: a small decoder-only language model of latent-attention layers, dynamic-tanh norms before and after every sublayer, squared-relu or
group-limited mixture feed-forwards, and layers that run with another layer's weights on a cache of their own.

This file reads the design's config.json and tensor names and assembles the mechanisms of ``layers.py`` into the serving protocol of ``serving.py``
(caches, step function, scheduler, sampling and command line are the framework's).  A step runs in one of two ways:

* prompts, large batches and float32: sublayer by sublayer from here (tile GEMMs, flash attention, the fused stream passes);
* up to ``DECODE_ROWS`` single tokens in bf16: one C call (``aria_latent_decode``) that enqueues every kernel of every layer."""
from __future__ import annotations

import ctypes
from dataclasses import dataclass, field
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from . import hip, ops
from .checkpoint import load_checkpoint_dir
from .layers import (DynamicTanh, GroupLimitedMixture, LatentAttention, LatentCache, SquaredReluFeedForward, _frozen, padded, rotation_table, up8)
from .registry import read_config

bf16, f32 = torch.bfloat16, torch.float32
DECODE_ROWS = 16


@dataclass
class DuguzenLayerConfig:
    mixer: dict
    mlp: Optional[dict]
    source: int          # the layer whose tensors it runs with (itself unless weights_of says otherwise)


@dataclass
class DuguzenConfig:
    vocab: int
    width: int
    eps: float
    layers: List[DuguzenLayerConfig] = field(default_factory=list)

    @classmethod
    def from_dict(cls, c: dict) -> "DuguzenConfig":
        layers = []
        for i, e in enumerate(c["layers"]):
            if e["type"] != "latent_attention":
                raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
            mlp = e.get("mlp")
            if mlp is not None and mlp["kind"] not in ("dense", "moe"):
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            src, seen = i, set()
            while c["layers"][src].get("weights_of") is not None:      # (a borrowed layer may itself name a borrowed one)
                seen.add(src)
                src = int(c["layers"][src]["weights_of"])
                if src in seen or not 0 <= src < len(c["layers"]):
                    raise ValueError(f"layer {i}: weights_of leads to no layer with tensors")
            if c["layers"][src]["mixer"] != e["mixer"] or c["layers"][src].get("mlp") != mlp:
                raise ValueError(f"layer {i} differs from layer {src}, whose weights it uses")
            layers.append(DuguzenLayerConfig(e["mixer"], mlp, src))
        return cls(int(c["vocab"]), int(c["width"]), float(c["norm"]["eps"]), layers)


class DuguzenLayer(nn.Module):
    """Weights of one layer: the mixer, the feed-forward, four norms (two without a feed-forward)."""

    def __init__(self, w: Dict[str, torch.Tensor], cfg: DuguzenLayerConfig, width: int, eps: float, dtype):
        super().__init__()

        def norm(name):
            return DynamicTanh(w[name + ".alpha"], w[name], w[name + ".b"], width)

        m = cfg.mixer
        rot = m["rot"]
        self.mixer = LatentAttention({k[4:]: v for k, v in w.items() if k.startswith("mix.")}, heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"],
                                     vdim=m["vdim"], kv_rank=m["kv_rank"], scale=float(m["scale"]), rot_dims=int(rot["dims"]), rot_base=float(rot["base"]),
                                     eps=eps, width=width, dtype=dtype)
        self.norm1, self.norm1b = norm("norm1"), norm("norm1b")
        self.norm2 = self.norm2b = self.mlp = None
        if cfg.mlp is not None:
            self.norm2, self.norm2b = norm("norm2"), norm("norm2b")
            if cfg.mlp["kind"] == "dense":
                self.mlp = SquaredReluFeedForward(w["mlp.up"], w["mlp.down"], width, dtype)
            else:
                r = cfg.mlp["router"]
                g = r.get("groups") or {"count": 1, "keep": 1}
                experts = [[w[f"mlp.e{e}.{part}"] for e in range(r["experts"])] for part in ("gate", "up", "down")]
                self.mlp = GroupLimitedMixture(*experts, w["mlp.router"], w["mlp.correction"], top=r["top"], groups=g["count"], keep=g["keep"],
                                               width=width, dtype=dtype)


class DuguzenForCausalLM(nn.Module):
    """``from_pretrained`` / ``from_tensors`` -> a model with the serving protocol (``setup_caches``, ``step``, ``vocab``, ``device``)."""

    dtypes = (bf16, f32)

    def __init__(self, config: DuguzenConfig, tensors: Dict[str, torch.Tensor], dtype=bf16):
        super().__init__()
        if dtype not in self.dtypes:
            raise TypeError(f"Duguzen computes in bf16 or float32, not {dtype}")
        self.config, self.dtype, self.vocab = config, dtype, config.vocab
        self.width = up8(config.width)       # zero columns up to a multiple of 8: these norms have no statistics, so they stay exactly zero
        own = sorted({l.source for l in config.layers})
        by_layer = {i: {k[len(f"l{i}."):]: v for k, v in tensors.items() if k.startswith(f"l{i}.")} for i in own}
        self.weights = nn.ModuleDict({str(i): DuguzenLayer(by_layer[i], config.layers[i], self.width, config.eps, dtype) for i in own})
        self.final = DynamicTanh(tensors["final.norm.alpha"], tensors["final.norm"], tensors["final.norm.b"], self.width)
        self.embed = _frozen(padded(tensors["embed"], config.vocab, self.width), dtype)
        self.head = _frozen(padded(tensors["head"], up8(config.vocab), self.width), dtype)
        self.caches: List[LatentCache] = []
        self.ropes: List[torch.Tensor] = []
        self._decode: Optional["_DecodeTables"] = None

    @classmethod
    def from_tensors(cls, config: dict, tensors: Dict[str, torch.Tensor], device="cuda", dtype=bf16) -> "DuguzenForCausalLM":
        return cls(DuguzenConfig.from_dict(config), tensors, dtype).to(device).eval()

    @classmethod
    def from_pretrained(cls, path: str, device="cuda", dtype=bf16) -> "DuguzenForCausalLM":
        return cls.from_tensors(read_config(path), load_checkpoint_dir(path), device, dtype)

    def _apply(self, fn, *a, **k):       # (the decode tables hold raw addresses)
        self._decode = None
        return super()._apply(fn, *a, **k)

    @property
    def device(self):
        return self.head.device

    def layer(self, i: int) -> DuguzenLayer:
        return self.weights[str(self.config.layers[i].source)]

    def setup_caches(self, slots: int, max_len: int) -> None:
        """A latent cache per LAYER RUN (layers that share weights do not share a cache) and one rotation table per distinct rotation."""
        n, max_len = len(self.config.layers), up8(max_len)
        if self.caches and self.caches[0].rows.shape[:2] == (slots, max_len) and self.caches[0].rows.device == self.device:
            return                           # same geometry: rows behind a sequence's position are never read
        self.caches = [self.layer(i).mixer.new_cache(slots, max_len, self.device) for i in range(n)]
        tables: Dict[tuple, torch.Tensor] = {}
        for i in range(n):
            m = self.layer(i).mixer
            key = (m.rot_dims, m.rot_base)
            if key not in tables:
                tables[key] = rotation_table(max_len, m.rot_dims, m.rot_base, self.device)
        self.ropes = [tables[(self.layer(i).mixer.rot_dims, self.layer(i).mixer.rot_base)] for i in range(n)]
        self._decode = None

    def next_norm(self, i: int) -> DynamicTanh:
        """the norm that reads the stream after layer run i"""
        return self.layer(i + 1).norm1 if i + 1 < len(self.config.layers) else self.final

    @torch.no_grad()
    def step(self, batch, trace: Optional[list] = None) -> torch.Tensor:
        """Run a ``serving.StepBatch``; -> float32 logits [wanted rows, vocab].  ``trace``: receives the residual stream after every layer run."""
        if not self.caches:
            raise RuntimeError("setup_caches() first")
        if batch.max_len > self.caches[0].rows.shape[1] or max(batch.slots) >= self.caches[0].rows.shape[0]:
            raise ValueError("the batch does not fit the caches")
        T = batch.ids.numel()
        if self.dtype == bf16 and trace is None and batch.longest == 1 and T <= DECODE_ROWS:
            if self._decode is None:
                self._decode = _DecodeTables(self)
            logits = self._decode.run(batch)
            return logits if batch.wanted is None or batch.wanted.numel() == T else logits[batch.wanted.long()]
        x = torch.empty((T, self.width), dtype=f32, device=self.device)
        h = ops.dyt_stream(x, None, self.layer(0).norm1.params(), ids=batch.ids, table=self.embed)
        for i in range(len(self.config.layers)):
            L = self.layer(i)
            y = L.mixer(h, batch, self.caches[i], self.ropes[i])
            h = ops.dyt_stream(x, L.norm1b.params(), (L.norm2 if L.mlp is not None else self.next_norm(i)).params(), y=y)
            if L.mlp is not None:
                h = ops.dyt_stream(x, L.norm2b.params(), self.next_norm(i).params(), **L.mlp(h))
            if trace is not None:
                trace.append(x.clone())
        if batch.wanted is not None:
            if batch.wanted.numel() == 0:
                return torch.empty((0, self.vocab), dtype=f32, device=self.device)
            h = ops.permute_any(h, batch.wanted.contiguous(), 1)
        return ops.linear_any(h, self.head, out_dtype=f32)[:, :self.vocab]


class _DecodeTables:
    """Pointer and size tables of ``aria_latent_decode`` for a model's weights and caches (re-made when either moves), scratch and logits buffers."""

    def __init__(self, model: DuguzenForCausalLM):
        n = len(model.config.layers)
        S = model.caches[0].rows.shape[1]
        self.vocab, self.n = model.vocab, n
        self.layers = (hip.LatentLayer * n)()
        self.scratch: Optional[torch.Tensor] = None
        for i in range(n):
            L, t = model.layer(i), self.layers[i]
            m = L.mixer
            t.mix, t.norm1b, t.next = m.shape(S), L.norm1b.params(), model.next_norm(i).params()
            t.w_in, t.w_uk, t.w_uv, t.w_o = (p.data_ptr() for p in (m.w_in, m.w_uk, m.w_uv, m.w_o))
            t.kv_norm, t.rope, t.cache = m.kv_norm.data_ptr(), model.ropes[i].data_ptr(), model.caches[i].rows.data_ptr()
            if L.mlp is not None:
                t.norm2, t.norm2b, t.ff = L.norm2.params(), L.norm2b.params(), L.mlp.ff
                if isinstance(L.mlp, SquaredReluFeedForward):
                    t.mlp, t.w_up, t.w_down = 1, L.mlp.up.data_ptr(), L.mlp.down.data_ptr()
                else:
                    t.mlp, t.E, t.groups, t.keep, t.k = 2, L.mlp.n_experts, L.mlp.groups, L.mlp.keep, L.mlp.top
                    t.w_gate, t.w_up, t.w_down = L.mlp.gate.data_ptr(), L.mlp.up.data_ptr(), L.mlp.down.data_ptr()
                    t.w_router, t.correction = L.mlp.router.data_ptr(), L.mlp.correction.data_ptr()
        self.stack = hip.LatentStack(n, model.width, model.head.shape[0], model.layer(0).norm1.params(), model.embed.data_ptr(), model.head.data_ptr())
        self.device, self.rows = model.device, model.head.shape[0]

    def run(self, batch) -> torch.Tensor:
        T, lib = batch.ids.numel(), hip.get_lib()
        stack, layers = ctypes.byref(self.stack), ctypes.byref(self.layers)
        need = int(lib.cdll.aria_latent_decode_scratch(stack, layers, T, batch.max_len))
        if self.scratch is None or self.scratch.numel() < need:
            self.scratch = torch.empty(need, dtype=torch.uint8, device=self.device)
        logits = torch.empty((T, self.rows), dtype=f32, device=self.device)
        for t in (batch.ids, batch.slot, batch.pos):
            assert t.dtype == torch.int32 and t.is_contiguous() and t.numel() == T
        lib.call("aria_latent_decode", stack, layers, T, batch.ids.data_ptr(), batch.slot.data_ptr(), batch.pos.data_ptr(), batch.max_len,
                 logits.data_ptr(), self.scratch.data_ptr(), self.scratch.numel(), ops._stream(logits))
        return logits[:, :self.vocab]
