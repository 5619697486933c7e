"""Kozipel: a small decoder-only language model whose layers mix tokens either by lightning attention (a matrix state per head with a constant decay) or
by two mixers side by side, chunk-local softmax attention and gated linear attention.  A span of layers may run several times with the same weights, the
embedding output added to the stream before every pass but the first; every pass has a cache and states of its own.

This file reads the design's config.json and tensor names and assembles the mechanisms of ``layers.py`` into the serving protocol of ``serving.py``
(caches, step function, scheduler, sampling and command line are the framework's).  A step runs in one of two ways:

* prompts, large batches and float32: sublayer by sublayer from here (tile GEMMs, flash attention and linear attention on the matrix pipe, the fused stream
  pass);
* up to ``DECODE_ROWS`` single tokens in bf16: one C call (``aria_mix_decode``) that enqueues every kernel of every layer run."""
from __future__ import annotations

import ctypes
from dataclasses import dataclass, field
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from . import hip, ops
from .checkpoint import load_checkpoint_dir
from .layers import ChunkAttention, LinearAttention, MixerGroup, ReluGatedFeedForward, RmsNorm, _frozen, padded, up8
from .registry import read_config

bf16, f32 = torch.bfloat16, torch.float32
DECODE_ROWS = 16


@dataclass
class KozipelLayerConfig:
    kind: str
    mixer: dict
    mlp: Optional[dict]


@dataclass
class KozipelRun:
    """One run of a layer; ``again``: it opens a pass after the first, the embedding output is added in front of it."""

    layer: int
    again: bool = False


@dataclass
class KozipelConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    residual_mult: float
    logit_softcap: float
    layers: List[KozipelLayerConfig] = field(default_factory=list)
    runs: List[KozipelRun] = field(default_factory=list)

    @classmethod
    def from_dict(cls, c: dict) -> "KozipelConfig":
        layers = []
        for i, e in enumerate(c["layers"]):
            if e["type"] not in ("lightning", "parallel"):
                raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
            mlp = e.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            layers.append(KozipelLayerConfig(e["type"], e["mixer"], mlp))
        n, loop = len(layers), c.get("loop") or {"start": 0, "stop": 0, "times": 1}
        start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
        if not 0 <= start <= stop <= n or times < 1:
            raise ValueError(f"loop over layers {start} .. {stop - 1} of {n}, {times} times")
        runs = [KozipelRun(i) for i in range(start)]
        for p in range(times):
            runs += [KozipelRun(i, p > 0 and i == start) for i in range(start, stop)]
        runs += [KozipelRun(i) for i in range(stop, n)]
        return cls(int(c["vocab"]), int(c["width"]), float(c["norm"]["eps"]), float(c["embedding"]["scale"]), float(c["residual_mult"]),
                   float(c["logit_softcap"]), layers, runs)


class KozipelLayer(nn.Module):
    """Weights of one layer: the mixer, the feed-forward (or none), their norms."""

    def __init__(self, w: Dict[str, torch.Tensor], cfg: KozipelLayerConfig, width: int, eps: float, dtype):
        super().__init__()

        def part(prefix):
            return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}

        m = cfg.mixer
        if cfg.kind == "lightning":
            mix = LinearAttention(part("mix."), heads=m["heads"], dim=m["dim"], vdim=m["vdim"], decay=m["decay"], silu_inputs=True, norm_heads=False, gate="sigmoid",
                                  eps=eps, width=width, dtype=dtype)
            self.mixer = MixerGroup([mix], width, dtype=dtype)
        else:
            a, b = m["left"], m["right"]
            left = ChunkAttention(part("mix.left."), heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"], vdim=a["vdim"], size=int(a["mask"]["size"]),
                                  scale=float(a["scale"]), width=width, dtype=dtype)
            right = LinearAttention(part("mix.right."), heads=b["heads"], dim=b["dim"], vdim=b["vdim"], tau=float(b["tau"]), q_scale=b["dim"] ** -0.5, eps=eps,
                                    width=width, dtype=dtype)
            self.mixer = MixerGroup([left, right], width, [RmsNorm(w[f"mix.{side}.out"], width) for side in ("left", "right")], dtype=dtype)
        self.norm1, self.norm2, self.mlp = RmsNorm(w["norm1"], width, 1.0), None, None
        if cfg.mlp is not None:
            self.norm2 = RmsNorm(w["norm2"], width, 1.0)
            self.mlp = ReluGatedFeedForward(w["mlp.gate"], w["mlp.up"], w["mlp.down"], width, dtype)


class KozipelForCausalLM(nn.Module):
    """``from_pretrained`` / ``from_tensors`` -> a model with the serving protocol (``setup_caches``, ``step``, ``vocab``, ``device``)."""

    dtypes = (bf16, f32)

    def __init__(self, config: KozipelConfig, tensors: Dict[str, torch.Tensor], dtype=bf16):
        super().__init__()
        if dtype not in self.dtypes:
            raise TypeError(f"Kozipel computes in bf16 or float32, not {dtype}")
        self.config, self.dtype, self.vocab = config, dtype, config.vocab
        self.width = up8(config.width)       # columns behind the true width: their norm weights and projection rows are zeros, the norms do not count them
        self.layers = nn.ModuleList(KozipelLayer({k[len(f"l{i}."):]: v for k, v in tensors.items() if k.startswith(f"l{i}.")}, e, self.width, config.eps, dtype)
                                    for i, e in enumerate(config.layers))
        self.final = RmsNorm(tensors["final.norm"], self.width, 1.0)
        self.embed = _frozen(padded(tensors["embed"], config.vocab, self.width), dtype)
        self.head = _frozen(padded(tensors["head"], up8(config.vocab), self.width), dtype)
        self.caches: List[list] = []
        self.geometry = None
        self._decode: Optional["_DecodeTables"] = None

    @classmethod
    def from_tensors(cls, config: dict, tensors: Dict[str, torch.Tensor], device="cuda", dtype=bf16) -> "KozipelForCausalLM":
        return cls(KozipelConfig.from_dict(config), tensors, dtype).to(device).eval()

    @classmethod
    def from_pretrained(cls, path: str, device="cuda", dtype=bf16) -> "KozipelForCausalLM":
        return cls.from_tensors(read_config(path), load_checkpoint_dir(path), device, dtype)

    def _apply(self, fn, *a, **k):       # (the decode tables hold raw addresses)
        self._decode = None
        return super()._apply(fn, *a, **k)

    @property
    def device(self):
        return self.head.device

    def setup_caches(self, slots: int, max_len: int) -> None:
        """Caches and states per layer RUN (passes of a repeated layer do not share them)."""
        geometry = (slots, up8(max_len), self.device)
        if self.geometry == geometry:
            return                           # a sequence reads nothing that it has not written itself
        self.caches = [self.layers[r.layer].mixer.new_cache(slots, up8(max_len), self.device) for r in self.config.runs]
        self.geometry, self._decode = geometry, None

    def _stream(self, x, batch, i, nxt, **src):
        """the stream pass behind a sublayer of run i that ends it: the next run's pass opening included"""
        c = self.config
        again = i + 1 < len(c.runs) and c.runs[i + 1].again
        emb = dict(ids=batch.ids, table=self.embed, scale=c.embedding_scale) if again else {}
        return ops.rms_stream(x, c.width, c.eps, nxt.weight, mult=c.residual_mult, **emb, **src)

    def next_norm(self, i: int) -> RmsNorm:
        """the norm that reads the stream after layer run i"""
        runs = self.config.runs
        return self.layers[runs[i + 1].layer].norm1 if i + 1 < len(runs) else self.final

    @torch.no_grad()
    def step(self, batch, trace: Optional[list] = None) -> torch.Tensor:
        """Run a ``serving.StepBatch``; -> float32 logits [wanted rows, vocab].  ``trace``: receives the residual stream after every layer run."""
        if not self.caches:
            raise RuntimeError("setup_caches() first")
        slots, max_len, _ = self.geometry
        if batch.max_len > max_len or max(batch.slots) >= slots:
            raise ValueError("the batch does not fit the caches")
        c, T = self.config, batch.ids.numel()
        if self.dtype == bf16 and trace is None and batch.longest == 1 and T <= DECODE_ROWS and all(L.mixer.one_call for L in self.layers):
            if self._decode is None:
                self._decode = _DecodeTables(self)
            logits = self._decode.run(batch)
            return logits if batch.wanted is None or batch.wanted.numel() == T else logits[batch.wanted.long()]
        x = torch.empty((T, self.width), dtype=f32, device=self.device)
        h = ops.rms_stream(x, c.width, c.eps, self.layers[c.runs[0].layer].norm1.weight, ids=batch.ids, table=self.embed, scale=c.embedding_scale)
        for i, run in enumerate(c.runs):
            L = self.layers[run.layer]
            src = L.mixer(h, batch, self.caches[i])
            if L.mlp is not None:
                src = L.mlp(ops.rms_stream(x, c.width, c.eps, L.norm2.weight, mult=c.residual_mult, **src))
            if trace is not None:      # (what is added in front of a later pass is not part of the layer)
                before = x.clone()
                ops.rms_stream(before, c.width, c.eps, None, mult=c.residual_mult, **src)
                trace.append(before)
            h = self._stream(x, batch, i, self.next_norm(i), **src)
        if batch.wanted is not None:
            if batch.wanted.numel() == 0:
                return torch.empty((0, self.vocab), dtype=f32, device=self.device)
            h = ops.permute_any(h, batch.wanted.contiguous(), 1)
        return ops.softcap_(ops.linear_any(h, self.head, out_dtype=f32), c.logit_softcap)[:, :self.vocab]


class _DecodeTables:
    """Pointer and size tables of ``aria_mix_decode`` for a model's weights and caches (re-made when either moves), scratch and logits buffers."""

    def __init__(self, model: KozipelForCausalLM):
        c = model.config
        n = len(c.runs)
        self.runs = (hip.MixLayer * n)()
        self.scratch: Optional[torch.Tensor] = None
        for i, run in enumerate(c.runs):
            L, t = model.layers[run.layer], self.runs[i]
            L.mixer.fill_table(t, model.caches[i])
            if L.mlp is not None:
                gate = L.mlp.gate_up[:L.mlp.ff]
                t.norm2, t.ff, t.w_gate, t.w_up = L.norm2.weight.data_ptr(), L.mlp.ff, gate.data_ptr(), L.mlp.gate_up[L.mlp.ff:].data_ptr()
                t.w_down = L.mlp.down.data_ptr()
            t.next = model.next_norm(i).weight.data_ptr()
            t.next_embedding = int(i + 1 < n and c.runs[i + 1].again)
        self.stack = hip.MixStack(n, model.width, c.width, model.head.shape[0], c.embedding_scale, c.residual_mult, c.eps, c.logit_softcap,
                                  model.layers[c.runs[0].layer].norm1.weight.data_ptr(), model.embed.data_ptr(), model.head.data_ptr())
        self.device, self.rows, self.vocab = model.device, model.head.shape[0], model.vocab

    def run(self, batch) -> torch.Tensor:
        T, lib = batch.ids.numel(), hip.get_lib()
        stack, runs = ctypes.byref(self.stack), ctypes.byref(self.runs)
        need = int(lib.cdll.aria_mix_decode_scratch(stack, runs, T, batch.max_len))
        if self.scratch is None or self.scratch.numel() < need:
            self.scratch = torch.empty(need, dtype=torch.uint8, device=self.device)
        logits = torch.empty((T, self.rows), dtype=f32, device=self.device)
        for t in (batch.ids, batch.slot, batch.pos):
            assert t.dtype == torch.int32 and t.is_contiguous() and t.numel() == T
        lib.call("aria_mix_decode", stack, runs, T, batch.ids.data_ptr(), batch.slot.data_ptr(), batch.pos.data_ptr(), batch.max_len,
                 logits.data_ptr(), self.scratch.data_ptr(), self.scratch.numel(), ops._stream(logits))
        return logits[:, :self.vocab]
