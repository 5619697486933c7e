"""Decoder mechanisms beside the ones of ``gptfast.py``, each a module whose sizes and constants are arguments:

* ``DynamicTanh`` -- a norm without statistics, tanh(alpha x) w + b; elementwise, so it always runs inside a pass over the fp32 residual stream
  (``ops.dyt_stream``) or a projection's epilogue, never as a launch of its own;
* ``LatentAttention`` + ``LatentCache`` -- keys and values as images of one low-rank latent per token, a rotated key part shared by the heads, a
  sigmoid output gate per head;
* ``SquaredReluFeedForward``; ``GroupLimitedMixture`` -- sigmoid router with a choice correction and group-limited top-k;
* ``RmsNorm`` -- its weight as a factor, evaluated inside a pass over the residual stream (``ops.rms_stream``);
* ``ChunkAttention`` + ``ChunkCache`` -- grouped-query attention inside chunks of positions; ``LinearAttention`` + ``LinearState`` -- a decaying matrix
  state per head, the decay constant or gated; ``MixerGroup`` -- mixers that read the same input side by side, their projections one matrix;
* ``ReluGatedFeedForward``.

Weights are held the way the kernels read them (padded, projections that share an input in one matrix) and packed once at load.  Modules exist in
bf16 and in float32 (``dtype``); the float32 form runs the 32-bit kernels throughout."""
from __future__ import annotations

import math
from typing import List, Optional, Sequence

import torch
import torch.nn as nn

from . import hip, ops
from .gptfast import _glu_pair_ready

bf16, f32 = torch.bfloat16, torch.float32


def up8(n: int) -> int:
    return (n + 7) // 8 * 8


def padded(t: torch.Tensor, *shape: int) -> torch.Tensor:
    """``t`` in the corner of a zero tensor of ``shape``."""
    out = torch.zeros(shape, dtype=t.dtype, device=t.device)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


def _frozen(t: torch.Tensor, dtype) -> nn.Parameter:
    return nn.Parameter(t.to(dtype).contiguous(), requires_grad=False)


class DynamicTanh(nn.Module):
    """tanh(alpha x) w + b with scalar alpha; parameters in float32 (norms are evaluated in 32-bit)."""

    def __init__(self, alpha: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor, dim: int):
        super().__init__()
        self.alpha = float(alpha)
        self.weight, self.bias = _frozen(padded(weight, dim), f32), _frozen(padded(bias, dim), f32)

    def params(self) -> hip.DyTParams:
        return hip.DyTParams(self.alpha, self.weight.data_ptr(), self.bias.data_ptr())


def rotation_table(positions: int, dims: int, base: float, device) -> torch.Tensor:
    """(cos, sin) of p base^(-2 i / dims), fp32 [positions, dims / 2, 2]; angles from float64."""
    f = base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)
    a = torch.arange(positions, dtype=torch.float64)[:, None] * f[None, :]
    return torch.stack([torch.cos(a), torch.sin(a)], -1).to(f32).to(device).contiguous()


class LatentCache:
    """One layer's static cache of latents: [slots, max length, row], row = [latent | rotated key part | zeros], a multiple of 64 columns (the decode
    kernel streams whole rows).  A slot belongs to one sequence; rows behind its position are never read."""

    def __init__(self, slots: int, max_len: int, row: int, dtype, device):
        self.rows = torch.zeros((slots, max_len, row), dtype=dtype, device=device)


class LatentAttention(nn.Module):
    """Latent attention with H heads of ``dim`` unrotated + ``rot_dim`` rotated query / key columns and ``vdim`` value columns over a latent of
    ``kv_rank``.  ``w``: the checkpoint's tensors q, dkv, dkv.norm, uk, uv, g, o (each [out, in])."""

    def __init__(self, w, *, heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, scale: float, rot_dims: int, rot_base: float, eps: float,
                 width: int, dtype=bf16):
        super().__init__()
        H, qd = heads, dim + rot_dim
        fused = ops.varlen_head(qd, vdim) if dtype == bf16 else None
        dq, dvp = fused or (up8(qd), up8(vdim))
        self.flash = fused is not None
        self.rot_dims, self.rot_base, self.dtype = rot_dims, rot_base, dtype
        cw, rp = (kv_rank + rot_dim + 63) // 64 * 64, up8(kv_rank)
        kv_off = H * dq
        g_off = kv_off + up8(kv_rank + rot_dim)
        ldp = g_off + up8(H)
        self.geometry = dict(H=H, dn=dim, dr=rot_dim, dv=vdim, R=kv_rank, rot=rot_dims, dq=dq, dvp=dvp, cw=cw, rp=rp, ldp=ldp, kv_off=kv_off, g_off=g_off,
                             scale=scale, eps=eps)
        D, like = w["q"].shape[1], dict(dtype=w["q"].dtype, device=w["q"].device)
        w_in = torch.zeros((ldp, width), **like)
        w_in[:kv_off].view(H, dq, width)[:, :qd, :D] = w["q"].view(H, qd, D)
        w_in[kv_off:kv_off + kv_rank + rot_dim, :D] = w["dkv"]
        w_in[g_off:g_off + H, :D] = w["g"]
        uk, uv = w["uk"].view(H, dim, kv_rank), w["uv"].view(H, vdim, kv_rank)
        w_o = torch.zeros((width, H, dvp), **like)
        w_o[:w["o"].shape[0], :, :vdim] = w["o"].view(-1, H, vdim)
        self.w_in, self.w_o = _frozen(w_in, dtype), _frozen(w_o.view(width, H * dvp), dtype)
        self.w_uk, self.w_uv = _frozen(padded(uk, H, dim, rp).view(H * dim, rp), dtype), _frozen(padded(uv, H, vdim, rp).view(H * vdim, rp), dtype)
        self.kv_norm = _frozen(w["dkv.norm"], f32)
        self.w_kv: Optional[nn.Parameter] = None
        if self.flash:
            # one cache row -> every head's padded key and value: the rotated part passes through identity rows
            kv = torch.zeros((H * (dq + dvp), cw), **like)
            keys, vals = kv[:H * dq].view(H, dq, cw), kv[H * dq:].view(H, dvp, cw)
            keys[:, :dim, :kv_rank], vals[:, :vdim, :kv_rank] = uk, uv
            keys[:, dim:qd, kv_rank:kv_rank + rot_dim] = torch.eye(rot_dim, **like)
            self.w_kv = _frozen(kv, dtype)

    def shape(self, S_cap: int) -> hip.LatentShape:
        return hip.LatentShape(S_cap=S_cap, **self.geometry)

    def new_cache(self, slots: int, max_len: int, device) -> LatentCache:
        return LatentCache(slots, max_len, self.geometry["cw"], self.dtype, device)

    def forward(self, h: torch.Tensor, batch, cache: LatentCache, rope: torch.Tensor) -> torch.Tensor:
        """h [T, D] normed input of the batch's tokens (``serving.StepBatch``) -> [T, D]."""
        g, s = self.geometry, self.shape(cache.rows.shape[1])
        proj = ops.linear_any(h, self.w_in)
        if batch.fresh and batch.longest > 1 and self.flash:
            # whole prompts: expand the new latents, flash attention over the packed sequences
            packed = ops.latent_rows(s, proj, batch.slot, batch.pos, rope, self.kv_norm, cache.rows)
            kv = ops.gemm(packed, self.w_kv)
            n = g["H"] * g["dq"]
            o = ops.attention_varlen(proj[:, :n], kv[:, :n], kv[:, n:], batch.cu, batch.longest, g["H"], g["dq"], g["dvp"], g["scale"],
                                     gate=proj[:, g["g_off"]:])
        else:
            o = ops.latent_decode_attention(s, proj, batch.slot, batch.pos, rope, self.kv_norm, self.w_uk, self.w_uv, cache.rows, batch.max_len)
        return ops.linear_any(o, self.w_o)


class SquaredReluFeedForward(nn.Module):
    """W_down relu(W_up h)^2."""

    def __init__(self, up: torch.Tensor, down: torch.Tensor, width: int, dtype=bf16):
        super().__init__()
        self.ff = up8(up.shape[0])
        self.up, self.down = _frozen(padded(up, self.ff, width), dtype), _frozen(padded(down, width, self.ff), dtype)

    def forward(self, h: torch.Tensor):
        return dict(y=ops.linear_any(ops.linear_any(h, self.up, relu_squared=True), self.down))


class GroupLimitedMixture(nn.Module):
    """``top`` of E experts W_down (silu(W_gate h) * (W_up h)); sigmoid scores, chosen by score + correction among the ``keep`` best of ``groups``
    equal groups, weighted by the plain scores.  forward returns the expert rows with their index and weights: the weighted sum belongs to the
    stream pass that follows."""

    def __init__(self, gate: List[torch.Tensor], up: List[torch.Tensor], down: List[torch.Tensor], router: torch.Tensor, correction: torch.Tensor, *,
                 top: int, groups: int, keep: int, width: int, dtype=bf16):
        super().__init__()
        E, F = len(gate), up8(gate[0].shape[0])
        if E > 256 or E % groups or not 0 < keep <= groups or not 0 < top <= min(64, keep * (E // groups)):
            raise ValueError(f"routing of {E} experts in {groups} groups, {keep} kept, top {top}")
        self.ff, self.top, self.groups, self.keep, self.n_experts = F, top, groups, keep, E
        pair = torch.stack([torch.stack([padded(t, F, width) for t in ts]) for ts in (gate, up)])   # one allocation: the fused launch's layout
        self.gate_up = _frozen(pair, dtype)
        self.down = _frozen(torch.stack([padded(t, width, F) for t in down]), dtype)
        self.router = _frozen(padded(router, up8(E), width), dtype)
        self.correction = _frozen(correction, f32)

    @property
    def gate(self):
        return self.gate_up[0]

    @property
    def up(self):
        return self.gate_up[1]

    def forward(self, h: torch.Tensor):
        logits = ops.linear_any(h, self.router, out_dtype=f32)
        weights, idx, counts = ops.moe_route_groups(logits, self.correction, self.groups, self.keep, self.top)
        offsets, sorted_src, inv = ops.moe_sort(idx, counts)
        g, u = self.gate, self.up
        if h.dtype == bf16 and ops.gather_fusable(h.shape[1]) and _glu_pair_ready(g, u):
            act = ops.grouped_gemm_swiglu_split_gather(h, ops.permuted_token_rows(sorted_src, self.top), g, u, offsets)[1]
        else:
            rows = ops.permute_any(h, sorted_src, self.top)
            act = ops.act_rows(ops.grouped_linear_any(rows, u, offsets), gate=ops.grouped_linear_any(rows, g, offsets))
        return dict(y=ops.grouped_linear_any(act, self.down, offsets), inv=inv, weights=weights)


class RmsNorm(nn.Module):
    """x / sqrt(mean(x^2) + eps) (weight + offset): the factor in float32, zeros behind the true width."""

    def __init__(self, weight: torch.Tensor, width: int, offset: float = 0.0):
        super().__init__()
        self.weight = _frozen(padded(weight.float() + offset, width), f32)


class ChunkCache:
    """One layer's static cache of chunk-local attention: [slots, kv heads, rows, key | value].  A sequence holds ONE chunk, position p in row p % size;
    rows behind its position in the chunk are never read."""

    def __init__(self, slots: int, max_len: int, heads: int, size: int, width: int, dtype, device):
        self.rows = torch.zeros((slots, heads, min(size, max_len), width), dtype=dtype, device=device)


class ChunkAttention(nn.Module):
    """Grouped-query softmax attention without positions, position i seeing the j <= i of its own chunk of ``size``.  ``w``: the checkpoint's tensors
    q, k, v, o.  The input projection's rows are ``w_in`` until a ``MixerGroup`` takes them."""

    def __init__(self, w, *, heads: int, kv_heads: int, dim: int, vdim: int, size: int, scale: float, width: int, dtype=bf16):
        super().__init__()
        if heads % kv_heads or size < 1:
            raise ValueError(f"{heads} query heads over {kv_heads} key heads in chunks of {size}")
        fused = ops.varlen_head(dim, vdim) if dtype == bf16 else None
        dq, dvp = fused or (up8(dim), up8(vdim))
        self.flash, self.dtype = fused is not None, dtype
        D = w["q"].shape[1]
        self.w_in = [padded(w["q"].view(heads, dim, D), heads, dq, D).view(-1, D), padded(w["k"].view(kv_heads, dim, D), kv_heads, dq, D).view(-1, D),
                     padded(w["v"].view(kv_heads, vdim, D), kv_heads, dvp, D).view(-1, D)]
        self.geometry = dict(H=heads, G=kv_heads, dq=dq, dvp=dvp, size=size, scale=scale)
        self.w_o = _frozen(padded(w["o"].view(-1, heads, vdim), width, heads, dvp).view(width, heads * dvp), dtype)

    def placed(self, offsets: Sequence[int], ldp: int) -> None:
        self.geometry.update(zip(("q_off", "k_off", "v_off"), offsets), ldp=ldp)

    def shape(self, cache: ChunkCache) -> hip.ChunkShape:
        return hip.ChunkShape(cap=cache.rows.shape[2], **self.geometry)

    def new_cache(self, slots: int, max_len: int, device) -> ChunkCache:
        g = self.geometry
        return ChunkCache(slots, max_len, g["G"], g["size"], g["dq"] + g["dvp"], self.dtype, device)

    def forward(self, proj: torch.Tensor, batch, cache: ChunkCache) -> torch.Tensor:
        g, s = self.geometry, self.shape(cache)
        if batch.fresh and batch.longest > 1 and self.flash:
            # whole prompts: every chunk is a sequence of its own
            cu, longest = batch.chunks(g["size"])
            q, k, v = (proj[:, g[n]:] for n in ("q_off", "k_off", "v_off"))
            o = ops.attention_varlen(q, k, v, cu, longest, g["H"], g["dq"], g["dvp"], g["scale"], kv_heads=g["G"])
            ops.chunk_rows(s, proj, cache.rows, batch)
        elif batch.longest == 1 and self.flash:
            o = ops.chunk_attention_decode(s, proj, cache.rows, batch)
        else:
            o = ops.chunk_attention_any(s, proj, cache.rows, batch)
        return ops.linear_any(o, self.w_o)


class LinearState:
    """One layer's recurrent states, float32 [slots, heads, key, value]; a sequence at position 0 starts from zeros whatever its slot holds."""

    def __init__(self, slots: int, heads: int, dim: int, vdim: int, device):
        self.rows = torch.zeros((slots, heads, dim, vdim), dtype=f32, device=device)


class LinearAttention(nn.Module):
    """S_t = diag(a_t) S_(t-1) + k_t v_t^T, o_t = q_scale S_t^T q_t per head, then an RMS norm (per head with a shared weight, or over all heads) and an
    output gate.  Decay: ``decay``, a constant per head; or, without it, gated per key channel: sigmoid(a2 (a1 h) + a2.b)^(1 / tau).  ``w``: the
    checkpoint's tensors q, k, v, g, o, norm (a1, a2, a2.b)."""

    def __init__(self, w, *, heads: int, dim: int, vdim: int, decay: Optional[Sequence[float]] = None, tau: float = 1.0, q_scale: float = 1.0, silu_inputs: bool = False,
                 norm_heads: bool = True, gate: str = "silu", eps: float, width: int, dtype=bf16):
        super().__init__()
        self.chunked = dtype == bf16 and dim <= 256
        dp = next(n for n in (64, 128, 256) if n >= dim) if self.chunked else up8(dim)
        dvp = (vdim + 63) // 64 * 64 if self.chunked else up8(vdim)
        self.eps, self.dtype, self.silu_gate = eps, dtype, {"silu": True, "sigmoid": False}[gate]
        D = w["q"].shape[1]

        def rows(name, n, to):
            return padded(w[name].view(heads, n, D), heads, to, D).view(-1, D)

        self.w_in = [rows("q", dim, dp), rows("k", dim, dp), rows("v", vdim, dvp), rows("g", vdim, dvp)]
        self.geometry = dict(H=heads, d=dim, dv=vdim, dp=dp, dvp=dvp, rank=0, silu=int(silu_inputs), q_scale=q_scale, inv_tau=1.0 / tau)
        self.decay = self.a2 = self.a_bias = None
        if decay is not None:
            if len(decay) != heads or min(decay) < 0:
                raise ValueError(f"{len(decay)} decays for {heads} heads")
            self.decay = _frozen(torch.tensor([[a, math.log2(a) if a > 0 else -math.inf] for a in decay], dtype=torch.float64), f32)
        else:
            rank = up8(w["a1"].shape[0])
            self.w_in.append(padded(w["a1"], rank, D))
            self.geometry["rank"] = rank
            self.a2 = _frozen(padded(w["a2"].view(heads, dim, -1), heads, dp, rank).view(heads * dp, rank), dtype)
            self.a_bias = _frozen(padded(w["a2.b"].view(heads, dim), heads, dp).view(-1), f32)
        self.norm_groups, self.norm_n = (heads, vdim) if norm_heads else (1, heads * vdim)
        norm = w["norm"].view(-1, vdim)
        self.norm = _frozen(padded(norm, norm.shape[0], dvp).view(-1), f32)
        self.w_o = _frozen(padded(w["o"].view(-1, heads, vdim), width, heads, dvp).view(width, heads * dvp), dtype)

    def placed(self, offsets: Sequence[int], ldp: int) -> None:
        self.geometry.update(zip(("q_off", "k_off", "v_off"), offsets), ldp=ldp, a_off=offsets[4] if len(offsets) > 4 else 0)
        self.g_off = offsets[3]

    def shape(self) -> hip.LinearShape:
        ptr = {n: t.data_ptr() for n, t in (("decay", self.decay), ("a2", self.a2), ("a_bias", self.a_bias)) if t is not None}
        return hip.LinearShape(**self.geometry, **ptr)

    def new_cache(self, slots: int, max_len: int, device) -> LinearState:
        g = self.geometry
        return LinearState(slots, g["H"], g["dp"], g["dvp"], device)

    def forward(self, proj: torch.Tensor, batch, cache: LinearState) -> torch.Tensor:
        run = ops.linear_chunks if self.chunked and batch.longest > 1 else ops.linear_step
        o = run(self.shape(), proj, cache.rows, batch)
        o = ops.norm_gate(o, proj[:, self.g_off:self.g_off + o.shape[1]], self.norm, self.norm_groups, self.norm_n, self.eps, self.silu_gate)
        return ops.linear_any(o, self.w_o)


class MixerGroup(nn.Module):
    """One mixer, or two side by side that read the same input: one input projection for all.  Two: the result is the half-sum of their outputs, each
    RMS-normed with its plain weight -- a step of the stream pass that follows, so forward returns that pass's operands."""

    def __init__(self, parts: Sequence[nn.Module], width: int, out_norms: Sequence[RmsNorm] = (), dtype=bf16):
        super().__init__()
        if len(parts) != max(1, len(out_norms)) or len(parts) > 2:
            raise ValueError(f"{len(parts)} mixers with {len(out_norms)} output norms")
        blocks = [b for p in parts for b in p.w_in]
        starts = [0]
        for b in blocks:
            starts.append(starts[-1] + up8(b.shape[0]))
        w_in = torch.zeros((starts[-1], width), dtype=blocks[0].dtype, device=blocks[0].device)
        for b, at in zip(blocks, starts):
            w_in[at:at + b.shape[0], :b.shape[1]] = b
        for p in parts:
            p.placed(starts[:len(p.w_in)], w_in.shape[0])
            starts = starts[len(p.w_in):]
            del p.w_in
        self.w_in = _frozen(w_in, dtype)
        self.parts, self.out_norms = nn.ModuleList(parts), nn.ModuleList(out_norms)

    def new_cache(self, slots: int, max_len: int, device) -> list:
        return [p.new_cache(slots, max_len, device) for p in self.parts]

    @property
    def one_call(self) -> bool:
        """aria_mix_decode takes the group: linear attention alone (one norm over all heads, a sigmoid gate), or chunk attention beside linear attention (a
        norm per head, a silu gate), in widths of its kernels."""
        lin = self.parts[-1]
        if self.w_in.dtype != bf16 or not isinstance(lin, LinearAttention) or lin.geometry["dp"] > 1024:
            return False
        if len(self.parts) == 1:
            return lin.norm_groups == 1 and not lin.silu_gate
        return isinstance(self.parts[0], ChunkAttention) and self.parts[0].flash and lin.norm.numel() == lin.geometry["dvp"] and lin.silu_gate

    def fill_table(self, t: hip.MixLayer, caches: list) -> None:
        lin = self.parts[-1]
        t.kind, t.right, t.g_off, t.w_in, t.w_o = len(self.parts) - 1, lin.shape(), lin.g_off, self.w_in.data_ptr(), lin.w_o.data_ptr()
        t.norm, t.state = lin.norm.data_ptr(), caches[-1].rows.data_ptr()
        if len(self.parts) == 2:
            t.left, t.w_o_left, t.ring = self.parts[0].shape(caches[0]), self.parts[0].w_o.data_ptr(), caches[0].rows.data_ptr()
            t.out_left, t.out_right = (n.weight.data_ptr() for n in self.out_norms)

    def forward(self, h: torch.Tensor, batch, caches: list) -> dict:
        proj = ops.linear_any(h, self.w_in)
        y = [p(proj, batch, c) for p, c in zip(self.parts, caches)]
        if len(y) == 1:
            return dict(y=y[0])
        return dict(y=y[0], pair=(y[1], self.out_norms[0].weight, self.out_norms[1].weight))


class ReluGatedFeedForward(nn.Module):
    """W_down (max(W_gate h, 0) * (W_up h)); gate and up rows in one matrix."""

    def __init__(self, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, width: int, dtype=bf16):
        super().__init__()
        self.ff = up8(up.shape[0])
        self.gate_up = _frozen(torch.cat([padded(t, self.ff, width) for t in (gate, up)]), dtype)
        self.down = _frozen(padded(down, width, self.ff), dtype)

    def forward(self, h: torch.Tensor) -> dict:
        return dict(y=ops.linear_any(ops.relu_glu(h, self.gate_up), self.down))
