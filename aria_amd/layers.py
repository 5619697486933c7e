"""Decoder mechanisms beside the ones of ``gptfast.py``, each a module whose sizes and constants are arguments:

* ``DynamicTanh`` -- a norm without statistics, tanh(alpha x) w + b; elementwise, so it always runs inside a pass over the fp32 residual stream
  (``ops.dyt_stream``) or a projection's epilogue, never as a launch of its own;
* ``LatentAttention`` + ``LatentCache`` -- keys and values as images of one low-rank latent per token, a rotated key part shared by the heads, a
  sigmoid output gate per head;
* ``SquaredReluFeedForward``; ``GroupLimitedMixture`` -- sigmoid router with a choice correction and group-limited top-k.

Weights are held the way the kernels read them (padded, projections that share an input in one matrix) and packed once at load.  Modules exist in
bf16 and in float32 (``dtype``); the float32 form runs the 32-bit kernels throughout."""
from __future__ import annotations

from typing import List, Optional

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
