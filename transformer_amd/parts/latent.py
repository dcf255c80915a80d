"""Attention over one cached latent row per token (``LatentAttentionSpec``).

The cache layer holds, per token, the normed latent c [kv_rank] and the rotated key part
[rope_dim] that all heads share: one "kv head" of keys only. The heads' key and value maps are
applied to the queries and to the attention's result instead of to the cached rows:

    qa_h = [Uk_h^T q_h(unrotated) | rotated q_h]      score = qa_h . [c | shared part] * scale
    out_h = Uv_h (sum_j p_j c_j) * sigmoid(g_h . h)

so a step reads kv_rank + rope_dim numbers per cached token whatever the number of heads, and
nothing is expanded per cached token. The first product of a step joins the query latent's
map (or the queries' own, where they have no latent), the key/value latent's map and the heads'
gates.
"""
from __future__ import annotations

import torch

from .. import kernels
from ..cache.storage import KVNeed
from ..config.spec import PositionSpec
from ..weights.loader import Param
from .base import Part, PartError, build_part, register_part
from .linear import adds_in_place, aligned_rows, finish, linear


class LatentAttention(Part):
    graph_safe = True

    def __init__(self, spec, dtype, device):
        s = spec
        q_rank = 1 if s.q_rank is None else s.q_rank
        if min(s.num_heads, s.nope_dim + s.rope_dim, s.value_dim, q_rank, s.kv_rank) < 1 or s.rope_dim < 0 \
                or s.nope_dim < 0:
            raise PartError(f"latent attention: heads {s.num_heads} of {s.nope_dim} + {s.rope_dim} / "
                            f"{s.value_dim}, ranks {s.q_rank} / {s.kv_rank}")
        if s.rot_dims % 2 or not 0 <= s.rot_dims <= s.rope_dim:
            raise PartError(f"{s.rot_dims} rotated coordinates do not fit a part of {s.rope_dim}")
        if s.kv_rank > kernels.LATENT_MAX_RANK or s.rope_dim > kernels.LATENT_MAX_RANK:
            raise PartError(f"latent attention takes latents and rotated parts up to {kernels.LATENT_MAX_RANK}, "
                            f"not {s.kv_rank} / {s.rope_dim}")
        for w in (s.window, s.cache_window):
            if w is not None and w < 1:
                raise PartError(f"attention window must be >= 1, got {w}")
        if s.cache_window is not None and (s.window is None or s.window > s.cache_window):
            raise PartError(f"a window of {s.window} reads past the {s.cache_window} tokens its cache keeps")
        self.spec, self.dtype = s, dtype
        self.H, self.dn, self.dr, self.dv = s.num_heads, s.nope_dim, s.rope_dim, s.value_dim
        self.kv_off = self.H * (self.dn + self.dr) if s.q_rank is None else s.q_rank
        self.gate_off = self.kv_off + (s.kv_rank + s.rope_dim if s.own_kv else 0)
        self.width = self.gate_off + (self.H if s.gated else 0)
        self.row = kernels.latent_row_width(s.kv_rank, s.rope_dim, dtype)      # a cached row, a wide query
        self.rotary = None
        if s.rot_dims:
            self.rotary = build_part(PositionSpec(head_dim=s.rot_dims, theta=s.rot_base, style="interleaved"),
                                     dtype, device)

    def params(self):
        s = self.spec
        # queries or their latent, kv latent + shared key part, gates
        p = {"in.weight": Param((self.width, s.hidden), "matrix"),
             "uk.weight": Param((self.H * self.dn, s.kv_rank), "matrix"),
             "uv.weight": Param((self.H * self.dv, s.kv_rank), "matrix"),
             "out.weight": Param((s.hidden, self.H * self.dv), "matrix")}
        if s.q_rank is not None:
            p["q_norm.weight"] = Param((s.q_rank,), "vector", init="around_one")
            p["uq.weight"] = Param((self.H * (self.dn + self.dr), s.q_rank), "matrix")
        if s.own_kv:
            p["kv_norm.weight"] = Param((s.kv_rank,), "vector", init="around_one")
        if s.sink:
            p["sink"] = Param((self.H,), "vector", init="zero")
        return p

    def cache_need(self):
        s = self.spec
        return KVNeed(1, self.row, s.cache_window, 0)

    def bind(self, tensors):
        super().bind(tensors)
        s = self.spec
        # per head: Uk^T and Uv as right operands. The framework's own product reads [N, K], the library's
        # (bfloat16) a contiguous [K, N]
        def packed(t):                      # contiguous strides also where an axis has one entry
            return torch.empty(t.shape, dtype=t.dtype, device=t.device).copy_(t)

        uk = tensors["uk.weight"].view(self.H, self.dn, s.kv_rank) if self.dn else None     # [K, N] of Uk^T
        uv = tensors["uv.weight"].view(self.H, self.dv, s.kv_rank)                          # [N, K]
        self.uk_op = None if uk is None else uk if self._by_library(uk) else packed(uk.transpose(1, 2))
        self.uv_op = packed(uv.transpose(1, 2)) if self._by_library(uv) else uv

    def _by_library(self, w) -> bool:
        return self.dtype == torch.bfloat16 and w.dtype == torch.bfloat16

    def _per_head(self, a, w, out):
        """out[:, h] = a[:, h] times the h-th right operand (``bind``): a [nt, H, K], out [nt, H, N]."""
        if not self._by_library(w):
            return kernels.gemm_simple_batched(a.transpose(0, 1), w, out.transpose(0, 1))
        torch.bmm(a.transpose(0, 1), w, out=out.transpose(0, 1))
        return out

    # with many rows the output projection can add itself to the residual stream (``into``); in
    # single-token steps the norms around the mixer ride on its products (``PreNormBlock``)
    def can_add(self, nt: int) -> bool:
        return adds_in_place(nt, self.w["out.weight"])

    def takes_scaled(self, nt: int) -> bool:
        return kernels.skinny_takes(nt, self.w["in.weight"])

    def can_fold(self, nt: int) -> bool:
        return kernels.skinny_folds(nt, self.w["out.weight"])

    def run(self, h, ctx, cache, layer, writes_cache=True, scale=None, fold=None, into=None):
        s, nt, H = self.spec, h.shape[0], self.H
        r, dr = s.kv_rank, self.dr
        if writes_cache != s.own_kv:
            raise PartError("a latent attention layer stores rows exactly when it forms them itself: "
                            "its schedule entry and its spec disagree")
        proj = linear(h, self.w["in.weight"], aligned_rows(ctx.ws, "latent.in", nt, self.width, self.dtype), scale=scale)
        kc, _, group = cache.layer_kv(layer)
        meta = ctx.kv[group]
        angles = self.rotary.angles(ctx) if self.rotary is not None else None
        cq = ctx.ws.take("latent.cq", (nt, s.q_rank), self.dtype) if s.q_rank is not None else None
        if cq is not None or s.own_kv:
            kernels.latent_prepare(proj, s.q_rank or 0, self.w.get("q_norm.weight"), cq, self.kv_off, r, dr, s.rot_dims,
                                   self.w.get("kv_norm.weight"), float(s.eps), angles,
                                   meta.dest if s.own_kv else None, kc if s.own_kv else None)
        if cq is not None:
            q = linear(cq, self.w["uq.weight"], ctx.ws.take("latent.q", (nt, H * (self.dn + dr)), self.dtype))
        else:
            q = proj[:, :self.kv_off]
        qa = ctx.ws.take("latent.qa", (nt, H, self.row), self.dtype)
        kernels.latent_query_rot(q, H, self.dn, dr, s.rot_dims, angles, qa, r)
        if self.dn:
            self._per_head(q.unflatten(1, (H, self.dn + dr))[:, :, :self.dn], self.uk_op, qa[:, :, :r])
        else:
            qa[:, :, :r].zero_()
        ol = ctx.ws.take("latent.ol", (nt, H, r), self.dtype)
        shares = kernels.latent_key_shares(ctx.batch, ctx.max_qlen, H, r, self.row, ctx.max_kv_len, s.window)
        kernels.latent_attention(qa, ol, kc, meta.block_table, ctx.cu_q, ctx.pos0, ctx.max_qlen, r, dr,
                                 float(s.scale), s.window,
                                 gate=proj[:, self.gate_off:] if s.gated else None, shares=shares,
                                 sink=self.w.get("sink"))
        o = ctx.ws.take("latent.o", (nt, H, self.dv), self.dtype)
        self._per_head(ol, self.uv_op, o)
        return finish(o.view(nt, H * self.dv), self.w["out.weight"], ctx.ws, "latent.delta", fold, into)


register_part("latent_attention", LatentAttention)
