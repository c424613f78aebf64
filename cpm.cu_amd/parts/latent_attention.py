"""Latent attention: keys and values of all heads come from one small latent vector per token.

Per token, a down projection gives kv_rank + rot_dim numbers: the first kv_rank, RMS-normed with a weight, are
the latent c; the last rot_dim are one rotated key part shared by all heads.  Head h's key is
[W_uk[h] c | rotated part], its value W_uv[h] c; its query is [q_plain (key_dim) | q_rot (rot_dim)] and the
score (q_plain . W_uk[h] c + q_rot . k_rot) * scale.  Only c and the rotated key part are cached.

The cache is read without expanding it: q_plain . (W_uk[h] c) = (W_uk[h]^T q_plain) . c, so the query is taken
into the latent space once per token and head, attention runs with one cached "head" of kv_rank + rot_dim
key features and kv_rank value features shared by all query heads, and W_uv[h] is applied to the attention's
output instead of to every cached token.  (The cache holds c twice, in the key and in the value layout of the
matrix cores' operands.)  Softmax in float, causal or over a sliding window (``mask_window``: the token itself and the
window - 1 before it; the cache then gives older pages back), optionally with a sink, exp(sink[h]) as a further term of
the denominator; an output gate sigmoid(W_g x), one number a head or one a value feature, read from the mixer's input;
output projection on the concatenated heads.

The queries are a projection of the mixer's input, or (``q_rank``) come from a latent of their own: c_q = rmsnorm(W_dq x)
with a weight, q = W_uq c_q.

A layer may read the latent cache that another layer wrote (``shares_cache``): it has no down projection and
brings its own W_uk, W_uv, queries and everything else.
"""
from __future__ import annotations

from typing import List, Mapping, Optional

import torch

from .. import ops
from ..cache.paged import CacheNeeds, CacheView, StreamSpec
from .base import MIXERS, Mixer, Part, PositionEncoding, Runtime, StepContext, WeightSpec
from .linear import Linear


def _pad16(n: int) -> int:
    return -(-n // 16) * 16


@MIXERS.register("latent_attention")
class LatentAttention(Mixer):
    def __init__(self, names: Mapping[str, str], hidden_size: int, num_heads: int, key_dim: int, rot_dim: int,
                 value_dim: int, kv_rank: int, position: Optional[PositionEncoding], scale: float, eps: float,
                 shares_cache: bool = False, q_rank: int = 0, mask_window: Optional[int] = None,
                 gate_features: bool = False):
        """``names``: checkpoint tensors for 'q' (or, with ``q_rank``, 'q_down', 'q_norm' and 'q_up'), 'down' and
        'down_norm' (unless shares_cache), 'up_k', 'up_v', 'gate', 'out', and optionally 'sink'.  ``position`` rotates
        the rot_dim part of queries and of the shared key part.  ``gate_features``: the gate has a number for every
        value feature of every head instead of one a head."""
        if rot_dim % 2:
            raise ValueError(f"latent_attention: {rot_dim} rotated features (an even number is needed)")
        if kv_rank + rot_dim > 1024:
            raise ValueError(f"latent_attention: {kv_rank} + {rot_dim} cached key features exceed the attention "
                             f"kernel's 1024")
        if q_rank < 0 or (mask_window is not None and mask_window <= 0):
            raise ValueError(f"latent_attention: a query rank of {q_rank}, a window of {mask_window} tokens")
        self.names = dict(names)
        self.hidden_size, self.nh, self.dim, self.rot, self.vdim, self.rank = (hidden_size, num_heads, key_dim, rot_dim,
                                                                              value_dim, kv_rank)
        self.position, self.scale, self.eps, self.shares_cache = position, float(scale), float(eps), bool(shares_cache)
        self.q_rank, self.window = int(q_rank), int(mask_window or 0)
        self.interleaved = position is not None and position.pairs == "interleaved"
        self.qw = key_dim + rot_dim                      # a head's query as projected
        self.dk = kv_rank + rot_dim                      # a head's query and the cached key as attended
        # everything that reads the mixer's input is one product: queries (or their latent), down projection, gate
        stacked = [(self.names["q_down"], self.q_rank) if self.q_rank else (self.names["q"], num_heads * self.qw)]
        self.down_off = stacked[0][1]
        if not shares_cache:
            stacked.append((self.names["down"], kv_rank + rot_dim))
        self.gate_off = sum(r for _, r in stacked)
        self.gate_width = num_heads * value_dim if gate_features else num_heads
        stacked.append((self.names["gate"], self.gate_width))
        self.proj = Linear(stacked, hidden_size)
        self.q_up = Linear([(self.names["q_up"], num_heads * self.qw)], self.q_rank) if self.q_rank else None
        self.o = Linear([(self.names["out"], hidden_size)], num_heads * value_dim)

    def parts(self) -> List[Part]:
        return [p for p in (self.proj, self.q_up, self.o, self.position) if p is not None]

    def weight_specs(self) -> List[WeightSpec]:
        specs = [WeightSpec(self.names["up_k"], (self.nh * self.dim, self.rank)),
                 WeightSpec(self.names["up_v"], (self.nh * self.vdim, self.rank))]
        if not self.shares_cache:
            specs.append(WeightSpec(self.names["down_norm"], (self.rank,), "norm"))
        if self.q_rank:
            specs.append(WeightSpec(self.names["q_norm"], (self.q_rank,), "norm"))
        if self.names.get("sink"):
            specs.append(WeightSpec(self.names["sink"], (self.nh,), "small"))
        return specs

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime):
        self.rt = rt
        # W_uk[h]^T as the weight of a product over heads: [H, kv_rank, key_dim]; W_uv[h]: [H, value_dim, kv_rank]
        uk = tensors[self.names["up_k"]].to(rt.dtype).view(self.nh, self.dim, self.rank)
        self.uk_t = uk.transpose(1, 2).contiguous()
        self.uv = tensors[self.names["up_v"]].to(rt.dtype).view(self.nh, self.vdim, self.rank).contiguous()
        if not self.shares_cache:
            self.down_norm = tensors[self.names["down_norm"]].to(torch.float32).contiguous()
        self.q_norm = tensors[self.names["q_norm"]].to(torch.float32).contiguous() if self.q_rank else None
        self.sink = tensors[self.names["sink"]].to(torch.float32).contiguous() if self.names.get("sink") else None

    def cache_needs(self) -> CacheNeeds:
        return CacheNeeds(streams=(("k", StreamSpec(_pad16(self.dk))), ("v", StreamSpec(_pad16(self.rank)))),
                          window=self.window or None)

    def reserve_workspace(self, ws, rt: Runtime, max_step_tokens: int, max_slots: int):
        keys = min(rt.max_seq_len, self.window) if self.window else rt.max_seq_len
        ops.reserve_attention_general(ws, rt.dtype, self.nh, 1, self.rank, _pad16(self.rank), keys, max_step_tokens)

    def _rotation(self):
        rot = self.position.rotary_params() if self.position is not None else None
        if self.rot and rot is None:
            raise ValueError("latent_attention: the position encoding must be a rotation (rotary_params)")
        inv_freq, mag = rot if rot is not None else (None, 1.0)
        if self.rot and inv_freq.shape[0] * 2 != self.rot:
            raise ValueError(f"latent_attention: the rotation covers {inv_freq.shape[0] * 2} features, the rotated "
                             f"part has {self.rot}")
        return inv_freq, mag

    def forward(self, h: torch.Tensor, ctx: StepContext, cache: CacheView, writes_cache: bool = True):
        if writes_cache == self.shares_cache:
            raise ValueError("latent_attention: a layer with a down projection writes its cache entry, a layer "
                             "without one reads another layer's")
        n, H, R = h.shape[0], self.nh, self.rank
        inv_freq, mag = self._rotation()
        with ctx.timed("attn_qkv_rope"):
            proj = self.proj.forward(h, ctx, "lat.proj")
            q_src, q_cols = proj, proj[:, :H * self.qw]
            q = ctx.ws.get("lat.q", (n, H * self.dk), self.rt.dtype)
            store = dict(interleaved=self.interleaved)
            cache_args = {}
            if writes_cache:
                cache_args = dict(down=proj[:, self.down_off:self.down_off + self.dk], norm_w=self.down_norm,
                                  kpool=cache.streams["k"], vpool=cache.streams["v"], page_table=cache.page_table,
                                  page_size=cache.page_size)
            args = (q, H, self.dim, self.rot, R, self.eps, ctx.positions, ctx.tok_slot, inv_freq, mag)
            if self.q_rank:
                # the two latents' norms and the cache's rows in one launch, then the queries from theirs
                cq = ctx.ws.get("lat.cq", (n, self.q_rank), self.rt.dtype)
                ops.latent_store(*args, cq_src=proj[:, :self.q_rank], cq_norm_w=self.q_norm, cq_out=cq, **cache_args, **store)
                q_src = q_cols = self.q_up.forward(cq, ctx, "lat.q_up")
            # the query in the latent space: [W_uk[h]^T q_plain | rotated q_rot] per head
            ops.gemm_heads(q_src, 0, self.qw, self.uk_t, q, 0, self.dk)
            # rotated query parts (and, where that has not happened, the cache's rows) to their places: one launch
            if self.rot or not self.q_rank:
                ops.latent_store(*args, q_src=q_cols, **({} if self.q_rank else cache_args), **store)
        o_lat = ctx.ws.get("lat.o_lat", (n, H * R), self.rt.dtype)
        with ctx.timed("attn_core"):
            ops.attention_any(q, o_lat, H, 1, self.dk, R, self.scale, cache.streams["k"], cache.streams["v"],
                              cache.page_table, cache.page_size, ctx, window=self.window, sink=self.sink)
        out = ctx.ws.get("lat.out", (n, H * self.vdim), self.rt.dtype)
        with ctx.timed("attn_up_v"):
            ops.gemm_heads(o_lat, 0, R, self.uv, out, 0, self.vdim, gate=proj[:, self.gate_off:self.gate_off + self.gate_width])
        with ctx.timed("attn_o"):
            return self.o.forward(out, ctx, "attn.o", out_dtype=torch.float32, partials=True)
