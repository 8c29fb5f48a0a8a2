"""Attention whose keys and values are expanded from one cached latent per token.

Per token the mixer caches ``c`` (an RMS-normed down-projection of ``kv_rank`` entries) and one rotated key part
of ``rot_dim`` entries that all heads share.  Head h's key is ``[W_uk,h c ; k_rot]``, its value ``W_uv,h c``, its
query ``[q_h ; q_rot,h]`` with rotation on the ``rot`` parts only.  Since ``q_h . (W_uk,h c) = (W_uk,h^T q_h) . c``
the queries are brought into the latent space instead of the keys out of it: attention then runs over the cached
rows themselves, which all heads share, and the weighted sum of latents is expanded by ``W_uv,h`` afterwards.
Options:

    sink        a learned sink per head in the softmax's denominator
    gate        "head": a sigmoid gate per head on the output; "entry": one per entry of the concatenated heads
    window      a query sees itself and the ``window - 1`` tokens before it (None: all)
    query_rank  queries are projected up from an RMS-normed latent of their own of this size (None: from x directly)
    own_keys    False: the mixer projects no keys; it attends to the rows another layer's run cached (the running order
                names which: ``LayerRun.reads_run``), with its own queries, up-projections, window and gate

Order of kernels: one product for query latent (or queries) | down-projection | gate (float32 out); norms, rotation and
cache write; the queries' up-projection; the queries' absorption (a product per head, which also rotates the rotated
parts); attention; the expansion by ``W_uv`` with the gate folded in; the output product.
"""

from __future__ import annotations

import torch

from ..kernels.hip import AttentionMeta, QueryTurn
from .base import MIXERS, POSITION_ENCODINGS, LatentCacheNeed, Mixer, ParamSpec, PartChoice


class LatentAttention(Mixer):
    graph_safe = True

    GATES = (None, "head", "entry")

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, rot_dim: int, value_dim: int, kv_rank: int,
                 scale: float, norm_eps: float, position_encoding: PartChoice | None = None, sink: bool = False,
                 gate: str | None = None, window: int | None = None, query_rank: int | None = None,
                 own_keys: bool = True, prefix: str = "", names: dict[str, str] | None = None):
        super().__init__(prefix)
        if gate not in self.GATES:
            raise ValueError(f"the output gate is one of {self.GATES}, got {gate!r}")
        self.hidden_size, self.num_heads = hidden_size, num_heads
        self.head_dim, self.rot_dim, self.value_dim, self.kv_rank = head_dim, rot_dim, value_dim, kv_rank
        self.scale = float(scale)
        self.norm_eps = float(norm_eps)
        self.has_sink, self.gate = bool(sink), gate
        self.window, self.query_rank, self.own_keys = window, query_rank, bool(own_keys)
        self.names = {"q": "q", "q_down": "dq", "q_down_norm": "dq.norm", "q_up": "uq", "down": "dkv",
                      "down_norm": "dkv.norm", "up_k": "uk", "up_v": "uv", "sink": "sink", "gate": "g", "o": "o",
                      **(names or {})}
        self.rope = position_encoding.build(POSITION_ENCODINGS) if position_encoding is not None else None
        if self.rope is not None and self.rope.dims > rot_dim:
            raise ValueError(f"{self.rope.dims} rotated dimensions do not fit a rotated part of {rot_dim}")
        self.up_k = self.up_v = None

    def children(self):
        return [self.rope] if self.rope is not None else []

    def cache_need(self):
        return LatentCacheNeed(self.kv_rank + self.rot_dim, self.window)

    @property
    def q_width(self) -> int:
        return self.num_heads * (self.head_dim + self.rot_dim)

    # the packed product's columns: query latent or queries, then the down-projection, then the gate
    @property
    def down_offset(self) -> int:
        return self.query_rank or self.q_width

    @property
    def gate_offset(self) -> int:
        return self.down_offset + (self.kv_rank + self.rot_dim if self.own_keys else 0)

    def param_specs(self):
        n, h = self.names, self.hidden_size
        rows = [(n["q_down"], self.query_rank) if self.query_rank else (n["q"], self.q_width)]
        if self.own_keys:
            rows.append((n["down"], self.kv_rank + self.rot_dim))
        if self.gate is not None:
            rows.append((n["gate"], self.num_heads * (self.value_dim if self.gate == "entry" else 1)))
        specs = {
            "proj.weight": ParamSpec.stacked(rows, (h,)),
            "up_k.weight": ParamSpec.single(n["up_k"], (self.num_heads * self.head_dim, self.kv_rank)),
            "up_v.weight": ParamSpec.single(n["up_v"], (self.num_heads * self.value_dim, self.kv_rank)),
            "o.weight": ParamSpec.single(n["o"], (h, self.num_heads * self.value_dim)),
        }
        norm = lambda name, size: ParamSpec.single(name, (size,), kind="vector", init="one_plus_normal")  # noqa: E731
        if self.own_keys:
            specs["down_norm.weight"] = norm(n["down_norm"], self.kv_rank)
        if self.query_rank:
            specs["q_down_norm.weight"] = norm(n["q_down_norm"], self.query_rank)
            specs["q_up.weight"] = ParamSpec.single(n["q_up"], (self.q_width, self.query_rank))
        if self.has_sink:
            specs["sink"] = ParamSpec.single(n["sink"], (self.num_heads,), kind="vector")
        return specs

    def finalize(self, device, dtype):
        # per head: the key up-projection transposed, [heads, rank, dim], so that absorbing a query is x W^T like
        # every other product; the value up-projection is [heads, vdim, rank] as stored
        H, d, dv, rank = self.num_heads, self.head_dim, self.value_dim, self.kv_rank
        self.up_k = self.params["up_k.weight"].view(H, d, rank).transpose(1, 2).contiguous()
        self.up_v = self.params["up_v.weight"].view(H, dv, rank)

    def _meta(self, ctx, group: int) -> AttentionMeta:
        key = ("latent attention meta", group)
        meta = ctx.memo.get(key)
        if meta is None:
            meta = AttentionMeta(
                token_seq=ctx.token_seq, positions=ctx.positions, block_tables=ctx.block_tables[group],
                cu_seqlens_q=ctx.cu_seqlens_q, context_lens=ctx.context_lens, num_seqs=ctx.num_seqs,
                num_tokens=ctx.num_tokens, max_q_len=ctx.max_q_len, max_context_len=ctx.max_context_len,
                page_size=ctx.page_sizes[group], num_prefill=ctx.num_prefill)
            ctx.memo[key] = meta
        return meta

    def _turns(self, ctx):
        """The step's cosines and sines, formed by the first layer with this rotation and read by the others."""
        rope = self.rope
        if rope is None or not rope.dims:
            return None
        key = ("rotation table", rope.identity)
        if key not in ctx.memo:
            ctx.memo[key] = ctx.ops.rotation_table(ctx.positions, rope.freq, rope.mult)
        return ctx.memo[key]

    def forward(self, ctx, x, cache):
        ops = ctx.ops
        T = x.shape[0]
        H, d, r, dv, rank = self.num_heads, self.head_dim, self.rot_dim, self.value_dim, self.kv_rank
        width = rank + r
        new = lambda *shape: torch.empty(shape, dtype=x.dtype, device=x.device)  # noqa: E731
        turns = self._turns(ctx)
        proj = ops.linear(x, self.params["proj.weight"], None, out_dtype=torch.float32)
        ld = proj.shape[1]
        q = proj
        query = None
        if self.query_rank:
            latent_q = new(T, self.query_rank)
            query = (0, self.params["q_down_norm.weight"], latent_q)
        writes = self.own_keys and cache.writes
        if writes or query is not None:
            ops.latent_prepare(proj, cache.pages, ctx.slot_mappings[cache.group] if writes else None, self.down_offset,
                               rank, r, self.p("down_norm.weight"), self.norm_eps, turns, query)
        if query is not None:
            q = ops.linear(latent_q, self.params["q_up.weight"], None, out_dtype=torch.float32)
        q_abs = new(T, H, width)
        ops.heads_gemm(q, 0, q.shape[1], d + r, self.up_k, q_abs, 0, H * width, width, H, T, rank, d, alpha=self.scale,
                       turn=QueryTurn(d, rank, r, turns, self.scale))
        latent = new(T, H, rank)
        ops.latent_attention(q_abs, cache.pages, latent, self._meta(ctx, cache.group), rank, self.p("sink"), self.window)
        out = new(T, H * dv)
        ops.heads_gemm(latent, 0, H * rank, rank, self.up_v, out, 0, H * dv, dv, H, T, dv, rank,
                       gate=proj if self.gate is not None else None, gate_offset=self.gate_offset, ldg=ld,
                       gate_entries=self.gate == "entry")
        return ops.linear(out, self.params["o.weight"], None, defer=True)


MIXERS.register("latent_attention", LatentAttention)
