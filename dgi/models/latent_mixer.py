"""The attention step of latent-attention layers, shared by the models that have them.

``latent_heads`` takes a layer's queries (decode rows first, then packed prompt portions) and the paged
rows ``[c | r]`` of the layer that owns the latent, and returns the heads' outputs side by side:

* decode rows, short portions, fp32 and geometries the matrix kernel does not take: the unrotated query part is
  folded through the key up-projection by a batched product over heads, ``latent_attn_rows`` (HIP) attends over
  the cached rows themselves and a batched product takes the weighted latent sums to values;
* long portions in bf16: the pages a portion can see (its window, or its whole context) are expanded once into
  per-head keys ``[U_k c | r]`` and values ``U_v c`` (one GEMM, ``latent_pages``), and the MFMA flash kernel runs on
  them: (dim + rot_dim + vdim) MACs per query, key and head instead of the 2 kv_rank + rot_dim of the folded form.

``LatentUp`` holds the two up-projections in the layouts both forms read.
"""
from __future__ import annotations

import os
from typing import Optional

import torch

from dgi import ops
from dgi.ops import latent, mix
from dgi.runtime.batch import AttnMeta

# prompt rows of a step from which the MFMA prompt path replaces the row-wise kernel, where the geometry allows it
# (DGI_LATENT_MFMA_ROWS; a huge value switches it off)
MFMA_PROMPT_ROWS = int(os.environ.get("DGI_LATENT_MFMA_ROWS", "64"))


class LatentUp:
    """Key and value up-projections of one layer: ``kv`` [H * (dim + vdim), kv_rank] (every head's key rows, then every
    head's value rows), ``uk`` [H, dim, kv_rank] and ``uv`` [H, vdim, kv_rank] views of it, and ``uv_t`` [H, kv_rank, vdim],
    the contiguous right operand of the batched product on decode rows (``refresh`` after the weights changed)."""
    __slots__ = ("kv", "uk", "uv", "uv_t")

    def __init__(self, m, device, dtype):
        H = m.heads
        self.kv = torch.zeros(H * (m.dim + m.vdim), m.kv_rank, device=device, dtype=dtype)
        self.uk = self.kv[:H * m.dim].view(H, m.dim, m.kv_rank)
        self.uv = self.kv[H * m.dim:].view(H, m.vdim, m.kv_rank)
        self.uv_t = None

    def refresh(self) -> None:
        self.uv_t = self.uv.transpose(1, 2).contiguous()


def _rows(m, up: LatentUp, q, cache, tables, cu, positions, cos_sin, inter: bool, sinks, max_keys: int = 0) -> torch.Tensor:
    """[H, n, vdim] head values of rows of queries on the cached latents (folded form)."""
    n, H = q.shape[0], m.heads
    q_lat = torch.bmm(q.view(n, H, m.qk_dim)[:, :, :m.dim].transpose(0, 1), up.uk)
    o_lat = torch.empty(H, n, m.kv_rank, device=q.device, dtype=q.dtype)
    latent.latent_attn_rows(q, q_lat, cache, tables, cu, positions, H, m.dim, m.rot_dim, m.kv_rank, m.scale, m.window,
                            cos_sin, inter, out=o_lat, max_keys=max_keys, sinks=sinks)
    return torch.bmm(o_lat, up.uv_t)


def mfma_prompt_ok(m, q: torch.Tensor) -> bool:
    """Whether prompt portions of this geometry take the MFMA flash kernel."""
    return (q.is_cuda and q.dtype == torch.bfloat16 and m.qk_dim % 8 == 0 and m.vdim % 8 == 0 and max(m.qk_dim, m.vdim) <= 128
            and q.stride(0) % 8 == 0 and q.data_ptr() % 16 == 0 and mix.masked_prefill_available()
            and not torch.cuda.is_current_stream_capturing())


def visible_pages(m, meta: AttnMeta, bs: int):
    """The pages the step's portions can see: (gather list [B * n] of page ids, table [B, max pages] that maps a page's
    place in its sequence to its place in the list).  With a window only the pages from the first visible key of a
    portion on are listed; places outside map to a listed page (the kernel masks their keys)."""
    plan = meta.page_plans.get((m.window, bs))
    if plan is None:
        plan = meta.page_plans[(m.window, bs)] = _visible_pages(m, meta, bs)
    return plan


def _visible_pages(m, meta: AttnMeta, bs: int):
    bt = meta.pre_block_tables
    B, mb = bt.shape
    used = min(mb, -(-meta.pre_max_context // bs)) if meta.pre_max_context else mb
    dev = bt.device
    n = used
    if m.window > 0 and meta.pre_max_len > 0:
        n = min(used, (m.window + meta.pre_max_len - 2) // bs + 2)
    place = torch.arange(mb, dtype=torch.int32, device=dev)[None, :]
    base = (torch.arange(B, dtype=torch.int32, device=dev) * n)[:, None]
    if n == used:
        return bt[:, :used].reshape(-1), (base + place.clamp(max=n - 1)).contiguous()
    lens = meta.pre_cu_seqlens[1:] - meta.pre_cu_seqlens[:-1]
    first = torch.clamp(meta.pre_context_lens - lens - (m.window - 1), min=0) // bs                     # [B] page of the first visible key
    first = torch.minimum(first, torch.full_like(first, used - n))[:, None]
    listed = torch.gather(bt, 1, (first + torch.arange(n, dtype=torch.int32, device=dev)[None, :]).long())
    return listed.reshape(-1), (base + (place - first).clamp(0, n - 1)).to(torch.int32).contiguous()


def prompt_heads(m, up: LatentUp, q, cache, meta: AttnMeta, cos_sin, inter: bool, sinks, gate, per_head: bool, out) -> torch.Tensor:
    """Gated head outputs [n, H * vdim] of the step's prompt rows ``q`` on the MFMA flash kernel."""
    bs = cache.shape[2]
    listed, table = visible_pages(m, meta, bs)
    lat = cache.view(cache.shape[0], bs, m.cache_dim).index_select(0, listed).view(-1, m.cache_dim)
    kt, vt = latent.latent_pages(ops.linear(lat[:, :m.kv_rank], up.kv), lat, bs, m.heads, m.dim, m.rot_dim, m.vdim)
    if cos_sin is not None:
        latent.rotate_heads(q, meta.positions[meta.num_decode:], cos_sin, inter, m.heads, m.qk_dim, m.dim)
    return mix.paged_prefill_masked(q, kt, vt, table, meta.pre_cu_seqlens, meta.pre_context_lens, m.heads, m.heads,
                                    m.scale, 0, gate, tiles=meta.pre_tiles, window=m.window, out=out, sinks=sinks,
                                    gate_heads=per_head)


def latent_heads(m, up: LatentUp, q: torch.Tensor, cache: torch.Tensor, meta: AttnMeta, cos_sin: Optional[torch.Tensor],
                 gate: Optional[torch.Tensor] = None, sinks: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Head outputs [T, H * vdim] of a step.  ``m``: ``LatentAttentionSpec``; ``q`` [T, H * (dim + rot_dim)] projected
    queries, not rotated (a step with prompt rows may rotate them in place); ``cache`` the pages of the layer that owns
    the latent; ``gate`` [T, H] or [T, H * vdim] output gate logits (``m.gate``); ``sinks`` [H] fp32."""
    T, nd = q.shape[0], meta.num_decode
    inter = m.rot is not None and m.rot.layout == "interleaved"
    per_head = m.gate == "head"
    out = torch.empty(T, m.o_size, device=q.device, dtype=q.dtype)

    def put(ov, lo, hi):
        latent.gate_heads(ov, None if gate is None else gate[lo:hi], per_head, out=out[lo:hi])

    if nd > 0:
        put(_rows(m, up, q[:nd], cache, meta.dec_block_tables, None, meta.positions[:nd], cos_sin, inter, sinks,
                  meta.dec_block_tables.shape[1] * cache.shape[2]), 0, nd)
    if meta.num_prefill_tokens >= MFMA_PROMPT_ROWS and mfma_prompt_ok(m, q):
        prompt_heads(m, up, q[nd:], cache, meta, cos_sin, inter, sinks, None if gate is None else gate[nd:], per_head, out[nd:])
    elif meta.num_prefill_tokens > 0:
        put(_rows(m, up, q[nd:], cache, meta.pre_block_tables, meta.pre_cu_seqlens, meta.positions[nd:], cos_sin, inter, sinks),
            nd, T)
    return out
