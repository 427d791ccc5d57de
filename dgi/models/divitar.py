"""Native Divitar decoder for the MI355X runtime.

Notation (T rows of a step, W the width, x the fp32 residual stream, rms(v) = sqrt(mean(v^2) + eps), r the residual
multiplier):

    embedding   x_t = E[tok_t]
    layer i     x += r Mix_i(x / rms(x) * n1)
                x += r FF_i(x / rms(x) * n2)                                 (if the layer has a feed-forward)
                y  = P_i (gelu(G_i x) * S[tok_t, i * d : (i + 1) * d])       per-layer token input, d = side_dim
                x += r y / rms(y) * ns
    logits      head(x / rms(x) * nf) * logit_scale

Mix is one of

* ``attention``: grouped-query softmax attention inside chunks of positions (a query sees the earlier keys of its own
  chunk, chunks counted from position 0); q and k with biases, half-split rotary pairs on the first dims of a head with
  all frequencies divided by one factor; the values are the keys as projected, before rotation; one sigmoid gate per head;
* ``latent_attention``: keys and values of all heads come from one normalised latent per token plus one rotated key part
  shared by the heads (``dgi.ops.latent``), queries straight from the layer's input; interleaved rotary pairs with
  ramp-scaled frequencies, a sliding window, and a learned logit per head in the softmax denominator.  A layer with
  ``kv_from = j`` has no latent of its own and reads layer j's cached rows with its own up-projections and window.

FF is W_d max(W_u h, 0)^2, or gated-SiLU experts chosen by sigmoid scores (fp32; the ``top`` largest, divided by their
sum, times a factor) beside a shared expert that every token takes.

Per layer the step executes (rows: decode rows first, then packed prompt portions)::

    stream_add_norm (HIP)   previous sublayer's residual add (+ the token input's unit-RMS norm) + n1 norm
    attention:   q | k | head-gate GEMM (biases in its epilogue) -> qk_rope (HIP: rotary of q in place, rotated and raw
                 keys into the pages) -> masked_attn_rows (HIP, decode rows, fp32) / paged_prefill_masked (HIP, MFMA),
                 chunk mask and head gate inside -> o GEMM
    latent:      q | latent GEMM -> latent_prep (HIP: latent norm + rotary key part -> cached row) ->
                 ``dgi.models.latent_mixer`` (rows on the cached latents / expanded pages on the MFMA kernel) -> o GEMM
    stream_add_norm (HIP)   x += r mix, n2 norm
    dense: up GEMM -> relu_sq (HIP) -> down GEMM;  moe: moe_router (HIP: fp32 logits and choice) -> moe_plan, moe_group,
                 moe_combine (HIP, grouped MFMA products) + shared expert
    stream_add_norm (HIP)   x += r ff (-> bf16 copy of x); G GEMM -> gelu_tanh x gathered token row (HIP) -> P GEMM

The stream, every norm, rotary angles, scores / softmax and the router are fp32 whatever ``dtype`` is; with bf16 the
projections and activations are bf16 with fp32 accumulation.  Pages come from the engine's block pool (every layer
that owns keys or a latent its own geometry); a sequence carries nothing else.
"""
from __future__ import annotations

from typing import Optional

import torch

from dgi import ops
from dgi.models.config import DivitarConfig
from dgi.models.latent_mixer import LatentUp, latent_heads
from dgi.ops import latent, mix, moe
from dgi.runtime.batch import AttnMeta


class DivitarLayerWeights:
    FIELDS = ("norm1", "norm2", "in_proj", "in_bias", "dkv_norm", "uk", "uv", "sink", "o", "up", "down", "router",
              "gate_up", "shared_gate_up", "shared_down", "side_gate", "side_proj", "side_norm")
    __slots__ = ("spec", "cos_sin", "up_kv", "router_bf16") + FIELDS

    def __init__(self, spec):
        for k in self.__slots__:
            setattr(self, k, None)
        self.spec = spec

    def in_parts(self) -> list:
        """(name, first row, end row) of the parts of the mixer's fused input projection."""
        m = self.spec.mixer
        if self.spec.type == "attention":
            sizes = [("q", m.q_size), ("k", m.k_size), ("g", m.heads)]
        else:
            sizes = [("q", m.q_size)] + ([("dkv", m.cache_dim)] if m.kv_from is None else [])
        out, at = [], 0
        for name, n in sizes:
            out.append((name, at, at + n))
            at += n
        return out

    def named(self):
        for k in self.FIELDS:
            t = getattr(self, k)
            if t is not None:
                yield k, t


class DivitarModel:
    """A Divitar causal LM (all layers on one device)."""

    routes_gemms = False       # projections are plain vendor GEMMs: no start-up routing table

    def __init__(self, cfg: DivitarConfig, device: torch.device | str = "cpu", dtype=torch.bfloat16,
                 layer_start: int = 0, layer_end: Optional[int] = None, has_embed: Optional[bool] = None,
                 has_head: Optional[bool] = None, seed: int = 0, init: str = "random",
                 checkpoint: Optional[str] = None):
        if layer_start != 0 or (layer_end is not None and layer_end != cfg.num_layers):
            raise ValueError("Divitar runs all its layers in one stage (layers may read an earlier layer's cache rows)")
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.layer_start, self.layer_end = 0, cfg.num_layers
        self.has_embed = self.has_head = True
        self.num_local_layers = cfg.num_layers
        self.kv_cache = None
        self.kv_layers: list = []
        self.layers: list[DivitarLayerWeights] = []
        self.embed = self.side_embed = self.head = self.final_norm = None
        self.capture_layers: tuple = ()
        self.captured: dict = {}
        self.layer_hook = None
        self.reduce = None
        self.mlp_pad = self.mlp_impl = self.proj_impl = self.fold_impl = None
        self.load_info: Optional[dict] = None
        self._tables: dict = {}
        # page-pool layer of every layer that owns pages; the others index their source's
        self.kv_index = {li: n for n, li in enumerate(cfg.kv_owners)}
        self._init_empty()
        if checkpoint:
            from dgi.models.weights import load_divitar_checkpoint
            self.load_info = load_divitar_checkpoint(self, checkpoint)
        elif init == "random":
            self._init_random(seed)
        self.finish_weights()

    # ------------------------------------------------------------------ weights
    def _init_empty(self):
        c, dev, dt = self.cfg, self.device, self.dtype
        W = c.hidden_size

        def e(*shape, dtype=dt):
            return torch.zeros(*shape, device=dev, dtype=dtype)

        for spec in c.layers:
            L = DivitarLayerWeights(spec)
            m, f = spec.mixer, spec.mlp
            L.norm1 = torch.ones(W, device=dev)
            rows = (L.in_parts()[-1][2] + 15) // 16 * 16       # padded with zero rows: 16-byte aligned projection rows
            L.in_proj = e(rows, W)
            if spec.type == "attention":
                L.in_bias = e(rows)
            else:
                if m.kv_from is None:
                    L.dkv_norm = torch.ones(m.kv_rank, device=dev)
                L.up_kv = LatentUp(m, dev, dt)
                L.uk, L.uv = L.up_kv.uk, L.up_kv.uv
                L.sink = e(m.heads, dtype=torch.float32)
            L.o = e(W, m.o_size)
            if f is not None:
                L.norm2 = torch.ones(W, device=dev)
                if f.kind == "dense":
                    L.up, L.down = e(f.ff, W), e(W, f.ff)
                else:
                    L.router = e(f.experts, W, dtype=torch.float32)
                    L.gate_up, L.down = e(f.experts, 2 * f.ff, W), e(f.experts, W, f.ff)
                    if f.shared_ff:
                        L.shared_gate_up, L.shared_down = e(2 * f.shared_ff, W), e(W, f.shared_ff)
            if c.side_dim > 0:
                L.side_gate, L.side_proj = e(c.side_dim, W), e(W, c.side_dim)
                L.side_norm = torch.ones(W, device=dev)
            self.layers.append(L)
        self.embed = e(c.vocab_size, W)
        if c.side_dim > 0:
            self.side_embed = e(c.vocab_size, c.side_dim * c.num_layers)
        self.final_norm = torch.ones(W, device=dev)
        self.head = e(c.vocab_size, W)

    def _init_random(self, seed: int):
        """Deterministic per-tensor values drawn on the CPU (the same on every device)."""
        c = self.cfg
        W = c.hidden_size
        gen = torch.Generator()

        def fill(t, std, mean=0.0):
            if t is not None:
                t.copy_((torch.randn(t.shape, generator=gen) * std + mean).to(t.dtype))

        for li, L in enumerate(self.layers):
            gen.manual_seed(seed * 1000003 + li * 7919 + 1)
            for n in (L.norm1, L.norm2, L.dkv_norm):
                fill(n, 0.1, 1.0)
            fill(L.side_norm, 0.05, 0.3)
            for name, lo, hi in L.in_parts():
                fill(L.in_proj[lo:hi], W ** -0.5)
                if L.in_bias is not None and name != "g":
                    fill(L.in_bias[lo:hi], 0.3)
            fill(L.sink, 1.0, 0.5)
            for t in (L.uk, L.uv, L.o, L.up, L.gate_up, L.down, L.shared_gate_up, L.shared_down):
                if t is not None:
                    fill(t, t.shape[-1] ** -0.5)
            fill(L.router, W ** -0.5 * 2)
            if L.router is not None:
                L.router.copy_(L.router.to(torch.bfloat16))           # as a bf16 checkpoint would hold it
            fill(L.side_gate, W ** -0.5)
            fill(L.side_proj, max(1, c.side_dim) ** -0.5)
        gen.manual_seed(seed * 1000003 + 17)
        fill(self.embed, 1.0)
        fill(self.side_embed, 1.0)
        fill(self.head, W ** -0.5)
        fill(self.final_norm, 0.1, 1.0)

    def _rope_table(self, rot) -> Optional[torch.Tensor]:
        if rot is None or rot.dims <= 0:
            return None
        key = (rot.dims, rot.base, tuple(sorted((rot.scaling or {}).items())), self.cfg.max_position)
        t = self._tables.get(key)
        if t is None:
            t = self._tables[key] = ops.rope_cos_sin(rot.dims, self.cfg.max_position, rot.base, rot.scaling,
                                                     device=self.device)
        return t

    def finish_weights(self) -> None:
        """Derived tables (after the weights are in place): rotary cos / sin by position, the value
        up-projection as the batched product reads it, the router in bf16 where that is exact."""
        for L in self.layers:
            L.cos_sin = self._rope_table(L.spec.mixer.rot)
            if L.up_kv is not None:
                L.up_kv.refresh()
            if L.router is not None:
                L.router_bf16 = moe.exact_bf16(L.router)

    def tensors(self):
        for i, L in enumerate(self.layers):
            for k, t in L.named():
                yield f"layers.{i}.{k}", t
        for k in ("embed", "side_embed", "final_norm", "head"):
            t = getattr(self, k)
            if t is not None:
                yield k, t

    def copy_from(self, other: "DivitarModel") -> "DivitarModel":
        src = dict(other.tensors())
        for name, t in self.tensors():
            if name in src:
                t.copy_(src[name])
        self.finish_weights()
        return self

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for _n, t in self.tensors())

    # ------------------------------------------------------------------ cache
    def attach_cache(self, pool) -> None:
        """Bind the engine's block pool: ``kv_layers[n]`` = pages of the n-th layer that owns pages (a latent's
        value half is empty)."""
        self.kv_cache = pool.kv
        self.kv_layers = pool.layers

    # ------------------------------------------------------------------ mixers
    @staticmethod
    def _mfma_prefill_ok(m, u: torch.Tensor) -> bool:
        return (u.is_cuda and u.dtype == torch.bfloat16 and m.dim % 8 == 0 and m.dim <= 128 and u.shape[1] % 8 == 0
                and mix.masked_prefill_available() and not torch.cuda.is_current_stream_capturing())

    def _attention(self, li: int, L, h: torch.Tensor, meta: AttnMeta) -> torch.Tensor:
        """Gated head outputs [T, H * dim] of a chunked-attention layer."""
        m = L.spec.mixer
        kc, vc = self.kv_layers[self.kv_index[li]]
        u = ops.linear(h, L.in_proj, L.in_bias)
        mix.qk_rope(u, meta.positions, meta.slot_mapping, L.cos_sin, m.heads, m.kv_heads, m.dim, m.vdim, kc, vc,
                    layout=m.rot.layout if m.rot is not None else "half", shared=m.shared_kv)
        gate = u[:, m.q_size + m.k_size:m.q_size + m.k_size + m.heads]
        out = torch.empty(u.shape[0], m.o_size, device=u.device, dtype=u.dtype)
        nd, pos = meta.num_decode, meta.positions
        if nd > 0:
            mix.masked_attn_rows(u[:nd], kc, vc, meta.dec_block_tables, None, pos[:nd], m.heads, m.kv_heads, m.scale, m.mask_size,
                                 gate[:nd], out=out[:nd], gate_heads=True,
                                 max_keys=meta.dec_block_tables.shape[1] * kc.shape[2])
        if meta.num_prefill_tokens > 0:
            bt, cu = meta.pre_block_tables, meta.pre_cu_seqlens
            if self._mfma_prefill_ok(m, u):
                mix.paged_prefill_masked(u[nd:], kc, vc, bt, cu, meta.pre_context_lens, m.heads, m.kv_heads, m.scale, m.mask_size,
                                         gate[nd:], tiles=meta.pre_tiles, out=out[nd:], gate_heads=True)
            else:
                mix.masked_attn_rows(u[nd:], kc, vc, bt, cu, pos[nd:], m.heads, m.kv_heads, m.scale, m.mask_size, gate[nd:],
                                     out=out[nd:], gate_heads=True)
        return out

    def _latent(self, li: int, L, h: torch.Tensor, meta: AttnMeta) -> torch.Tensor:
        """Head outputs [T, H * vdim] of a latent-attention layer."""
        m = L.spec.mixer
        own = m.kv_from is None
        cache = self.kv_layers[self.kv_index[li if own else m.kv_from]][0]
        u = ops.linear(h, L.in_proj)
        if own:
            latent.latent_prep(u[:, m.q_size:], 0, m.kv_rank, m.rot_dim, None, L.dkv_norm, self.cfg.norm_eps, meta.positions,
                               meta.slot_mapping, L.cos_sin, m.rot is not None and m.rot.layout == "interleaved", cache)
        return latent_heads(m, L.up_kv, u[:, :m.q_size], cache, meta, L.cos_sin, sinks=L.sink)

    def _ff(self, L, h: torch.Tensor) -> torch.Tensor:
        f = L.spec.mlp
        if f.kind == "dense":
            return ops.linear(latent.relu_sq(ops.linear(h, L.up)), L.down)
        idx, wts = moe.moe_router(h, L.router, L.router_bf16, f.top, f.renorm, f.scale)
        shared = None
        if f.shared_ff:
            shared = ops.linear(moe.silu_mul(ops.linear(h, L.shared_gate_up)), L.shared_down)
        return moe.moe_experts(h, idx, wts, L.gate_up, L.down, shared)

    # ------------------------------------------------------------------ forward
    def forward_layers(self, x: torch.Tensor, meta: AttnMeta, ids: torch.Tensor,
                       trim_last: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Run every layer on the fp32 stream ``x`` [T, W] (updated in place; returned).  ``trim_last`` (row indices):
        after the last layer's attention — which has written every row's cache entries — only those rows go on; the
        returned stream holds just them."""
        c, dt = self.cfg, self.dtype
        eps, mult = c.norm_eps, c.residual_mult
        n = len(self.layers)
        pend = (None, None)            # (y, post-norm weight) of the sublayer whose residual add is due
        for li, L in enumerate(self.layers):
            h = latent.stream_add_norm(x, *pend, L.norm1, eps, dt, mult=mult)
            att = (self._attention if L.spec.type == "attention" else self._latent)(li, L, h, meta)
            if li == n - 1 and trim_last is not None:
                att, x, ids = (t.index_select(0, trim_last) for t in (att, x, ids))
            y = ops.linear(att, L.o)
            if self.reduce is not None:
                self.reduce(y)
            if L.spec.mlp is not None:
                h = latent.stream_add_norm(x, y, None, L.norm2, eps, dt, mult=mult)
                y = self._ff(L, h)
                if self.reduce is not None:
                    self.reduce(y)
            pend = (y, None)
            if L.side_gate is not None:
                # the token input reads the stream itself: finish the add, then gate a slice of the token's row
                xb = latent.stream_add_norm(x, y, None, None, eps, None if dt == torch.float32 else dt, mult=mult)
                g = latent.gelu_tanh(ops.linear(x if xb is None else xb, L.side_gate), self.side_embed, ids,
                                     li * c.side_dim)
                pend = (ops.linear(g, L.side_proj), L.side_norm)
            if self.capture_layers and li in self.capture_layers:
                latent.stream_add_norm(x, *pend, None, eps, None, mult=mult)
                pend = (None, None)
                self.captured[li] = x.clone()
            if self.layer_hook is not None:
                self.layer_hook(li)
        if pend[0] is not None:
            latent.stream_add_norm(x, *pend, None, eps, None, mult=mult)
        return x

    def embed_tokens(self, ids: torch.Tensor) -> torch.Tensor:
        return latent.embed_rows(ids, self.embed)

    def forward(self, meta: AttnMeta, input_ids: Optional[torch.Tensor] = None,
                hidden: Optional[torch.Tensor] = None) -> torch.Tensor:
        """fp32 logits [n, V] of the step's logits rows."""
        ids = input_ids.to(torch.int32)
        x = self.embed_tokens(ids)
        idx = meta.logits_indices
        trim = idx is not None and bool(self.layers) and not self.capture_layers and idx.shape[0] < x.shape[0]
        x = self.forward_layers(x, meta, ids, trim_last=idx if trim else None)
        if idx is not None and not trim:
            x = x.index_select(0, idx)
        return self.compute_logits(x)

    def compute_logits(self, x: torch.Tensor) -> torch.Tensor:
        hn = latent.stream_add_norm(x.contiguous(), None, None, self.final_norm, self.cfg.norm_eps, self.dtype)
        return mix.scale_softcap(ops.linear(hn, self.head), self.cfg.logit_scale, 0.0)
