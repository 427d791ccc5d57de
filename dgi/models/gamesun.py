"""Native Gamesun decoder for the MI355X runtime.

Notation (T rows of a step, W the width, x the fp32 residual stream, rms(v) = sqrt(mean(v^2) + eps)):

    embedding   x_t = s E[tok_t] + pos(p_t)                  pos: sin / cos interleaved, computed from the position
    layer       h = x / rms(x) * n1;  x += (L / rms(L) * wl + R / rms(R) * wr) / 2
                h = x / rms(x) * n2;  x += Wd (silu(Wg h) * (Wu h))           (or no feed-forward)
    logits      E (x / rms(x) * nf)

L and R are two mixers on the same h: an attention over the last ``window`` positions without rotation, and a
linear recurrence.

* ``parallel``: L — q, k, v with biases; the heads' scaled scores are mixed by a learned matrix; the weight of a
  visible key is sigmoid(score + a number per head), not normalised; output projection with bias.  R — gated linear
  attention: a decay sigmoid(z)^(1/tau) per key channel, z = A2 (A1 h) + b; per-head RMS norm (weight shared by the
  heads), times silu(gate).
* ``parallel_2``: L — softmax attention whose scaled scores are multiplied by a learned number per head.  R —
  lightning attention: SiLU on q, k and v, a constant decay per head; one RMS norm over all heads, times
  sigmoid(gate).

Per layer the step executes (rows: decode rows first, then packed prompt portions)::

    one GEMM for both branches' projections (bias in its epilogue)
    kv_rows (HIP)                       k | v columns into the pages
    parallel:   sigmoid_attn_rows (HIP, decode rows: keys split over workgroups) / sigmoid_prefill (HIP, MFMA)
    parallel_2: masked_attn_rows (HIP) / paged_prefill_masked (HIP, MFMA)
    lowrank_decay (HIP, fp32)           the decays of a gated recurrence
    linear_scan (HIP, gla / lightning)  -> head_norm_gate (HIP)
    two output GEMMs -> pair_add_norm (HIP: both branch norms, their mean, the residual add, the next norm)
    gate | up GEMM -> glu_silu (HIP) -> down GEMM -> stream_add_norm (HIP: residual add + next norm)

The stream, every norm, positions, scores and attention weights, decays and recurrent state are fp32 whatever
``dtype`` is; with bf16 the large projections take bf16 inputs with fp32 accumulation.  Pages come from the engine's
block pool (every layer its own geometry), states from ``dgi.kv.state_pool.StatePool``.
"""
from __future__ import annotations

from typing import Optional

import torch

from dgi import ops
from dgi.models.config import GamesunConfig, GatedLinearSpec
from dgi.ops import latent, linrec, mix, moe
from dgi.runtime.batch import AttnMeta


class GamesunLayerWeights:
    FIELDS = ("norm1", "norm2", "in_proj", "in_bias", "talk", "pb", "temp", "o_left", "o_bias", "out_left",
              "a1", "a2", "a2_b", "decay", "rnorm", "o_right", "out_right", "gate_up", "down")
    __slots__ = ("spec",) + FIELDS

    def __init__(self, spec):
        for k in self.FIELDS:
            setattr(self, k, None)
        self.spec = spec

    def in_rows(self, left: str = "left.", right: str = "right.") -> list:
        """(name, rows) of the fused projection, in order: the left branch's q | k | v, the right one's q | k | v | gate."""
        a, r = self.spec.mixer.left, self.spec.mixer.right
        return [(left + "q", a.q_size), (left + "k", a.k_size), (left + "v", a.v_size), (right + "q", r.qk_size),
                (right + "k", r.qk_size), (right + "v", r.inner), (right + "g", r.inner)]

    def named(self):
        for k in self.FIELDS:
            t = getattr(self, k)
            if t is not None:
                yield k, t


class GamesunModel:
    """A Gamesun causal LM (all layers on one device)."""

    routes_gemms = False       # projections are plain vendor GEMMs: no start-up routing table

    def __init__(self, cfg: GamesunConfig, device: torch.device | str = "cpu", dtype=torch.bfloat16,
                 layer_start: int = 0, layer_end: Optional[int] = None, has_embed: Optional[bool] = None,
                 has_head: Optional[bool] = None, seed: int = 0, init: str = "random",
                 checkpoint: Optional[str] = None):
        if layer_start != 0 or (layer_end is not None and layer_end != cfg.num_layers):
            raise ValueError("Gamesun runs all its layers in one stage (per-sequence state is not passed between stages)")
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.layer_start, self.layer_end = 0, cfg.num_layers
        self.has_embed = self.has_head = True
        self.num_local_layers = cfg.num_layers
        self.kv_cache = None
        self.kv_layers: list = []
        self.state = None
        self.layers: list[GamesunLayerWeights] = []
        self.embed = self.final_norm = self.freqs = None
        self.capture_layers: tuple = ()
        self.captured: dict = {}
        self.layer_hook = None
        self.reduce = None
        self.mlp_pad = self.mlp_impl = self.proj_impl = self.fold_impl = None
        self.load_info: Optional[dict] = None
        if checkpoint:
            from dgi.models.weights import gamesun_checkpoint_shapes
            gamesun_checkpoint_shapes(cfg, checkpoint)
        self._init_empty()
        if checkpoint:
            from dgi.models.weights import load_gamesun_checkpoint
            self.load_info = load_gamesun_checkpoint(self, checkpoint)
        elif init == "random":
            self._init_random(seed)

    # ------------------------------------------------------------------ weights
    def _init_empty(self):
        c, dev = self.cfg, self.device
        W, f32 = c.hidden_size, torch.float32

        def e(*shape, dtype=self.dtype):
            return torch.zeros(*shape, device=dev, dtype=dtype)

        def ones(n):
            return torch.ones(n, device=dev)

        for spec in c.layers:
            L = GamesunLayerWeights(spec)
            a, r, f = spec.mixer.left, spec.mixer.right, spec.mlp
            L.norm1 = ones(W)
            n_in = sum(rows for _n, rows in L.in_rows())
            L.in_proj = e(n_in, W)
            L.o_left, L.out_left = e(W, a.o_size), ones(W)
            if a.bias:
                L.in_bias, L.o_bias = e(n_in), e(W)
            if a.talk:
                L.talk, L.pb = e(a.heads, a.heads, dtype=f32), e(a.heads, dtype=f32)
            if a.head_temp:
                L.temp = ones(a.heads)
            L.o_right, L.out_right = e(W, r.inner), ones(W)
            if isinstance(r, GatedLinearSpec):
                if r.decay_rank <= 0:
                    raise ValueError("Gamesun: gated linear attention needs decay_rank (read from the checkpoint, or given)")
                L.a1, L.a2, L.a2_b = e(r.decay_rank, W, dtype=f32), e(r.qk_size, r.decay_rank, dtype=f32), e(r.qk_size, dtype=f32)
                L.rnorm = ones(r.vdim)
            else:
                L.decay = torch.tensor(r.decay, dtype=f32, device=dev)
                L.rnorm = ones(r.inner)
            if f is not None:
                L.norm2 = ones(W)
                L.gate_up, L.down = e(2 * f.ff, W), e(W, f.ff)
            self.layers.append(L)
        self.embed = e(c.vocab_size, W)
        self.final_norm = ones(W)
        self.freqs = mix.sinusoid_freqs(W, device=dev)

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
            a = L.spec.mixer.left
            for n in (L.norm1, L.norm2, L.rnorm, L.out_left, L.out_right):
                fill(n, 0.1, 1.0)
            fill(L.in_proj, W ** -0.5)
            if L.in_bias is not None:
                fill(L.in_bias[: a.q_size + a.k_size + a.v_size], 0.3)
            fill(L.o_bias, 0.1)
            fill(L.talk, 0.5 * a.heads ** -0.5)
            if L.talk is not None:
                L.talk.diagonal().add_(1.0)
            fill(L.pb, 0.5, -3.0)
            fill(L.temp, 0.3, 1.0)
            fill(L.a1, W ** -0.5)
            if L.a2 is not None:
                fill(L.a2, L.a2.shape[1] ** -0.5)
            fill(L.a2_b, 0.5, 2.0)
            for t in (L.o_left, L.o_right, L.gate_up, L.down):
                if t is not None:
                    fill(t, t.shape[1] ** -0.5)
        gen.manual_seed(seed * 1000003 + 17)
        fill(self.embed, W ** -0.5)
        fill(self.final_norm, 0.1, 1.0)

    def tensors(self):
        for i, L in enumerate(self.layers):
            for k, t in L.named():
                yield f"layers.{i}.{k}", t
        for k in ("embed", "final_norm"):
            yield k, getattr(self, k)

    def copy_from(self, other: "GamesunModel") -> "GamesunModel":
        src = dict(other.tensors())
        for name, t in self.tensors():
            if name in src:
                t.copy_(src[name])
        return self

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for _n, t in self.tensors())

    # ------------------------------------------------------------------ cache and state
    def state_fields(self) -> dict:
        """What one sequence carries besides pages: name -> (shape, dtype) per layer."""
        return {f"mem.{i}": ((L.spec.mixer.right.heads, L.spec.mixer.right.dim, L.spec.mixer.right.vdim), torch.float32)
                for i, L in enumerate(self.layers)}

    def attach_cache(self, pool, state_pool=None) -> None:
        """Bind the engine's block pool (``kv_layers[i]`` = pages of layer i's attention) and state pool."""
        self.kv_cache = pool.kv
        self.kv_layers = pool.layers
        if state_pool is not None:
            self.state = state_pool

    # ------------------------------------------------------------------ mixers
    def _left(self, i: int, L, u: torch.Tensor, meta: AttnMeta) -> torch.Tensor:
        """Head outputs [T, H * vdim] of the attention branch; ``u`` rows = q | k | v | ..."""
        a = L.spec.mixer.left
        kc, vc = self.kv_layers[i]
        mix.kv_rows(u[:, a.q_size:], meta.slot_mapping, a.kv_heads, a.dim, a.vdim, kc, vc)
        out = torch.empty(u.shape[0], a.o_size, device=u.device, dtype=u.dtype)
        nd, pos = meta.num_decode, meta.positions
        win = a.window
        if nd > 0:
            bt = meta.dec_block_tables
            if a.weights == "sigmoid":
                mix.sigmoid_attn_rows(u[:nd], kc, vc, bt, None, pos[:nd], a.heads, a.kv_heads, a.scale, win, L.talk, L.pb,
                                      out=out[:nd], max_keys=bt.shape[1] * kc.shape[2])
            else:
                mix.masked_attn_rows(u[:nd], kc, vc, bt, None, pos[:nd], a.heads, a.kv_heads, a.scale, 0, None, out=out[:nd],
                                     window=win, head_scale=L.temp)
        if meta.num_prefill_tokens > 0:
            bt, cu = meta.pre_block_tables, meta.pre_cu_seqlens
            if (a.weights == "sigmoid" and mix.sigmoid_prefill_ok(u, kc, vc, a.heads, a.kv_heads)
                    and not torch.cuda.is_current_stream_capturing()):
                mix.sigmoid_prefill(u[nd:], kc, vc, bt, cu, meta.pre_context_lens, a.heads, a.kv_heads, a.scale, win, L.talk,
                                    L.pb, tiles=meta.pre_tiles, out=out[nd:])
            elif a.weights == "sigmoid":
                mix.sigmoid_attn_rows(u[nd:], kc, vc, bt, cu, pos[nd:], a.heads, a.kv_heads, a.scale, win, L.talk, L.pb,
                                      out=out[nd:], max_keys=bt.shape[1] * kc.shape[2])
            elif (u.is_cuda and u.dtype == torch.bfloat16 and max(a.dim, a.vdim) <= 128 and a.dim % 8 == 0 and a.vdim % 8 == 0
                  and u.shape[1] % 8 == 0 and mix.masked_prefill_available() and not torch.cuda.is_current_stream_capturing()):
                # MFMA flash kernel (bf16 heads of up to 128 dims); other geometries and fp32: the row-wise kernel
                mix.paged_prefill_masked(u[nd:], kc, vc, bt, cu, meta.pre_context_lens, a.heads, a.kv_heads, a.scale, 0, None,
                                         tiles=meta.pre_tiles, out=out[nd:], window=win, head_scale=L.temp)
            else:
                mix.masked_attn_rows(u[nd:], kc, vc, bt, cu, pos[nd:], a.heads, a.kv_heads, a.scale, 0, None, out=out[nd:],
                                     window=win, head_scale=L.temp)
        return out

    def _right(self, i: int, L, h: torch.Tensor, u: torch.Tensor, meta: AttnMeta) -> torch.Tensor:
        """Gated, normed read-out [T, inner] of the recurrence; ``u`` rows = q | k | v | gate."""
        r = L.spec.mixer.right
        q, k, v, g = u.split((r.qk_size, r.qk_size, r.inner, r.inner), dim=1)
        where = (self.state[f"mem.{i}"], meta.positions, meta.seq_row0, meta.seq_slots, r.heads, r.dim, r.vdim)
        if isinstance(r, GatedLinearSpec):
            y = linrec.gla_scan(q, k, v, linrec.lowrank_decay(h, L.a1, L.a2, L.a2_b, r.tau), *where)
            return linrec.head_norm_gate(y, g, L.rnorm, r.heads, self.cfg.norm_eps, "silu", self.dtype)
        y = linrec.lightning_scan(q, k, v, L.decay, *where)
        return linrec.head_norm_gate(y, g, L.rnorm, 1, self.cfg.norm_eps, "sigmoid", self.dtype)

    def _mixers(self, i: int, L, h: torch.Tensor, meta: AttnMeta):
        """Outputs [T, W] of the two branches."""
        a = L.spec.mixer.left
        u = ops.linear(h, L.in_proj, L.in_bias)
        left = ops.linear(self._left(i, L, u, meta), L.o_left, L.o_bias)
        right = ops.linear(self._right(i, L, h, u[:, a.q_size + a.k_size + a.v_size:], meta), L.o_right)
        return left, right

    # ------------------------------------------------------------------ forward
    def forward_layers(self, x: torch.Tensor, meta: AttnMeta) -> torch.Tensor:
        """Run every layer on the fp32 stream ``x`` [T, W] (updated in place)."""
        eps, dt = self.cfg.norm_eps, self.dtype
        n = len(self.layers)
        h = latent.stream_add_norm(x, None, None, self.layers[0].norm1, eps, dt) if n else None
        for i, L in enumerate(self.layers):
            left, right = self._mixers(i, L, h, meta)
            nxt = self.layers[i + 1].norm1 if i + 1 < n else None          # the next layer's norm rides on this layer's last add
            nxt_dt = dt if nxt is not None else None
            if L.gate_up is None:
                h = linrec.pair_add_norm(x, left, right, L.out_left, L.out_right, nxt, eps, nxt_dt)
            else:
                h = linrec.pair_add_norm(x, left, right, L.out_left, L.out_right, L.norm2, eps, dt)
                y = ops.linear(moe.silu_mul(ops.linear(h, L.gate_up)), L.down)
                if self.reduce is not None:
                    self.reduce(y)
                h = latent.stream_add_norm(x, y, None, nxt, eps, nxt_dt)
            if self.capture_layers and i in self.capture_layers:
                self.captured[i] = x.clone()
            if self.layer_hook is not None:
                self.layer_hook(i)
        return x

    def embed_tokens(self, ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        return mix.embed_sinusoid(ids, positions, self.embed, self.cfg.embedding_scale, self.freqs)

    def forward(self, meta: AttnMeta, input_ids: Optional[torch.Tensor] = None,
                hidden: Optional[torch.Tensor] = None) -> torch.Tensor:
        """fp32 logits [n, V] of the step's logits rows."""
        if meta.seq_slots is None:
            raise RuntimeError("Gamesun needs the step's sequence tables (a runner built with a state pool)")
        x = self.forward_layers(self.embed_tokens(input_ids, meta.positions), meta)
        idx = meta.logits_indices
        if idx is not None:
            x = x.index_select(0, idx.long())
        return self.compute_logits(x)

    def compute_logits(self, x: torch.Tensor) -> torch.Tensor:
        hn = latent.stream_add_norm(x.contiguous(), None, None, self.final_norm, self.cfg.norm_eps, self.dtype)
        return ops.linear(hn, self.embed).float()
