"""Divitar in the framework against the plain float64 oracle (tests/divitar_oracle.py): every mechanism alone, then the
model through the engine's scheduler, block pool and step — whole prompts, token-by-token decoding, portions down to
two tokens, unequal batches, reused pages and request slots, keys just inside / outside every window and chunk, at page
borders and far away, first tokens, long decoding, other geometries, greedy generation, shared prefixes, the checkpoint
layout and the trace runner.  The same tests run the CPU reference ops here and the HIP kernels on a GPU box."""
import copy
import json
import os
import subprocess
import sys

import pytest
import torch

import divitar_oracle as orc
from dgi import ops
from dgi.engine import EngineConfig, LLMEngine
from dgi.models import latent_mixer as lm
from dgi.models.config import (AttentionSpec, DenseSpec, DivitarConfig, LatentAttentionSpec, LayerSpec, MoeSpec, RotarySpec,
                               get_config)
from dgi.ops import latent, mix, moe
from dgi.runtime.batch import AttnMeta
from dgi.sched.request import SamplingParams

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]
F64 = torch.float64
I32 = torch.int32
RAMP = {"factor": 3.0, "original": 64.0, "fast": 6.0, "slow": 1.0}
A, L = "attention", "latent_attention"


def att(heads, kv_heads, dim, dims, chunk=0, base=100.0, factor=2.0, scale=None):
    return AttentionSpec(heads, kv_heads, dim, dim, scale or dim ** -0.5, RotarySpec(base, dims, {"factor": factor}, "half"),
                         "chunk" if chunk else "causal", chunk, gate_heads=True, shared_kv=True, qk_norm="none",
                         qk_norm_weight=False, bias=True)


def lat(heads, dim, rot_dim, vdim, kv_rank, window=0, kv_from=None, base=100.0, scale=None, ramp=RAMP):
    return LatentAttentionSpec(heads, dim, rot_dim, vdim, kv_rank, 0, scale or (dim + rot_dim) ** -0.5,
                               RotarySpec(base, rot_dim, ramp, "interleaved"), "window" if window else "causal", window,
                               kv_from=kv_from, sink=True)


def dense(ff):
    return DenseSpec(ff, act="relu_sq")


def experts(n, top, ff, shared, scale=1.0):
    return MoeSpec(n, 0, top, ff, shared, score="sigmoid", selection_bias=False, renorm=True, scale=scale)


def small_cfg(**kw) -> DivitarConfig:
    """Seven layers that differ in everything: group counts 1 / 2 / 3, rotated spans shorter than the head, chunks of
    5, 8 and 17, windows of 4, 9 and 23, two layers reading another's latent with their own heads and windows, experts
    with top 2 of 5 and top = all, with and without a shared expert, a layer without feed-forward; latent + key part of
    16 (vector kernel) and of 11 (element-wise)."""
    args = dict(name="t", vocab_size=53, hidden_size=32, layers=[
        LayerSpec(L, lat(3, 8, 4, 6, 12, window=9), dense(40)),
        LayerSpec(A, att(6, 2, 8, 4, chunk=8), experts(5, 2, 12, 20, 1.7)),
        LayerSpec(L, lat(2, 6, 4, 10, 12, window=4, kv_from=0), None),
        LayerSpec(A, att(3, 3, 7, 6, chunk=5, base=30.0, factor=5.0), experts(3, 3, 8, 0, 0.6)),
        LayerSpec(L, lat(1, 5, 2, 3, 9, window=23, ramp=dict(RAMP, factor=1.5)), experts(4, 1, 6, 8, 2.5)),
        LayerSpec(L, lat(5, 3, 4, 4, 12, window=9, kv_from=0), dense(24)),
        LayerSpec(A, att(4, 1, 12, 12, chunk=17), dense(16)),
    ], residual_mult=0.6, logit_scale=1.7, side_dim=6, norm_eps=1e-5, max_position=512)
    args.update(kw)
    return DivitarConfig(**args)


def engine(cfg, device, dtype=torch.float32, num_blocks=96, bs=4, seed=3, max_len=256, seqs=4, graphs=False, prefix=False):
    return LLMEngine(EngineConfig(model="divitar-test", device=device, dtype=dtype, block_size=bs, num_blocks=num_blocks,
                                  max_num_seqs=seqs, max_model_len=max_len, max_num_batched_tokens=max_len,
                                  enable_prefix_caching=prefix, use_graphs=graphs, token_align=0, decode_lookahead=graphs,
                                  seed=seed, graph_buckets=(1, 2, 4) if graphs else None), model_cfg=copy.deepcopy(cfg))


def toks(n, seed=0, vocab=53):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def config_dict(cfg: DivitarConfig) -> dict:
    """The design's config.json for ``cfg``."""
    layers = []
    for l in cfg.layers:
        m, f = l.mixer, l.mlp
        mixer = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale,
                 "rot": {"base": m.rot.base, "dims": m.rot.dims, "scaling": dict(m.rot.scaling)}}
        if m.mask_size:
            mixer["mask"] = {"size": m.mask_size}
        if l.type == A:
            mixer["kv_heads"] = m.kv_heads
        else:
            mixer.update(rot_dim=m.rot_dim, kv_rank=m.kv_rank)
            if m.kv_from is not None:
                mixer["kv_from"] = m.kv_from
        if f is None:
            mlp = None
        elif f.kind == "dense":
            mlp = {"kind": "dense", "ff": f.ff}
        else:
            mlp = {"kind": "moe", "expert": {"ff": f.ff}, "router": {"experts": f.experts, "top": f.top, "scale": f.scale}}
            if f.shared_ff:
                mlp["shared"] = {"ff": f.shared_ff}
        layers.append({"type": l.type, "mixer": mixer, "mlp": mlp})
    d = {"architecture": "Divitar", "vocab": cfg.vocab_size, "width": cfg.hidden_size, "norm": {"eps": cfg.norm_eps},
         "residual_mult": cfg.residual_mult, "logit_scale": cfg.logit_scale, "layers": layers}
    if cfg.side_dim:
        d["token_side"] = {"dim": cfg.side_dim}
    return d


def params(model) -> dict:
    """The model's weights under the checkpoint's tensor names (CPU, model dtype)."""
    P = {"embed": model.embed, "side.embed": model.side_embed, "head": model.head, "final.norm": model.final_norm}
    for i, w in enumerate(model.layers):
        p, m, f = f"l{i}.", w.spec.mixer, w.spec.mlp
        P[p + "norm1"], P[p + "norm2"] = w.norm1, w.norm2
        q = m.heads * (m.dim if w.spec.type == A else m.dim + m.rot_dim)
        P[p + "mix.q"], P[p + "mix.o"] = w.in_proj[:q], w.o
        if w.spec.type == A:
            k = m.kv_heads * m.dim
            P[p + "mix.k"], P[p + "mix.g"] = w.in_proj[q:q + k], w.in_proj[q + k:q + k + m.heads]
            P[p + "mix.q.b"], P[p + "mix.k.b"] = w.in_bias[:q], w.in_bias[q:q + k]
        else:
            if m.kv_from is None:
                P[p + "mix.dkv"] = w.in_proj[q:q + m.kv_rank + m.rot_dim]
                P[p + "mix.dkv.norm"] = w.dkv_norm
            P[p + "mix.uk"] = w.uk.reshape(m.heads * m.dim, m.kv_rank)
            P[p + "mix.uv"] = w.uv.reshape(m.heads * m.vdim, m.kv_rank)
            P[p + "mix.sink"] = w.sink
        if f is not None and f.kind == "dense":
            P[p + "mlp.up"], P[p + "mlp.down"] = w.up, w.down
        elif f is not None:
            P[p + "mlp.router"] = w.router
            for e in range(f.experts):
                P[f"{p}mlp.e{e}.gate"], P[f"{p}mlp.e{e}.up"] = w.gate_up[e, :f.ff], w.gate_up[e, f.ff:]
                P[f"{p}mlp.e{e}.down"] = w.down[e]
            if f.shared_ff:
                P[p + "mlp.shared.gate"], P[p + "mlp.shared.up"] = w.shared_gate_up[:f.shared_ff], w.shared_gate_up[f.shared_ff:]
                P[p + "mlp.shared.down"] = w.shared_down
        P[p + "side.gate"], P[p + "side.proj"], P[p + "side.norm"] = w.side_gate, w.side_proj, w.side_norm
    return {k: v.detach().cpu().contiguous() for k, v in P.items() if v is not None}


def oracle_logits(eng, tokens, layers=False, cfg=None):
    P = {k: v.to(F64) for k, v in params(eng.model).items()}
    return orc.forward(P, cfg or config_dict(eng.model_cfg), tokens, layers)


def feed_all(eng, rid, tokens, cuts):
    """Feed `tokens` in portions of the given sizes (the rest one by one); logits of every position."""
    out, at = [], 0
    for n in list(cuts) + [1] * len(tokens):
        if at >= len(tokens):
            break
        part = tokens[at:at + n]
        out.append(eng.feed([(rid, part, list(range(len(part))))])[0])
        at += len(part)
    return torch.cat(out, 0)


def close(a, b, tol):
    assert a.shape == b.shape
    err = (a.double().cpu() - b.double().cpu()).abs().max().item()
    assert err <= tol, f"max abs difference {err} > {tol}"


def rnd(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64) * scale


# ----------------------------------------------------------------------------------- mechanisms
def test_config_reads_every_size_and_rejects_bad_sharing():
    cfg = small_cfg()
    d = config_dict(cfg)
    c = DivitarConfig.from_dict(d, "t")
    c.max_position = cfg.max_position
    assert c == cfg
    assert c.kv_owners == [0, 1, 3, 4, 6]
    assert c.kv_layer_shapes() == [(1, 16, 0), (2, 8, 8), (3, 7, 7), (1, 11, 0), (1, 12, 12)]
    assert c.layers[1].mlp.renorm and c.layers[1].mlp.scale == 1.7 and c.layers[3].mlp.shared_ff == 0
    bare = copy.deepcopy(d)
    for k in ("residual_mult", "logit_scale", "token_side"):
        bare.pop(k)
    for l in bare["layers"]:
        l["mixer"].pop("mask")
        l["mixer"]["rot"].pop("scaling")
    c = DivitarConfig.from_dict(bare)
    assert (c.residual_mult, c.logit_scale, c.side_dim) == (1.0, 1.0, 0)
    assert all(l.mixer.mask_kind == "causal" and l.mixer.rot.scaling is None for l in c.layers)
    for li, key, val in ((2, "kv_from", 2), (5, "kv_from", 2), (5, "kv_from", 1), (5, "rot_dim", 2), (5, "kv_rank", 10),
                         (1, "vdim", 4), (1, "kv_heads", 4)):
        bad = copy.deepcopy(d)
        bad["layers"][li]["mixer"][key] = val
        with pytest.raises(ValueError):
            DivitarConfig.from_dict(bad)
    for path, val in ((("mixer", "rot", "dims"), 5), (("mixer", "rot", "dims"), 20), (("type",), "mamba")):
        bad = copy.deepcopy(d)
        at = bad["layers"][1]
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = val
        with pytest.raises(ValueError):
            DivitarConfig.from_dict(bad)
    bad = copy.deepcopy(d)
    bad["layers"][5]["mixer"]["rot"]["base"] = 7.0            # shares layer 0's key part, so it must turn like it
    with pytest.raises(ValueError):
        DivitarConfig.from_dict(bad)


@pytest.mark.parametrize("dims,base,scaling", [(8, 100.0, {"factor": 4.0}), (6, 50000.0, {"factor": 1.0}), (16, 500.0, RAMP),
                                               (4, 10000.0, {"factor": 2.0, "original": 2048.0, "fast": 32.0, "slow": 1.0}),
                                               (12, 1e6, {"factor": 8.0, "original": 4.0, "fast": 2.0, "slow": 1.5}), (10, 77.0, None)])
def test_rotary_tables(dims, base, scaling):
    """Linear and ramp scaling (a ramp inside the pairs, one that is empty, one wholly before / behind them)."""
    rot = {"dims": dims, "base": base, "scaling": scaling}
    t = ops.rope_cos_sin(dims, 300, base, scaling)
    ramp = scaling is not None and "fast" in scaling
    fs, stretch = orc.ramp_freqs(rot) if ramp else (orc.linear_freqs(rot), 1.0)
    a = torch.arange(300, dtype=F64)[:, None] * torch.tensor(fs, dtype=F64)
    close(t, torch.cat([a.cos(), a.sin()], -1) * stretch, 1e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [37, 64, 1024, 2052])
def test_residual_multiplier_and_embedding(device, dtype, W):
    T, eps, mult = 5, 1e-3, 0.37
    x0, y = rnd(T, W, seed=1), rnd(T, W, seed=2, scale=3.0).to(dtype)
    pw, nw = rnd(W, seed=3) + 1, rnd(W, seed=4) + 1
    tol = 1e-5 if dtype == torch.float32 else 0.008
    for post, nxt in ((None, nw), (pw, nw), (pw, None)):
        x = x0.float().to(device)
        got = latent.stream_add_norm(x, y.to(device), None if post is None else post.float().to(device),
                                     None if nxt is None else nxt.float().to(device), eps, dtype, mult=mult)
        add = y.to(F64) if post is None else orc.rms_norm(y.to(F64), post, eps)
        want = x0 + mult * add
        close(x, want, 1e-5)
        norm = want if nxt is None else orc.rms_norm(want, nxt, eps)
        close(got.float(), norm, tol * max(1.0, norm.abs().max().item()))
    table = rnd(11, W, seed=5).to(dtype)
    ids = torch.tensor([3, 0, 10, 3, 7], dtype=I32)
    close(latent.embed_rows(ids.to(device), table.to(device)), table.to(F64)[ids.long()], 1e-7)
    close(latent.embed_rows(ids.to(device), table.to(device), 2.5), 2.5 * table.to(F64)[ids.long()], 1e-5)
    close(latent.relu_sq(y.to(device)).float(), orc.relu_squared(y.to(F64)), 1e-4 if dtype == torch.float32 else 0.5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layout", ["half", "interleaved"])
@pytest.mark.parametrize("H,G,dk,dv,rd,shared", [(4, 2, 16, 16, 16, True), (3, 3, 7, 7, 4, True), (6, 1, 32, 32, 16, True),
                                                 (2, 1, 64, 64, 0, True), (4, 2, 24, 40, 16, False), (2, 2, 6, 9, 6, False)])
def test_rotary_write_with_values_from_raw_keys(device, dtype, layout, H, G, dk, dv, rd, shared):
    """q rotated in place, rotated keys into the key pages, the keys as projected (or the v columns) into the value
    pages; scattered slots, a row that is not written; 16-byte and element-wise paths."""
    T, bs, extra = 6, 4, 8
    pos = torch.tensor([0, 1, 37, 38, 100, 255], dtype=I32)
    slots = torch.tensor([5, 6, 12, -1, 27, 0], dtype=I32)
    n = (H + G) * dk + (0 if shared else G * dv)
    u = rnd(T, (n + extra + 7) // 8 * 8, seed=6).to(dtype)
    rot = {"dims": rd, "base": 60.0}
    cs = ops.rope_cos_sin(rd, 256, 60.0).to(device) if rd else None
    kc = torch.zeros(7, G, bs, dk, dtype=dtype, device=device)
    vc = torch.zeros(7, G, bs, dv, dtype=dtype, device=device)
    got = u.clone().to(device)
    mix.qk_rope(got, pos.to(device), slots.to(device), cs, H, G, dk, dv, kc, vc, layout=layout, shared=shared)
    got, kc, vc = got.cpu(), kc.cpu(), vc.cpu()
    turn = (lambda v, p: v) if rd == 0 else (lambda v, p: (orc.rotate_halves if layout == "half" else orc.rotate_pairs)(v, p, rot))
    tol = 1e-5 if dtype == torch.float32 else 0.03
    u64 = u.to(F64)
    for t in range(T):
        for h in range(H):
            close(got[t, h * dk:(h + 1) * dk].double(), turn(u64[t, h * dk:(h + 1) * dk], int(pos[t])), tol)
        s = int(slots[t])
        for g in range(G):
            k = u64[t, (H + g) * dk:(H + g + 1) * dk]
            v = k if shared else u64[t, (H + G) * dk + g * dv:(H + G) * dk + (g + 1) * dv]
            if s >= 0:
                close(kc[s // bs, g, s % bs].double(), turn(k, int(pos[t])), tol)
                close(vc[s // bs, g, s % bs].double(), v, 0)                        # values: bit for bit
    assert torch.equal(got[:, H * dk:], u[:, H * dk:])
    flat = kc.permute(0, 2, 1, 3).reshape(-1, G * dk)
    written = {int(s) for s in slots if s >= 0}
    assert all(flat[i].abs().sum() == 0 for i in range(flat.shape[0]) if i not in written)


def paged(rows_k, rows_v, bs, seed, dtype):
    """(k pages, v pages, page ids) of one sequence's keys / values [N, G, d] scattered over a pool."""
    N, G, _ = rows_k.shape
    nblk = (N + bs - 1) // bs
    perm = (torch.randperm(nblk, generator=torch.Generator().manual_seed(seed)) + 1).to(I32)
    kc = torch.zeros(nblk + 1, G, bs, rows_k.shape[2], dtype=dtype)
    vc = torch.zeros(nblk + 1, G, bs, rows_v.shape[2], dtype=dtype)
    for j in range(N):
        kc[int(perm[j // bs]), :, j % bs] = rows_k[j].to(dtype)
        vc[int(perm[j // bs]), :, j % bs] = rows_v[j].to(dtype)
    return kc, vc, perm


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,chunk", [(4, 2, 16, 64), (6, 2, 8, 17), (3, 3, 7, 5), (8, 1, 32, 100), (18, 1, 16, 40), (2, 2, 16, 0)])
def test_chunked_attention_rows_with_head_gates(monkeypatch, device, dtype, H, G, d, chunk):
    """Decode rows over scattered pages, one sigmoid gate per head.  For every query one key dominates a head's scores;
    it sits at the chunk's first place, just before it, at page borders, at position 0 or far back: seeing it or not
    changes the output completely."""
    N, bs, scale = 300, 4, 0.4
    queries = [299, 298, 200, 201, 255, 256, 64, 63, 1, 0, 136, 119]
    k, v = rnd(N, G, d, seed=8, scale=0.5), rnd(N, G, d, seed=9)
    q = rnd(len(queries), H * d + 8, seed=10)
    planted = {}
    for qi, p in enumerate(queries):
        lo = (p // chunk) * chunk if chunk else 0
        j = [lo, lo - 1, p - p % bs, max(0, p - 150), lo, lo - 1][qi % 6]
        if 0 <= j <= p and j not in planted.values() and j not in queries:
            planted[p] = j
            h = qi % H
            w = q[qi, h * d:(h + 1) * d]
            k[j, h // (H // G)] = w / w.norm() * 30
    gate = rnd(len(queries), H + 3, seed=11)
    k, v, q, gate = (t.to(dtype) for t in (k, v, q, gate))
    kc, vc, perm = paged(k, v, bs, 12, dtype)
    tables = perm[None, :].repeat(len(queries), 1).contiguous()
    out = mix.masked_attn_rows(q.to(device), kc.to(device), vc.to(device), tables.to(device), None,
                               torch.tensor(queries, dtype=I32, device=device), H, G, scale, chunk, gate.to(device)[:, :H],
                               gate_heads=True)
    # the same keys cut into runs over several workgroups
    monkeypatch.setattr(mix, "masked_split_runs", lambda rows, groups, keys: 3)
    runs = mix.masked_attn_rows(q.to(device), kc.to(device), vc.to(device), tables.to(device), None,
                                torch.tensor(queries, dtype=I32, device=device), H, G, scale, chunk, gate.to(device)[:, :H],
                                gate_heads=True, max_keys=N, sinks=torch.full((H,), -90.0, device=device))
    close(runs.float(), out.float(), 1e-5 if dtype == torch.float32 else 0.02)
    q64, k64, v64 = q.to(F64), k.to(F64), v.to(F64)
    for qi, p in enumerate(queries):
        lo = orc.chunk_start(p, chunk)
        for h in range(H):
            g = h // (H // G)
            pr = torch.softmax(k64[lo:p + 1, g] @ q64[qi, h * d:(h + 1) * d] * scale, 0)
            want = pr @ v64[lo:p + 1, g] * torch.sigmoid(gate[qi, h].to(F64))
            close(out[qi, h * d:(h + 1) * d], want, 1e-5 if dtype == torch.float32 else 0.04)
        if p in planted:
            j, h = planted[p], qi % H
            o = out[qi, h * d:(h + 1) * d].double().cpu() / torch.sigmoid(gate[qi, h].to(F64))
            hit = (o - v64[j, h // (H // G)]).norm() < 0.1 * v64[j, h // (H // G)].norm()
            assert hit == (lo <= j), (p, j, lo)


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,d,chunk", [(4, 2, 64, 100), (2, 1, 128, 64), (6, 3, 40, 77), (4, 4, 8, 30), (3, 1, 96, 1), (2, 2, 72, 0)])
def test_mfma_prompt_kernel_with_chunks_and_head_gates(H, G, d, chunk):
    """The MFMA prompt kernel with a chunk mask and one gate per head against the plain form: two portions on top of
    cached tokens, chunks that end inside 64-key tiles and span several, dominating keys at a chunk's edges."""
    bs, scale = 16, 0.2
    lens, ctx = [200, 77], [330, 77]
    tables = torch.zeros(2, 24, dtype=I32)
    q = rnd(sum(lens), (H * d + H + 7) // 8 * 8, seed=20, scale=0.5).to(torch.bfloat16)
    gate = q[:, H * d:H * d + H]
    caches, base = [], 1
    data = []
    for b, c in enumerate(ctx):
        k, v = rnd(c, G, d, seed=21 + b, scale=0.5).to(torch.bfloat16), rnd(c, G, d, seed=23 + b).to(torch.bfloat16)
        if b == 0 and chunk > 1:
            r = 150                                             # row 150 of the first portion sits at position 280
            lo = 280 // chunk * chunk
            k[lo, 0] = (q[r, :d].float() * 6).to(torch.bfloat16)
            k[lo - 1, 0] = (q[r, :d].float() * 9).to(torch.bfloat16)
        kc, vc, perm = paged(k, v, bs, 30 + b, torch.bfloat16)
        tables[b, :len(perm)] = perm - 1 + base
        base += len(perm)
        caches.append((kc[1:], vc[1:]))
        data.append((k.to(F64), v.to(F64)))
    z = lambda t: torch.zeros_like(t[:1])                       # noqa: E731
    kc = torch.cat([z(caches[0][0])] + [c[0] for c in caches])
    vc = torch.cat([z(caches[0][1])] + [c[1] for c in caches])
    cu = torch.tensor([0, lens[0], sum(lens)], dtype=I32)
    out = mix.paged_prefill_masked(q.cuda(), kc.cuda(), vc.cuda(), tables.cuda(), cu.cuda(), torch.tensor(ctx, dtype=I32).cuda(), H, G,
                                   scale, chunk, gate.cuda(), gate_heads=True)
    q64 = q.to(F64)
    for b in range(2):
        k, v = data[b]
        for i in range(0, lens[b], 7):
            p, t = ctx[b] - lens[b] + i, int(cu[b]) + i
            lo = orc.chunk_start(p, chunk)
            for h in range(H):
                g = h // (H // G)
                pr = torch.softmax(k[lo:p + 1, g] @ q64[t, h * d:(h + 1) * d] * scale, 0)
                close(out[t, h * d:(h + 1) * d], pr @ v[lo:p + 1, g] * torch.sigmoid(gate[t, h].to(F64)), 0.04)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kr,rd,q0,pad", [(12, 4, 10, 3), (64, 32, 24, 8), (9, 2, 5, 3), (520, 8, 16, 0), (1048, 16, 8, 8), (24, 8, 16, 0)])
def test_latent_write_without_a_query_latent(device, dtype, kr, rd, q0, pad):
    """Latent norm + rotary of the key part into scattered slots, from columns behind the query projection."""
    T, eps, bs = 5, 1e-4, 4
    u = rnd(T, q0 + kr + rd + pad, seed=5).to(dtype)
    w = rnd(kr, seed=7) + 1
    pos = torch.tensor([0, 1, 30, 31, 200], dtype=I32)
    slots = torch.tensor([9, 10, 4, -1, 0], dtype=I32)
    rot = {"dims": rd, "base": 50.0, "scaling": RAMP}
    cache = torch.zeros(4, 1, bs, kr + rd, dtype=dtype, device=device)
    got = latent.latent_prep(u.to(device)[:, q0:], 0, kr, rd, None, w.float().to(device), eps, pos.to(device), slots.to(device),
                             ops.rope_cos_sin(rd, 256, 50.0, RAMP).to(device), True, cache)
    assert got is None
    flat = cache.cpu().view(-1, kr + rd)
    u64 = u.to(F64)
    for t in range(T):
        if slots[t] >= 0:
            want = torch.cat([orc.rms_norm(u64[t, q0:q0 + kr], w, eps), orc.rotate_pairs(u64[t, q0 + kr:q0 + kr + rd], int(pos[t]), rot)])
            close(flat[int(slots[t])], want, 1e-5 if dtype == torch.float32 else 0.03)
    assert {i for i in range(16) if flat[i].abs().sum() > 0} == {0, 4, 9, 10}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dim,rd,kr,window", [(3, 8, 4, 12, 5), (2, 4, 6, 8, 0), (5, 6, 2, 9, 17), (6, 16, 16, 32, 64),
                                                (19, 8, 32, 64, 33), (4, 24, 16, 144, 129)])
def test_latent_rows_with_sinks(device, dtype, H, dim, rd, kr, window):
    """Rows on cached latents with a learned logit per head in the denominator: ordinary sinks, one that takes nearly all
    the weight, one that takes none; keys in one run and cut into several; first tokens (a single visible key)."""
    N, bs, scale = 300, 4, 0.3
    queries = [299, 298, 255, 256, 130, 64, 1, 0]
    T = len(queries)
    c, r = rnd(N, kr, seed=12, scale=0.5).to(dtype), rnd(N, rd, seed=13, scale=0.5).to(dtype)
    q = rnd(T, H * (dim + rd), seed=15).to(dtype)
    q_lat = rnd(H, T, kr, seed=16).to(dtype)
    sinks = rnd(H, seed=17) + 1.0
    sinks[0], sinks[1 % H] = 40.0, -40.0
    rot = {"dims": rd, "base": 100.0, "scaling": RAMP}
    cs = ops.rope_cos_sin(rd, 512, 100.0, RAMP).to(device)
    cache, _v, perm = paged(torch.cat([c, r], 1)[:, None], torch.zeros(N, 1, 1), bs, 18, dtype)
    tables = perm[None, :].repeat(T, 1).contiguous().to(device)
    pos = torch.tensor(queries, dtype=I32, device=device)
    want = torch.zeros(H, T, kr, dtype=F64)
    for t, p in enumerate(queries):
        lo = orc.window_start(p, window)
        for h in range(H):
            qr = orc.rotate_pairs(q[t].to(F64).view(H, -1)[h, dim:], p, rot)
            s = (c[lo:p + 1].to(F64) @ q_lat[h, t].to(F64) + r[lo:p + 1].to(F64) @ qr) * scale
            want[h, t] = orc.softmax_with_sink(s, sinks[h]) @ c[lo:p + 1].to(F64)
    tol = 2e-5 if dtype == torch.float32 else 0.05
    for max_keys in (0, N):
        out = torch.full((H, T, kr), 7.0, dtype=dtype, device=device)
        latent.latent_attn_rows(q.to(device), q_lat.to(device), cache.to(device), tables, None, pos, H, dim, rd, kr, scale, window, cs,
                                True, out, max_keys=max_keys, sinks=sinks.float().to(device))
        close(out, want, tol)
    assert want[0].abs().max() < 1e-6 and want[1 % H].abs().max() > 0.1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dim,rd,dv,kr", [(3, 5, 2, 7, 9), (4, 16, 8, 24, 32), (2, 32, 32, 64, 48)])
def test_latent_pages_layout(device, dtype, H, dim, rd, dv, kr):
    n, bs = 3, 4
    lat_, kv = rnd(n * bs, kr + rd, seed=1).to(dtype), rnd(n * bs, H * (dim + dv), seed=2).to(dtype)
    kt, vt = (t.cpu() for t in latent.latent_pages(kv.to(device), lat_.to(device), bs, H, dim, rd, dv))
    for p in range(n):
        for s in range(bs):
            for h in range(H):
                row = kv[p * bs + s]
                assert torch.equal(kt[p, h, s], torch.cat([row[h * dim:(h + 1) * dim], lat_[p * bs + s, kr:]]))
                assert torch.equal(vt[p, h, s], row[H * dim + h * dv:H * dim + (h + 1) * dv])


@pytest.mark.parametrize("window", [0, 1, 5, 16, 33, 1000])
@pytest.mark.parametrize("hints", [True, False])
def test_visible_pages_cover_every_visible_key(window, hints):
    """Whatever the window and the cut of the prompt, every key that some row of a portion sees maps to the page that
    holds it, and a short window lists few pages."""
    bs, mb = 4, 60
    lens, ctx = [1, 7, 40, 2], [1, 100, 133, 240]
    tables = torch.stack([torch.randperm(500, generator=torch.Generator().manual_seed(b))[:mb] + 1 for b in range(4)]).to(I32)
    cu = torch.tensor([0, 1, 8, 48, 50], dtype=I32)
    meta = AttnMeta(torch.zeros(50, dtype=I32), torch.zeros(50, dtype=I32), 0, num_prefill_tokens=50, pre_block_tables=tables,
                    pre_cu_seqlens=cu, pre_context_lens=torch.tensor(ctx, dtype=I32), pre_max_len=40 if hints else 0,
                    pre_max_context=240 if hints else 0)
    m = lat(1, 2, 2, 2, 2, window=window)
    listed, table = lm.visible_pages(m, meta, bs)
    assert table.dtype == I32 and table.shape == tables.shape
    assert 0 <= int(table.min()) and int(table.max()) < listed.numel()
    for b in range(4):
        for j in range(orc.window_start(ctx[b] - lens[b], window), ctx[b]):
            assert int(listed[int(table[b, j // bs])]) == int(tables[b, j // bs])
    if hints and 0 < window <= 33:
        assert listed.numel() <= 4 * ((40 + window) // bs + 2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,top,scale", [(6, 2, 1.0), (5, 5, 2.5), (70, 3, 0.3), (4, 1, 1.7)])
def test_renormalised_sigmoid_routing(device, E, top, scale):
    z = rnd(9, E, seed=3, scale=2.0).float()
    z[2] = -60.0                                                   # every score almost zero
    z[3] = -120.0                                                  # every score zero in fp32: the sum's 1e-20 decides
    idx, w = moe.moe_route(z.to(device), None, top, score="sigmoid", renorm=True, scale=scale)
    for t in range(9):
        if t == 3:
            assert torch.isfinite(w[t]).all() and w[t].abs().max() <= scale
            continue
        es, ws = orc.route(z[t].to(F64), top, scale)
        assert idx[t].tolist() == es
        close(w[t], torch.stack(ws), 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,E,top,W", [(1, 6, 2, 24), (16, 16, 16, 64), (37, 17, 3, 520), (100, 64, 8, 40), (33, 48, 5, 1032),
                                       (9, 70, 4, 64), (5, 33, 1, 20), (40, 1, 1, 8)])
def test_router_logits_and_choice(device, dtype, T, E, top, W):
    """Rows straight to routes and weights, with a router that bf16 holds exactly and with one that it does not: fp32
    logits either way, so the choice is the plain one wherever the scores are apart."""
    h = rnd(T, W + 8, seed=50).to(dtype)[:, :W]
    for exact in (True, False):
        router = rnd(E, W, seed=51, scale=2 * W ** -0.5).float()
        if exact:
            router = router.to(torch.bfloat16).float()
        rb = moe.exact_bf16(router)
        assert (rb is not None) == exact
        idx, w = moe.moe_router(h.to(device), router.to(device), None if rb is None else rb.to(device), top, True, 1.3)
        for t in range(T):
            z = router.to(F64) @ h[t].to(F64)
            es, ws = orc.route(z, top, 1.3)
            gap = torch.sort(torch.sigmoid(z), descending=True).values
            if top < E and gap[top - 1] - gap[top] < 1e-5:
                continue
            assert sorted(idx[t].tolist()) == sorted(es)
            got = dict(zip(idx[t].tolist(), w[t].tolist()))
            assert all(abs(got[e] - float(x)) < 1e-5 for e, x in zip(es, ws))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,E,top,W,ff", [(1, 6, 2, 24, 12), (5, 6, 2, 24, 16), (70, 6, 3, 40, 72), (40, 3, 3, 136, 8), (3, 70, 8, 64, 24),
                                          (300, 5, 2, 72, 40), (900, 4, 2, 64, 96), (33, 1, 1, 16, 264), (257, 2, 1, 200, 136)])
def test_experts_every_path(device, dtype, T, E, top, W, ff):
    """Gated-SiLU experts with weights on the outputs and a shared addend, few and many rows per expert (every tile size of
    the grouped products, widths that end inside a tile), experts that nobody chose, one expert, top = all."""
    h = rnd(T, W, seed=30).to(dtype)
    gu, dn = rnd(E, 2 * ff, W, seed=32, scale=W ** -0.5).to(dtype), rnd(E, W, ff, seed=33, scale=ff ** -0.5).to(dtype)
    shared = rnd(T, W, seed=34).to(dtype)
    z = rnd(T, E, seed=31, scale=1.5).float()
    if E > 3:
        z[:, 2] = -30.0                                            # nobody takes expert 2
    idx, wts = moe.moe_route(z.to(device), None, top, score="sigmoid", renorm=True, scale=1.4)
    got = moe.moe_experts(h.to(device), idx, wts, gu.to(device), dn.to(device), shared.to(device)).float().cpu()
    P = {}
    for e in range(E):
        P[f"e{e}.gate"], P[f"e{e}.up"], P[f"e{e}.down"] = gu[e, :ff].to(F64), gu[e, ff:].to(F64), dn[e].to(F64)
    want = shared.to(F64)
    ys = [orc.glu(P, f"e{e}", h.to(F64)) for e in range(E)]
    for t in range(T):
        for e, w in zip(idx[t].tolist(), wts[t].tolist()):
            want[t] += w * ys[e][t]
    close(got, want, 2e-5 if dtype == torch.float32 else 0.05)


@pytest.mark.gpu
@pytest.mark.parametrize("tile", [16, 32, 64, 128])
@pytest.mark.parametrize("T,E,top,W,ff", [(150, 5, 2, 72, 40), (7, 12, 3, 64, 136), (260, 3, 1, 320, 264)])
def test_grouped_products_every_tile(monkeypatch, tile, T, E, top, W, ff):
    """Every tile size on the same experts, with the clamped activation and the weights on the inputs too; identity routes
    (no expert of their own) pass through the sort."""
    h = rnd(T, W, seed=40).to(torch.bfloat16)
    gu, dn = rnd(E, 2 * ff, W, seed=41, scale=W ** -0.5).to(torch.bfloat16), rnd(E, W, ff, seed=42, scale=ff ** -0.5).to(torch.bfloat16)
    wts = rnd(T, top, seed=43).abs().float()
    monkeypatch.setattr(moe, "group_tile", lambda p, e, w: tile)
    for act, weigh, routes in (("silu", "output", E + 2), ("clamped", "input", max(E, top))):
        idx = torch.stack([torch.randperm(routes, generator=torch.Generator().manual_seed(t))[:top] for t in range(T)]).to(I32)
        kw = dict(act=act, limit=0.8, weigh=weigh)
        got = moe.moe_experts(h.cuda(), idx.cuda(), wts.cuda(), gu.cuda(), dn.cuda(), None, **kw)
        close(got.float(), moe.moe_experts(h, idx, wts, gu, dn, None, **kw).float(), 0.06)


# ----------------------------------------------------------------------------------- the model in the engine
@pytest.mark.parametrize("device", DEVICES)
def test_layer_streams_match_oracle(device):
    eng = engine(small_cfg(), device)
    t = toks(29, 1)
    eng.model.capture_layers = tuple(range(7))
    got = eng.feed([("a", t, list(range(len(t))))], ["a"])[0]
    want, streams = oracle_logits(eng, t, True)
    for i, s in enumerate(streams):
        close(eng.model.captured[i], s, 2e-4)
    close(got, want, 3e-4)


VARIANTS = {
    "base": {},
    "no_side_plain_scales": {"side_dim": 0, "residual_mult": 1.0, "logit_scale": 1.0},
    "one_latent_layer": {"layers": [LayerSpec(L, lat(1, 1, 2, 1, 1, window=1), None)]},       # sizes of one, a window of one
    "one_attention_layer": {"layers": [LayerSpec(A, att(1, 1, 2, 2, chunk=1), None)]},        # chunks of one token
    "no_masks": {"layers": [LayerSpec(A, att(4, 2, 8, 4), dense(8)), LayerSpec(L, lat(2, 3, 2, 4, 12), experts(2, 2, 8, 4)),
                            LayerSpec(L, lat(1, 2, 2, 4, 12, kv_from=1), None)]},
    "vector_sizes": {"layers": [LayerSpec(L, lat(4, 16, 8, 16, 24, window=11), dense(64)),
                                LayerSpec(A, att(8, 4, 16, 16, chunk=13), experts(8, 1, 16, 32)),
                                LayerSpec(L, lat(8, 8, 8, 8, 24, window=6, kv_from=0), experts(6, 4, 24, 16, 1.5)),
                                LayerSpec(A, att(2, 2, 32, 16, chunk=32), dense(32))], "hidden_size": 64, "side_dim": 16},
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("variant", list(VARIANTS))
def test_whole_decode_and_portions_match_oracle(device, variant):
    """Whole prompt, token by token, and portions of several sizes (down to two tokens, across pages, windows and
    chunks): all equal the oracle; other layer orders and sizes too."""
    eng = engine(small_cfg(**VARIANTS[variant]), device)
    t = toks(45, 2)
    want = oracle_logits(eng, t)
    close(eng.feed([("w", t, list(range(len(t))))], ["w"])[0], want, 4e-4)
    for name, cuts in (("d", [1]), ("p", [2, 2, 7, 3, 16, 2, 5]), ("q", [30, 2]), ("r", [1, 13])):
        got = feed_all(eng, name, t, cuts)
        eng.feed([], [name])
        close(got, want, 4e-4)
    assert eng.pool.num_used == 0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_batches_reuse_pages(device, dtype):
    """Six requests of different lengths through four places and a pool too small for all of them: portions beside
    single tokens, requests sitting steps out, steps in which nothing is asked for, pages used again — every position
    equals the request run alone."""
    eng = engine(small_cfg(), device, dtype=dtype, num_blocks=40, bs=4)
    solo = engine(small_cfg(), device, dtype=dtype)
    solo.model.copy_from(eng.model)
    lens = {"a": 41, "b": 7, "c": 30, "d": 2, "e": 23, "f": 35}
    seqs = {k: toks(n, 10 + i) for i, (k, n) in enumerate(lens.items())}
    want = {k: solo.feed([(k, v, list(range(len(v))))], [k])[0] for k, v in seqs.items()}
    plan = [[("a", 5), ("b", 2)], [("a", 1), ("b", 1), ("c", 9), ("d", 2)], [("a", 17), ("c", 1)],
            [("b", 4), ("c", 2), ("a", 1), ("e", 3)], [("e", 20), ("a", 17)], [("c", 18), ("f", 6)], [("f", 1)], [("f", 28)]]
    at = {k: 0 for k in seqs}
    got = {k: [] for k in seqs}
    for si, step in enumerate(plan):
        entries, end = [], []
        for k, n in step:
            part = seqs[k][at[k]:at[k] + n]
            entries.append((k, part, [] if si == 2 else list(range(len(part)))))
            at[k] += n
            if at[k] == len(seqs[k]):
                end.append(k)
        for (k, part, _w), out in zip(entries, eng.feed(entries, end)):
            got[k].append(want[k][at[k] - len(part):at[k]] if si == 2 else out)
    assert at == lens and eng.pool.num_used == 0
    if dtype == torch.float32:
        for k in seqs:
            close(torch.cat(got[k], 0), want[k], 2e-4)
        close(want["a"], oracle_logits(solo, seqs["a"]), 4e-4)
    else:       # an expert choice that flips on a close call moves a whole row: rows are judged by their median
        for k in seqs:
            assert (torch.cat(got[k], 0) - want[k]).abs().amax(1).median().item() < 0.1


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens_and_long_decoding(device):
    """A sequence of one token; 137 single-token steps, far past every window and chunk (23 at most) and over many pages."""
    eng = engine(small_cfg(), device, max_len=256)
    t = toks(140, 5)
    want = oracle_logits(eng, t)
    close(eng.feed([("one", t[:1], [0])], ["one"])[0], want[:1], 2e-4)
    got = feed_all(eng, "x", t, [3])
    close(got, want, 4e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["window", "chunk", "sink", "values"])
def test_edges_and_sinks_decide_the_logits(device, kind):
    """One layer whose softmax is sharp: the logits follow the oracle (prompt rows, portions and decode rows), and the
    oracle with a mask that is one token longer or shorter, with another sink, or — for the values — fed with rotated
    keys in their place, differs clearly; so a fault of that kind could not hide."""
    if kind in ("window", "sink"):
        layer = LayerSpec(L, lat(2, 4, 2, 4, 6, window=6, scale=6.0 if kind == "window" else 1.0), None)
    else:
        layer = LayerSpec(A, att(2, 1, 6, 4, chunk=6, scale=6.0), None)
    eng = engine(small_cfg(layers=[layer], side_dim=0), device, bs=4)
    if kind == "sink":
        eng.model.layers[0].sink.copy_(torch.tensor([3.0, -2.0]))
    t = toks(30, 9)
    want = oracle_logits(eng, t)
    close(eng.feed([("w", t, list(range(30)))], ["w"])[0], want, 5e-4)
    close(feed_all(eng, "d", t, [9, 2]), want, 5e-4)
    P = {k: v.to(F64) for k, v in params(eng.model).items()}
    d = config_dict(eng.model_cfg)
    if kind in ("window", "chunk"):
        for other in (5, 7):
            d["layers"][0]["mixer"]["mask"]["size"] = other
            assert (orc.forward(P, d, t) - want)[8:].abs().max() > 0.05
    elif kind == "sink":
        P["l0.mix.sink"] = torch.full((2,), -100.0, dtype=F64)
        assert (orc.forward(P, d, t) - want)[1:].abs().max() > 0.05
    else:
        real = orc.attention

        def rotated_values(P_, pre, m, h):          # the mistake: values taken after rotation
            T, H, G, dd = h.shape[0], int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
            q = (h @ P_[pre + "mix.q"].T + P_[pre + "mix.q.b"]).view(T, H, dd)
            k = (h @ P_[pre + "mix.k"].T + P_[pre + "mix.k.b"]).view(T, G, dd)
            kr = torch.stack([orc.rotate_halves(k[i, 0], i, m["rot"]) for i in range(T)])
            g = torch.sigmoid(h @ P_[pre + "mix.g"].T)
            out = torch.zeros(T, H * dd, dtype=F64)
            for i in range(T):
                lo = orc.chunk_start(i, int(m["mask"]["size"]))
                for hh in range(H):
                    s = kr[lo:i + 1] @ orc.rotate_halves(q[i, hh], i, m["rot"]) * float(m["scale"])
                    out[i, hh * dd:(hh + 1) * dd] = torch.softmax(s, 0) @ kr[lo:i + 1] * g[i, hh]
            return out @ P_[pre + "mix.o"].T
        orc.attention = rotated_values
        try:
            assert (orc.forward(P, d, t) - want)[1:].abs().max() > 0.05
        finally:
            orc.attention = real


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_scheduler(device):
    eng = engine(small_cfg(), device, max_len=128)
    prompts = [toks(9, 20), toks(17, 21), toks(3, 22)]
    reqs = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True))
    P = {k: v.to(F64) for k, v in params(eng.model).items()}
    cd = config_dict(eng.model_cfg)
    for p, r in zip(prompts, reqs):
        lg = orc.forward(P, cd, list(p) + r.output[:-1])[len(p) - 1:]
        for tok, row in zip(r.output, lg):
            top2 = torch.topk(row, 2).values
            assert tok == int(row.argmax()) or (top2[0] - top2[1]) < 1e-3
    assert eng.pool.num_used == 0


@pytest.mark.parametrize("device", DEVICES)
def test_shared_prefix_pages(device):
    """A sequence carries nothing but pages, so prompts that share a prefix share its pages: the second prompt starts
    from the first one's and generates what it generates without sharing."""
    plain, shared = engine(small_cfg(), device, max_len=128), engine(small_cfg(), device, max_len=128, prefix=True)
    shared.model.copy_from(plain.model)
    head = toks(33, 40)
    sp = SamplingParams(max_tokens=6, temperature=0.0, ignore_eos=True)
    prompts = [head + toks(5, 41), head + toks(9, 42)]
    want = [plain.generate([p], sp)[0].output for p in prompts]
    assert [shared.generate([p], sp)[0].output for p in prompts] == want
    assert shared.stats["prefill_tokens"] < sum(len(p) for p in prompts)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_decode_equals_eager_decode(dtype):
    """Decode steps replayed as hipGraphs produce the tokens of the eager engine; replays follow each other with eager
    prompt steps between them, pages reused by later batches."""
    cfg = small_cfg(**VARIANTS["vector_sizes"])
    eager, graph = engine(cfg, "cuda", dtype, max_len=128), engine(cfg, "cuda", dtype, max_len=128, graphs=True)
    graph.model.copy_from(eager.model)
    prompts = [toks(9, 60), toks(17, 61), toks(3, 62)]
    sp = SamplingParams(max_tokens=14, temperature=0.0, ignore_eos=True)
    want = [r.output for r in eager.generate(prompts, sp)]
    for _ in range(3):
        assert [r.output for r in graph.generate(prompts, sp)] == want
    assert graph.runner.graphs is not None and graph.runner.graphs.captured
    assert graph.pool.num_used == 0


def test_preempted_sequence_is_recomputed():
    cfg = small_cfg()
    big = engine(cfg, "cpu", max_len=128)
    sp = SamplingParams(max_tokens=20, temperature=0.0, ignore_eos=True)
    ref = big.generate([toks(20, 30), toks(22, 31)], sp)
    tight = engine(cfg, "cpu", num_blocks=18, bs=4, max_len=128)
    tight.model.copy_from(big.model)
    got = tight.generate([toks(20, 30), toks(22, 31)], sp)
    assert tight.scheduler.num_preemptions > 0
    assert [r.output for r in got] == [r.output for r in ref]


def write_checkpoint(eng, path):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config_dict(eng.model_cfg), f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in params(eng.model).items()},
              os.path.join(path, "model.safetensors"))


def test_checkpoint_layout_and_trace_runner(tmp_path):
    """config.json + safetensors in the design's naming -> registry, loader, engine; the replay command writes the
    logits of the wanted places, step by step."""
    src = engine(small_cfg(), "cpu", dtype=torch.bfloat16)          # bf16 weights survive the file bit for bit
    ck = str(tmp_path / "model")
    write_checkpoint(src, ck)
    cfg = get_config(ck)
    assert isinstance(cfg, DivitarConfig) and cfg.kv_owners == [0, 1, 3, 4, 6]
    eng = LLMEngine(EngineConfig(model=ck, device="cpu", dtype=torch.float32, block_size=4, num_blocks=64, max_num_seqs=4,
                                 max_model_len=128, max_num_batched_tokens=128, enable_prefix_caching=False, use_graphs=False, token_align=0))
    assert eng.model.load_info["tensors"] == len(params(src.model))
    t = toks(21, 40)
    want = oracle_logits(eng, t)
    close(eng.feed([("a", t, list(range(len(t))))], ["a"])[0], want, 4e-4)
    out = tmp_path / "out"
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": t[:6], "want": [0, 5]}, {"id": "y", "tokens": t[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": t[6:7], "want": [0]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": t[7:], "want": [13]}], "end": ["x"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", ck, "--dtype", "float32", "--out",
                        str(out), "--max-tokens", "64", "--device", "cpu"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    import numpy as np
    for step, rows in ((0, [0, 5]), (1, [6]), (2, [20])):
        got = torch.from_numpy(np.fromfile(str(out / f"{step}.f32"), dtype="<f4").reshape(len(rows), -1))
        close(got, want[rows], 4e-4)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("variant", ["base", "vector_sizes"])
def test_kernels_match_the_reference_ops_on_a_prompt_batch(dtype, variant):
    """The HIP kernels against the CPU reference ops through the same engine code, over a batch of portions and decode
    rows: fp32 within rounding at every position; bf16 at the typical position."""
    cfg = small_cfg(**VARIANTS[variant])
    cpu, gpu = engine(cfg, "cpu", dtype=dtype), engine(cfg, "cuda", dtype=dtype)
    cpu.model.copy_from(gpu.model)
    a, b = toks(50, 50), toks(33, 51)
    for eng in (cpu, gpu):
        eng.out = [eng.feed([("a", a[:40], list(range(40))), ("b", b[:2], [0, 1])]),
                   eng.feed([("a", a[40:41], [0]), ("b", b[2:], list(range(31)))]),
                   eng.feed([("a", a[41:], list(range(9)))], ["a", "b"])]
    x = torch.cat([u for o in cpu.out for u in o], 0)
    y = torch.cat([v for o in gpu.out for v in o], 0).cpu()
    if dtype == torch.float32:
        close(y, x, 4e-4)
    else:
        assert (y - x).abs().amax(1).median().item() < 0.1


@pytest.mark.gpu
def test_mfma_prompt_path_of_latent_layers(monkeypatch):
    """Long bf16 portions of latent layers run on expanded pages and the MFMA kernel: same logits as the rows on the
    cached latents (portions on top of cached tokens, two prompts and a decode row in one step, windows shorter than the
    prompt, key and value sizes that differ, sinks, a shared latent)."""
    cfg = small_cfg(hidden_size=64, layers=[
        LayerSpec(L, lat(4, 32, 32, 64, 40, window=70), dense(64)),
        LayerSpec(L, lat(2, 48, 32, 72, 40, window=33, kv_from=0), None),
        LayerSpec(A, att(4, 2, 64, 32, chunk=50), dense(32)),
        LayerSpec(L, lat(3, 16, 16, 24, 24, window=130), dense(64))])
    a, b, c = toks(200, 70), toks(90, 71), toks(40, 72)

    def run():
        eng = engine(cfg, "cuda", dtype=torch.bfloat16, num_blocks=64, bs=16, max_len=512)
        for w in eng.model.layers:
            if w.sink is not None:
                w.sink.copy_(torch.linspace(-1.0, 4.0, w.sink.numel()))
        out = [eng.feed([("a", a[:150], list(range(150))), ("c", c[:39], [38])]),
               eng.feed([("a", a[150:], list(range(50))), ("b", b, list(range(90))), ("c", c[39:], [0])], ["a", "b", "c"])]
        return torch.cat([o for step in out for o in step], 0), oracle_logits(eng, a)

    calls = []
    real = lm.prompt_heads
    monkeypatch.setattr(lm, "prompt_heads", lambda *x, **k: (calls.append(1), real(*x, **k))[1])
    fast, want = run()
    assert len(calls) == 6                                   # every latent layer of both steps
    monkeypatch.setattr(lm, "MFMA_PROMPT_ROWS", 1 << 30)
    slow, _ = run()
    assert len(calls) == 6
    close(fast, slow, 0.06 * max(1.0, slow.abs().max().item()))
    close(fast[:150], want[:150], 0.1 * max(1.0, want.abs().max().item()))


def test_bench_arch_compare_option_runs():
    """`bench.py --arch-compare divitar` (tiny size, CPU): one JSON line with a row per model and phase numbers."""
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bench.py"), "--arch-compare", "divitar", "--arch-sizes", "tiny",
                        "--prompt-len", "40", "--concurrency", "2", "--steps", "2", "--warmup", "1",
                        "--max-batched-tokens", "128"], capture_output=True, text=True, timeout=600,
                       env={**os.environ, "CUDA_VISIBLE_DEVICES": "", "HIP_VISIBLE_DEVICES": ""})
    assert r.returncode == 0, r.stderr[-2000:]
    out = json.loads(r.stdout.strip().splitlines()[-1])
    assert [x["model"] for x in out["rows"]] == ["divitar", "depelix", "llama"]
    assert all(x["prefill_tok_s"] > 0 and x["decode_tok_s"] > 0 for x in out["rows"])


def test_worker_engine_serves_a_checkpoint_dir(tmp_path):
    """The worker's native engine picks the model class from config.json and generates through the same LLMEngine."""
    sys.path.insert(0, os.path.join(ROOT, "worker"))
    from engines.llm_native import NativeLLMEngine
    d = str(tmp_path / "ckpt")
    write_checkpoint(engine(small_cfg(vocab_size=300), "cpu", torch.bfloat16), d)
    e = NativeLLMEngine({"model_id": d, "device": "cpu", "max_model_len": 128, "max_num_batched_tokens": 128,
                         "num_blocks": 64, "max_num_seqs": 4})
    e.load_model()
    assert type(e.engine.model).__name__ == "DivitarModel"
    out = e.batch_inference([{"messages": [{"role": "user", "content": "hi"}], "max_tokens": 5, "temperature": 0.0}])
    assert out[0]["usage"]["completion_tokens"] == 5


def test_split_plan_of_decode_rows():
    assert mix.masked_split_runs(32, 8, 8192) == 1 and mix.masked_split_runs(1, 8, 8192) == 16
    assert mix.masked_split_runs(1, 1, 500) == 1 and mix.masked_split_runs(4, 2, 1 << 20) == 32
