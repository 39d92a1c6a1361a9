"""Dibizen's side of bench.py --design: the Llama of equal size and the
kernel pairs, at the sizes of the model's first layer of each kind.

Like kernels: Llama's attention for attention and for the recurrences, dense
products of the same weights (decode) or of the same rows (prompts) for the
experts', its elementwise and norm kernels for the others.
"""
from __future__ import annotations

from typing import Dict

import numpy as np
import torch

from helix_amd import ops
from helix_amd.engine.design_bench import _row, _time
from helix_amd.engine.design_bench_hybrid import _prefill_meta
from helix_amd.models.dibizen import DibizenConfig
from helix_amd.models.gla import LightningSpec
from helix_amd.models.llama import LlamaConfig
from helix_amd.models.mixer_group import MixerGroup
from helix_amd.models.moe import Mixture
from helix_amd.models.rotary_attention import AttnSpec, RotaryTables
from helix_amd.models.selective import SelectiveSpec
from helix_amd.ops import gated, routed


def _spec(l):
    return l.mixer.members[0].spec


def _first(z: DibizenConfig, kind):
    return next(l for l in z.layers if isinstance(_spec(l), kind))


def twin(z: DibizenConfig) -> LlamaConfig:
    """Same width, depth, vocabulary and attention heads; a dense
    feed-forward with the weights that a token's experts have (three
    matrices instead of two)."""
    l = _first(z, AttnSpec)
    m = _spec(l)
    return LlamaConfig(
        name=f"llama-as-{z.name}", vocab_size=z.vocab_size,
        hidden_size=z.hidden_size, num_layers=z.num_layers,
        intermediate_size=l.ff.ff * l.ff.router.top * 2 // 3,
        num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim,
        max_position=z.max_position)


@torch.inference_mode()
def kernels(z: DibizenConfig, device, decode_batch: int = 256,
            decode_len: int = 1024, prompts: int = 8,
            prompt_len: int = 2048) -> Dict[str, dict]:
    W, S, bs, dt = z.hidden_size, z.streams, 16, torch.bfloat16
    out: Dict[str, dict] = {}

    def rand(*shape, dtype=dt, std=1.0):
        return torch.randn(*shape, device=device, dtype=dtype) * std

    def i32(x):
        return torch.tensor(x, dtype=torch.int32, device=device)

    def pair(name, new, like):
        out[name] = {"new": new, "like": like,
                     "ratio": round(new["distance"] / like["distance"], 2)}

    def group(kind):
        mod = MixerGroup(_first(z, kind).mixer, W, 1e-5).to(dt).to(device)
        return mod, mod.cores[0], _spec(_first(z, kind))

    # --- decode attention: the cached K and V of every row once
    mod, core, s = group(AttnSpec)
    p = core.params
    H, G, D, E = s.heads, s.kv_heads, s.dim, s.vdim
    width = mod.in_proj.weight.shape[0]
    like_rows = {}
    for B, L in ((decode_batch, decode_len), (64, 4096), (1, 4096)):
        nb = L // bs
        bt = torch.randperm(B * nb, device=device).int().view(B, nb)
        lens, zz = i32([L] * B), rand(B, width)
        q = zz[:, :H * D].unflatten(1, (H, D))
        gate = zz[:, core.gate_at:core.gate_at + H * E]
        kc, vc = rand(B * nb, G, bs, D), rand(B * nb, G, E, bs)
        scale = RotaryTables(lens.long() - 1).temperature(s.q_temp)
        o = rand(B, H * E)
        ws = torch.empty(2 * gated.attn_scratch_floats(B, p, L) + 2,
                         device=device)
        t = _time(lambda: gated.attn_rows(
            o, q, p, (kc, vc), bt, lens, L, workspace=ws, row_scale=scale,
            gate=gate))
        nbytes = 2.0 * B * L * G * (D + E)
        new = _row(t, nbytes)
        vl, lq = vc.view(B * nb, G, bs, E), rand(B, H, D)
        lws = ops.decode_workspace(B, H, D, L, device)
        t = _time(lambda: ops.paged_attn_decode(lq, kc, vl, bt, lens, s.scale,
                                                lws, L))
        like_rows[B] = _row(t, nbytes)
        pair(f"decode_attention_b{B}_l{L}", new, like_rows[B])
        del kc, vc, vl

    # --- prompts
    light, lcore, ls = group(LightningSpec)
    lp = lcore.params
    scan, score, ss = group(SelectiveSpec)
    sp, sw = score.params, score.weights
    sw.A.uniform_(-8, -0.1)
    sw.dt_b.normal_(-3.0, 0.5)
    twin_ff = twin(z).intermediate_size
    for B, L in ((prompts, prompt_len), (1, 8192)):
        nb, T, tag = L // bs, B * L, f"_b{B}_l{L}"
        meta = _prefill_meta(B, L, bs, np.random.permutation(
            B * nb).reshape(B, nb), device)
        pairs = B * L * (L + 1) / 2
        zz, o = rand(T, width), rand(T, H * E)
        q = zz[:, :H * D].unflatten(1, (H, D))
        gate = zz[:, core.gate_at:core.gate_at + H * E]
        kc, vc = rand(B * nb, G, bs, D), rand(B * nb, G, E, bs)
        scale = RotaryTables(meta.positions).temperature(s.q_temp)
        nbytes = 2.0 * T * (H + G) * (D + E)
        flops = 2.0 * pairs * H * (D + E)
        t = _time(lambda: gated.attn_prompt(
            o, q, p, (kc, vc), meta, row_scale=scale, gate=gate), reps=5)
        new = _row(t, nbytes + 2.0 * T * H * E, flops)
        k, v, lq = rand(T, G, D), rand(T, G, D), rand(T, H, D)
        like = _row(_time(lambda: ops.attn_prefill(
            lq, k, v, meta.cu_seqlens, L, s.scale), reps=5), nbytes, flops)
        pair("prefill_attention" + tag, new, like)
        del kc, vc, k, v, lq, zz, o
        gu = rand(T, 2 * twin_ff)
        act = _row(_time(lambda: ops.silu_and_mul(gu)),
                   2.0 * T * 3 * twin_ff)
        del gu
        # lightning attention
        H2, D2, E2, C = ls.heads, ls.dim, ls.vdim, gated.GLA_CHUNK
        zz, y = rand(T, light.in_proj.weight.shape[0]), rand(T, H2 * E2)
        (shape, _), = ls.cache_layer().tensors
        state = torch.zeros(B, *shape, device=device)
        steps = gated.decay_chunk_steps(y, zz, lp, lcore.weights, state, meta)
        # q, k, v in; two terms of q, k and the scores and v out
        inside = 2.0 * T * H2 * (4 * D2 + E2 + 2 * C)
        pair("decay_operands" + tag, _row(
            _time(steps[0], reps=5), 2.0 * T * H2 * (2 * D2 + E2) + inside),
            act)
        flops = 2.0 * T * H2 * (2 * D2 * E2 + C / 2 * E2)
        pair("decay_chunks" + tag, _row(
            _time(steps[1], reps=5), inside + 2.0 * T * H2 * E2, flops), like)
        pair("row_norm_gate" + tag, _row(
            _time(steps[2], reps=5), 2.0 * T * H2 * E2 * 3), act)

        def whole():
            for f in steps:
                f()
        # the three together against what has to move at least
        pair("lightning_prompt" + tag, _row(
            _time(whole, reps=5), 2.0 * T * H2 * (2 * D2 + 3 * E2), flops),
            like)
        del zz, y, steps
        # selective scan
        I, N = ss.inner, ss.state
        zz, y = rand(T, scan.in_proj.weight.shape[0]), rand(T, I)
        ring = torch.zeros(B, ss.conv, I, dtype=dt, device=device)
        state = torch.zeros(B, N, I, device=device)
        pair("conv" + tag, _row(_time(lambda: routed.conv_silu(
            zz, sp, sw, ring, meta.state_slots, meta.positions,
            meta.cu_seqlens, L), reps=5), 2.0 * T * I * 2), act)
        x, raw = rand(T, I), rand(T, I, dtype=torch.float32)
        bc = rand(T, sw.x.shape[0], dtype=torch.float32)
        t = _time(lambda: routed.scan_prompt(y, x, zz, sp, sw, state, raw, bc,
                                             meta), reps=5)
        # x, z, y and the step sizes
        pair("scan" + tag, _row(t, T * I * 10.0), like)
        del zz, y, x, raw, bc

    # --- single tokens: the state in and out
    for B in (decode_batch, 1):
        slots = torch.arange(B, device=device, dtype=torch.int32)
        pos = torch.full((B,), 77, device=device)
        zz = rand(B, light.in_proj.weight.shape[0])
        o = rand(B, H2 * E2)
        (shape, _), = ls.cache_layer().tensors
        state = torch.zeros(B, *shape, device=device)
        C = gated._native()
        t = _time(lambda: C.decay_step(
            o, zz, lp.q_at, lp.k_at, lp.v_at, lp.vdim, lcore.decay, state,
            slots, pos, None))
        pair(f"decay_step_b{B}", _row(
            t, B * H2 * (8.0 * D2 * E2 + 2.0 * (2 * D2 + 2 * E2))),
            like_rows[B])
        zz = rand(B, scan.in_proj.weight.shape[0])
        y, x, raw = rand(B, I), rand(B, I), rand(B, I, dtype=torch.float32)
        ring = torch.zeros(B, ss.conv, I, dtype=dt, device=device)
        state = torch.zeros(B, N, I, device=device)
        bc = rand(B, sw.x.shape[0], dtype=torch.float32)
        t = _time(lambda: routed._native().scan_step(
            y, x, zz, sp.z_at, raw, sw.dt_b, bc, sp.b_at, sp.c_at, sw.A,
            sw.D, state, slots, pos))
        pair(f"scan_step_b{B}", _row(t, B * I * (8.0 * N + 10) + 4.0 * N * I),
             like_rows[B])
        gu = rand(B, 2 * twin_ff)
        act = _row(_time(lambda: ops.silu_and_mul(gu)),
                   2.0 * B * 3 * twin_ff)
        pair(f"conv_b{B}", _row(_time(lambda: routed.conv_silu(
            zz, sp, sw, ring, slots, pos)), B * I * 2.0 * (2 + ss.conv)
            + 4.0 * I * ss.conv), act)
        pair(f"row_norm_gate_b{B}", _row(_time(lambda: C.row_norm_gate(
            o, o, o, lcore.norm_w, 1e-5)), 2.0 * B * H2 * E2 * 3), act)
        del state

    # --- the mixture of experts
    ff = _first(z, AttnSpec).ff
    moe, r, F = Mixture(ff, W).to(dt).to(device), ff.router, ff.ff
    moe.ups.normal_(0, 0.02)
    moe.downs.normal_(0, 0.02)
    moe.router.normal_(0, 0.02)
    for T in (1, 8, 64, decode_batch, prompts * prompt_len):
        h = rand(T, W)
        logits = gated.project32(h, moe.router)
        ids, wt, rank, hist = routed._route(logits, moe.correction, r)
        height = routed.tile_height(ids.numel(), r, h, moe.ups, moe.downs)
        lists = routed.expert_lists(ids, rank, hist, r, *height)
        steps, rows = routed.expert_products(h, moe.ups, moe.downs, lists,
                                             r.top)
        real = ids[ids < r.experts]
        n, touched = real.numel(), real.unique().numel()
        flops = 2.0 * n * W * F
        wbytes = 2.0 * touched * W * F
        # as many rows of a dense product with a matrix of one expert's
        # size (prompts), or a row with as many weights (decoding)
        few = T <= decode_batch
        a, b = (rand(T, W), rand(touched * F, W)) if few else \
            (rand(n, W), rand(F, W))
        gemm = _time(lambda: torch.nn.functional.linear(a, b), reps=10)
        like = _row(gemm, wbytes if few else 0, flops)
        pair(f"experts_up_t{T}", _row(
            _time(steps[0], reps=10), wbytes + 2.0 * n * (W + F), flops), like)
        a, b = (rand(T, touched * F), rand(W, touched * F)) if few else \
            (rand(n, F), rand(W, F))
        gemm = _time(lambda: torch.nn.functional.linear(a, b), reps=10)
        like = _row(gemm, wbytes if few else 0, flops)
        pair(f"experts_down_t{T}", _row(
            _time(steps[1], reps=10), wbytes + 2.0 * n * (W + F), flops), like)
        del a, b
        # a dense model has nothing like these
        t = _time(lambda: routed._route(logits, moe.correction, r))
        out[f"route_t{T}"] = {
            "new": _row(t, 4.0 * T * (r.outputs + 3 * r.top))}
        t = _time(lambda: routed.expert_lists(ids, rank, hist, r, *height))
        out[f"place_t{T}"] = {"new": _row(t, 4.0 * T * r.top * 4)}

        # --- streams
        x, y = rand(T, S, W, dtype=torch.float32), rand(T, W)
        around = [torch.ones(n, device=device) / S for n in (S, S * S, S)]
        norm = routed.TanhNorm(torch.ones(1, device=device),
                               torch.ones(W, device=device),
                               torch.zeros(W, device=device))
        back = routed.Return(around[1].view(S, S), around[2])
        res, w16 = rand(T, W), torch.ones(W, device=device, dtype=dt)
        like = _row(_time(lambda: ops.fused_add_rms_norm(y, res, w16, 1e-6)),
                    T * W * 8.0)
        moved = T * W * (8.0 * S + 2)
        pair(f"streams_t{T}", _row(_time(lambda: routed.hyper_step(
            x, y, back, around[0], norm)), moved + 2.0 * T * W), like)
        rr = routed.RoutedRows(rows, lists.slot, wt, h)
        pair(f"streams_routed_t{T}", _row(_time(lambda: routed.hyper_step(
            x, rr, back, around[0], norm)),
            moved + 2.0 * (n + T) * W), like)
        # --- cache write
        zz = rand(T, width)
        slots = torch.arange(T, device=device)
        npg = -(-T // bs)
        kc, vc = rand(npg, G, bs, D), rand(npg, G, E, bs)
        t = _time(lambda: gated.attn_epilogue(zz, p, (kc, vc), slots))
        new = _row(t, 2.0 * T * 2 * G * (D + E))
        qkv_w = H * D + G * (D + E)
        qkv, vl = rand(T, qkv_w), vc.view(npg, G, bs, E)
        lcs = ops.make_cos_sin_cache(D, T, device=device)
        t = _time(lambda: ops.rope_qkv_cache(
            slots, qkv, lcs, H, G, D, kv_cache=(kc, vl), slot_mapping=slots))
        pair(f"cache_write_t{T}", new, _row(t, 2.0 * T * 2 * qkv_w))
        del rows, rr, x, y, zz, kc, vc, vl, qkv, lists, steps
    torch.cuda.empty_cache()
    return out
