"""Nibezen's side of bench.py --design: the Llama of equal size and the
kernel pairs, at the sizes of the model's first layer of each kind.

Like kernels: attention for attention and for the state-space mixer, the
other elementwise and norm kernels for theirs, a plain GEMM of equal weights
for the small per-head products around latent attention.
"""
from __future__ import annotations

from typing import Dict

import numpy as np
import torch

from helix_amd import ops
from helix_amd.engine.design_bench import _row, _time
from helix_amd.models.latent import LatentAttention, LatentSpec
from helix_amd.models.llama import LlamaConfig
from helix_amd.models.meta import PrefillMeta
from helix_amd.models.nibezen import NibezenConfig
from helix_amd.models.ssm import Mamba2Mixer, SSMSpec
from helix_amd.ops import hybrid


def _first(z: NibezenConfig, kind):
    return next(l for l in z.layers if isinstance(l.mixer, kind))


def twin(z: NibezenConfig) -> LlamaConfig:
    """Same width, vocabulary, heads, window and feed-forward, a layer for
    every layer run; 4 query heads to a key/value head."""
    l = _first(z, LatentSpec)
    return LlamaConfig(
        name=f"llama-as-{z.name}", vocab_size=z.vocab_size,
        hidden_size=z.hidden_size, num_layers=len(z.runs()),
        intermediate_size=l.ff, num_heads=l.mixer.heads,
        num_kv_heads=l.mixer.heads // 4, head_dim=l.mixer.vdim,
        max_position=z.max_position, sliding_window=l.mixer.window)


def _prefill_meta(B: int, L: int, bs: int, tables: np.ndarray, dev):
    pos = np.tile(np.arange(L), B)
    which = np.repeat(np.arange(B), L)

    def put(a, dt):
        return torch.as_tensor(np.ascontiguousarray(a)).to(dt).to(dev)

    i32, i64 = torch.int32, torch.int64
    return PrefillMeta(
        cu_seqlens=put(np.arange(B + 1) * L, i32), max_seqlen=L,
        slot_mapping=put(tables[which, pos // bs] * bs + pos % bs, i64),
        positions=put(pos, i64), max_len=L,
        block_tables=put(tables, i32), seq_lens=put(np.full(B, L), i32),
        row_seq=put(which, i32), row_len=put(pos + 1, i32),
        state_slots=put(np.arange(B), i32), starts=np.zeros(B, dtype=int),
        ends=np.full(B, L), host_tables=tables, block_size=bs)


@torch.inference_mode()
def kernels(z: NibezenConfig, device, decode_batch: int = 256,
            decode_len: int = 1024, prompts: int = 8,
            prompt_len: int = 2048) -> Dict[str, dict]:
    la, sl = _first(z, LatentSpec), _first(z, SSMSpec)
    m, s, W, F = la.mixer, sl.mixer, z.hidden_size, la.ff
    H, D, R, E, K, bs = m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, 16
    G = H // 4
    dt, C = torch.bfloat16, hybrid._native()
    out: Dict[str, dict] = {}

    def rand(*shape, dtype=dt, std=1.0):
        return torch.randn(*shape, device=device, dtype=dtype) * std

    def i32(x):
        return torch.tensor(x, dtype=torch.int32, device=device)

    def pair(name, new, like):
        out[name] = {"new": new, "like": like,
                     "ratio": round(new["distance"] / like["distance"], 2)}

    mod = LatentAttention(m, W, 1e-6).to(dt).to(device)
    for w in (mod.uk, mod.ukt, mod.uv):
        w.copy_(rand(*w.shape, std=0.05))
    p = mod.params

    # --- decode: rows of latents against rows of keys and values
    for B, L in ((decode_batch, decode_len), (64, 4096), (1, 4096)):
        nb = L // bs
        bt = torch.randperm(B * nb, device=device).int().view(B, nb)
        lens, keys = i32([L] * B), p.max_keys(L)
        cache = rand(B * nb, 1, bs, p.row)
        q = rand(B, H, p.row)
        parts = hybrid.latent_parts(B, H, keys)
        o, part, ml = rand(B, H, p.rank_pad), None, None
        if parts > 1:
            part = rand(B, parts, H, p.rank_pad, dtype=torch.float32)
            ml = torch.empty(B, parts, H, 2, device=device)
        one = o if parts == 1 else None
        t = _time(lambda: C.latent_rows(one, part, ml, q, cache, bt, None,
                                        lens, p.rank_pad, p.scale, p.window))
        new = _row(t, 2.0 * B * keys * p.row,
                   2.0 * B * keys * H * (p.row + p.rank_pad))
        qd = rand(B, H, E)
        kc, vc = rand(B * nb, G, bs, E), rand(B * nb, G, bs, E)
        ws = ops.decode_workspace(B, H, E, L, device)
        t = _time(lambda: ops.paged_attn_decode(
            qd, kc, vc, bt, lens, m.scale, ws, L, window=m.window))
        like = _row(t, 4.0 * B * keys * G * E)
        pair(f"decode_attention_b{B}_l{L}", new, like)
        zz = rand(B, mod.in_proj.weight.shape[0])
        gate, dst = zz[:, mod.gate_at:mod.gate_at + H], rand(B, H * E)

        def value_out():
            if parts > 1:
                C.latent_merge(o, part, ml)
            C.latent_out(dst, o, mod.uv, gate)
        for name, fn, wts, act in (
                ("absorb", lambda: C.latent_absorb(
                    q, zz, 0, p.head_cols, p.dim_pad, mod.uk, mod.ukt,
                    p.rank_pad), H * D * K, H * (D + K)),
                ("value_out", value_out, H * E * K,
                    H * (E + K * (1 if parts == 1 else 2 * parts)))):
            new = _row(_time(fn), 2.0 * (wts + B * act), 2.0 * B * wts)
            x, w = rand(B, W), rand(wts // W, W)
            like = _row(_time(lambda: ops.linear(x, w)),
                        2.0 * (wts + B * (W + wts // W)), 2.0 * B * wts)
            pair(f"{name}_b{B}_l{L}", new, like)
        del cache, kc, vc, part

    # --- prefill attention: score and value products of the visible pairs
    for B, L in ((prompts, prompt_len), (1, 8192)):
        nb, T = L // bs, B * L
        meta = _prefill_meta(B, L, bs, np.random.permutation(
            B * nb).reshape(B, nb), device)
        win = min(m.window or L, L)
        pairs = B * (win * (win + 1) / 2 + (L - win) * win)
        zz = rand(T, mod.in_proj.weight.shape[0])
        gate, dst = zz[:, mod.gate_at:mod.gate_at + H], rand(T, H * E)
        (c,) = meta.context(m.window)
        rows = c.slots.shape[0]
        lat, k = rand(rows, p.row), rand(rows, H * p.dim_pad)
        vt = rand(H * E, rows)
        t = _time(lambda: C.latent_prompt(
            dst, zz, 0, p.head_cols, H, k, lat[:, p.rank_pad:], vt,
            meta.cu_seqlens, c.start, c.length, L, p.scale, p.window, gate),
            reps=5)
        new = _row(t, 2.0 * T * H * (2 * D + R + 2 * E),
                   2.0 * pairs * H * (D + R + E))
        qd, kd, vd = rand(T, H, E), rand(T, G, E), rand(T, G, E)
        t = _time(lambda: ops.attn_prefill(
            qd, kd, vd, meta.cu_seqlens, L, m.scale, window=m.window),
            reps=5)
        like = _row(t, 2.0 * T * (2 * H + 2 * G) * E, 4.0 * pairs * H * E)
        pair(f"prefill_attention_b{B}_l{L}", new, like)
        # the state-space mixer over the same prompts
        sm = Mamba2Mixer(s, W, 1e-6).to(dt).to(device)
        sp, n = sm.params, s.channels
        zs = rand(T, sm.in_proj.weight.shape[0])
        y = rand(T, s.inner)
        cache = tuple(torch.zeros(B, *sh, dtype=d or dt, device=device)
                      for sh, d in s.cache_layer().tensors)
        wts = hybrid.SSMWeights(sm.conv_w, sm.conv_b, sm.dt_bias, sm.A_log,
                                sm.D)
        conv, scan = hybrid.ssm_chunk_steps(y, zs, sp, wts, cache, meta)
        conv()
        # operands are written once, B twice
        obytes = 2.0 * T * (2 * n + s.groups * s.state + 4 * s.heads)
        gu = rand(T, 2 * F)
        t_el = _time(lambda: ops.silu_and_mul(gu))
        pair(f"conv_chunks_b{B}_l{L}", _row(_time(conv, reps=5), obytes),
             _row(t_el, 2.0 * T * 3 * F))
        Q = hybrid.SSM_CHUNK
        flops = 2.0 * T * s.heads * (
            Q / 2 * (s.state + s.vdim) + 2 * s.state * s.vdim)
        new = _row(_time(scan, reps=5),
                   2.0 * T * (3 * s.inner + 3 * s.groups * s.state
                              + 4 * s.heads), flops)
        pair(f"ssm_chunks_b{B}_l{L}", new, like)
        del zz, lat, k, vt, qd, kd, vd, zs, gu

    # --- state-space decode: the state in and out
    for B in (decode_batch, 1):
        sm = Mamba2Mixer(s, W, 1e-6).to(dt).to(device)
        zs, y = rand(B, sm.in_proj.weight.shape[0]), rand(B, s.inner)
        cache = tuple(torch.zeros(B, *sh, dtype=d or dt, device=device)
                      for sh, d in s.cache_layer().tensors)
        wts = hybrid.SSMWeights(sm.conv_w, sm.conv_b, sm.dt_bias, sm.A_log,
                                sm.D)
        slots = torch.arange(B, device=device, dtype=torch.int32)
        pos = torch.full((B,), 77, device=device)
        t = _time(lambda: hybrid.ssm_step(y, zs, sm.params, wts, cache,
                                          slots, pos))
        new = _row(t, B * (8.0 * s.inner * s.state
                           + 2.0 * (2 * s.inner + (s.conv + 1)
                                    * s.channels)))
        like = out[f"decode_attention_b{B}_l"
                   f"{decode_len if B == decode_batch else 4096}"]["like"]
        pair(f"ssm_step_b{B}", new, like)
        del cache

    # --- the rest: one pass over their operands
    for T in (decode_batch, prompts * prompt_len):
        zz = rand(T, mod.in_proj.weight.shape[0])
        slots = torch.arange(T, device=device)
        npg = -(-T // bs)
        cache = rand(npg, 1, bs, p.row)
        t = _time(lambda: hybrid.latent_epilogue(
            zz, p, slots, mod.kv_norm_w, 1e-6, cache, slots))
        new = _row(t, 2.0 * T * (2 * H * R + 2 * p.row))
        qkv_w = (H + 2 * G) * E
        qkv, cs = rand(T, qkv_w), ops.make_cos_sin_cache(E, T, device=device)
        kc, vc = rand(npg, G, bs, E), rand(npg, G, bs, E)
        t = _time(lambda: ops.rope_qkv_cache(
            slots, qkv, cs, H, G, E, kv_cache=(kc, vc), slot_mapping=slots))
        pair(f"epilogue_t{T}", new, _row(t, 2.0 * T * 2 * qkv_w))
        gu = rand(T, 2 * F)
        new = _row(_time(lambda: hybrid.silu_mul(gu, F, F)), 2.0 * T * 3 * F)
        pair(f"activation_t{T}", new, _row(
            _time(lambda: ops.silu_and_mul(gu)), 2.0 * T * 3 * F))
        x, y = rand(T, W, dtype=torch.float32), rand(T, W)
        w32 = torch.ones(W, device=device)
        new = _row(_time(lambda: hybrid.residual_norm(
            x, y, w32, 0.7, w32, 1e-6, dt, x_out=x)), T * W * 12.0)
        res, w16 = rand(T, W), torch.ones(W, device=device, dtype=dt)
        like = _row(_time(lambda: ops.fused_add_rms_norm(y, res, w16, 1e-6)),
                    T * W * 8.0)
        pair(f"residual_norm_t{T}", new, like)
        yi = rand(T, s.inner)
        wi, wl = torch.ones(s.inner, device=device), rand(s.inner)
        new = _row(_time(lambda: hybrid.group_rms_norm(
            yi, s.norm_groups, wi, 1e-6)), 4.0 * T * s.inner)
        pair(f"group_norm_t{T}", new, _row(
            _time(lambda: ops.rms_norm(yi, wl, 1e-6)), 4.0 * T * s.inner))
        del zz, cache, qkv, kc, vc, gu
    torch.cuda.empty_cache()
    return out
