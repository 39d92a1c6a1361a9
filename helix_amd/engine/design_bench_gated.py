"""Motolix's side of bench.py --design: the Llama of equal size and the
kernel pairs, at the sizes of the model's first layer of each kind.

Like kernels: Llama's attention for attention and for linear attention, its
elementwise and norm kernels for the others.
"""
from __future__ import annotations

from typing import Dict

import numpy as np
import torch

from helix_amd import ops
from helix_amd.engine.design_bench import _row, _time
from helix_amd.engine.design_bench_hybrid import _prefill_meta
from helix_amd.models.llama import LlamaConfig
from helix_amd.models.mixer_group import MixerGroup
from helix_amd.models.motolix import MotolixConfig
from helix_amd.models.rotary_attention import RotaryTables
from helix_amd.ops import gated


def _first(z: MotolixConfig, members: int):
    return next(l for l in z.layers if len(l.mixer.members) == members)


def twin(z: MotolixConfig) -> LlamaConfig:
    """Same width, vocabulary and feed-forward, the sigmoid layers' heads, a
    layer for every layer run."""
    l = _first(z, 1)
    m = l.mixer.members[0].spec
    return LlamaConfig(
        name=f"llama-as-{z.name}", vocab_size=z.vocab_size,
        hidden_size=z.hidden_size, num_layers=len(z.runs()),
        intermediate_size=l.ff, num_heads=m.heads, num_kv_heads=m.kv_heads,
        head_dim=m.dim, max_position=z.max_position)


@torch.inference_mode()
def kernels(z: MotolixConfig, device, decode_batch: int = 256,
            decode_len: int = 1024, prompts: int = 8,
            prompt_len: int = 2048) -> Dict[str, dict]:
    one, two = _first(z, 1), _first(z, 2)
    W, F, bs, dt = z.hidden_size, one.ff, 16, torch.bfloat16
    out: Dict[str, dict] = {}

    def rand(*shape, dtype=dt, std=1.0):
        return torch.randn(*shape, device=device, dtype=dtype) * std

    def i32(x):
        return torch.tensor(x, dtype=torch.int32, device=device)

    def pair(name, new, like):
        out[name] = {"new": new, "like": like,
                     "ratio": round(new["distance"] / like["distance"], 2)}

    groups = {k: MixerGroup(l.mixer, W, 1e-5).to(dt).to(device)
              for k, l in (("sigmoid", one), ("softmax", two))}
    gla = groups["softmax"].cores[1]
    gs, gp = gla.spec, gla.params
    gla.a2.normal_(0, 0.02)
    gla.a2_b.normal_(2.0, 1.0)

    # --- decode attention: the cached K and V of every row once
    for kind, mod in groups.items():
        core = mod.cores[0]
        s, p = core.spec, core.params
        H, G, D, E = s.heads, s.kv_heads, s.dim, s.vdim
        for B, L in ((decode_batch, decode_len), (64, 4096), (1, 4096)):
            nb = L // bs
            bt = torch.randperm(B * nb, device=device).int().view(B, nb)
            lens, q = i32([L] * B), rand(B, H, p.dim_pad)
            kc, vc = rand(B * nb, G, bs, D), rand(B * nb, G, E, bs)
            vcs = RotaryTables(lens.long() - 1).get(s.value_rotary,
                                                    core.value_freqs)
            o = rand(B, H * E)
            ws = torch.empty(2 * gated.attn_scratch_floats(B, p, L) + 2,
                             device=device)
            t = _time(lambda: gated.attn_rows(o, q, p, (kc, vc), bt, lens, L,
                                              vcs, workspace=ws))
            nbytes = 2.0 * B * L * G * (D + E)
            new = _row(t, nbytes)
            vl = vc.view(B * nb, G, bs, E)
            lws = ops.decode_workspace(B, H, D, L, device)
            t = _time(lambda: ops.paged_attn_decode(
                q, kc, vl, bt, lens, s.scale, lws, L))
            pair(f"decode_{kind}_b{B}_l{L}", new, _row(t, nbytes))
            del kc, vc, vl

    # --- prompts: score and value products of the visible pairs
    for B, L in ((prompts, prompt_len), (1, 8192)):
        nb, T = L // bs, B * L
        meta = _prefill_meta(B, L, bs, np.random.permutation(
            B * nb).reshape(B, nb), device)
        pairs = B * L * (L + 1) / 2
        for kind, mod in groups.items():
            core = mod.cores[0]
            s, p = core.spec, core.params
            H, G, D, E = s.heads, s.kv_heads, s.dim, s.vdim
            kc, vc = rand(B * nb, G, bs, D), rand(B * nb, G, E, bs)
            q, o = rand(T, H, p.dim_pad), rand(T, H * E)
            vcs = RotaryTables(meta.positions).get(s.value_rotary,
                                                   core.value_freqs)
            nbytes = 2.0 * T * (H + G) * (D + E)
            flops = 2.0 * pairs * H * (D + E)
            t = _time(lambda: gated.attn_prompt(o, q, p, (kc, vc), meta, vcs),
                      reps=5)
            new = _row(t, nbytes, flops)
            k, v = rand(T, G, D), rand(T, G, E)
            t = _time(lambda: ops.attn_prefill(q, k, v, meta.cu_seqlens, L,
                                               s.scale), reps=5)
            like = _row(t, nbytes, flops)
            pair(f"prefill_{kind}_b{B}_l{L}", new, like)
            del kc, vc, q, o, k, v
        # linear attention over the same prompts
        H, D, E = gs.heads, gs.dim, gs.vdim
        zz = rand(T, groups["softmax"].in_proj.weight.shape[0])
        y = rand(T, H * E)
        (shape, _), = gs.cache_layer().tensors
        state = torch.zeros(B, *shape, device=device)
        steps = gated.gla_chunk_steps(y, zz, gp, gla.weights, state, meta)
        C = gated.GLA_CHUNK
        gu = rand(T, 2 * F)
        act = _row(_time(lambda: ops.silu_and_mul(gu)), 2.0 * T * 3 * F)
        # q, k, v in; two terms of q, k and the scores and v out
        inside = 2.0 * T * H * (4 * D + E + 2 * C)
        pair(f"gla_operands_b{B}_l{L}", _row(
            _time(steps[0], reps=5), 2.0 * T * H * (2 * D + E) + inside),
            act)
        flops = 2.0 * T * H * (2 * D * E + C / 2 * E)
        pair(f"gla_chunks_b{B}_l{L}", _row(
            _time(steps[1], reps=5), inside + 2.0 * T * H * E, flops), like)
        pair(f"head_norm_gate_b{B}_l{L}", _row(
            _time(steps[2], reps=5), 2.0 * T * H * E * 3), act)
        # the three together against what has to move at least
        def whole():
            for s in steps:
                s()
        pair(f"gla_prompt_b{B}_l{L}", _row(
            _time(whole, reps=5), 2.0 * T * H * (2 * D + 3 * E), flops),
            like)
        del zz, y, gu, steps

    # --- linear attention, single tokens: the state in and out
    for B in (decode_batch, 1):
        H, D, E = gs.heads, gs.dim, gs.vdim
        zz = rand(B, groups["softmax"].in_proj.weight.shape[0])
        y = rand(B, H * E)
        (shape, _), = gs.cache_layer().tensors
        state = torch.zeros(B, *shape, device=device)
        slots = torch.arange(B, device=device, dtype=torch.int32)
        pos = torch.full((B,), 77, device=device)
        t = _time(lambda: gated.gla_step(y, zz, gp, gla.weights, state, slots,
                                         pos))
        new = _row(t, B * H * (8.0 * D * E + 2.0 * (2 * D + 3 * E)))
        like = out[f"decode_softmax_b{B}_l"
                   f"{decode_len if B == decode_batch else 4096}"]["like"]
        pair(f"gla_step_b{B}", new, like)
        del state

    # --- the rest: one pass over their operands
    for T in (decode_batch, prompts * prompt_len):
        slots = torch.arange(T, device=device)
        npg = -(-T // bs)
        for kind, mod in groups.items():
            core = mod.cores[0]
            s, p = core.spec, core.params
            H, G, D, E = s.heads, s.kv_heads, s.dim, s.vdim
            zz = rand(T, mod.in_proj.weight.shape[0])
            kc, vc = rand(npg, G, bs, D), rand(npg, G, E, bs)
            tables = RotaryTables(slots)
            cs = tables.get(s.rotary, core.freqs)
            vcs = tables.get(s.value_rotary, core.value_freqs)
            t = _time(lambda: gated.attn_epilogue(
                zz, p, (kc, vc), slots, cs, vcs, core.q_norm, core.k_norm,
                1e-5))
            cols = sum(n for _, n in s.inputs())
            new = _row(t, 2.0 * T * (cols + H * D + G * (D + E)))
            qkv_w = H * D + G * (D + E)
            qkv = rand(T, qkv_w)
            lcs = ops.make_cos_sin_cache(D, T, device=device)
            vl = vc.view(npg, G, bs, E)
            t = _time(lambda: ops.rope_qkv_cache(
                slots, qkv, lcs, H, G, D, kv_cache=(kc, vl),
                slot_mapping=slots))
            pair(f"epilogue_{kind}_t{T}", new, _row(t, 2.0 * T * 2 * qkv_w))
            del zz, kc, vc, vl, qkv
        gu = rand(T, 2 * F)
        new = _row(_time(lambda: gated.gated_mul(gu, F, F)), 2.0 * T * 3 * F)
        pair(f"activation_t{T}", new, _row(
            _time(lambda: ops.silu_and_mul(gu)), 2.0 * T * 3 * F))
        x, y = rand(T, W, dtype=torch.float32), rand(T, W)
        norm = gated.Norm(torch.ones(W, device=device),
                          torch.zeros(W, device=device))
        new = _row(_time(lambda: gated.stream_add(x, y, norm, norm, 1e-5)),
                   T * W * 12.0)
        res, w16 = rand(T, W), torch.ones(W, device=device, dtype=dt)
        like = _row(_time(lambda: ops.fused_add_rms_norm(y, res, w16, 1e-6)),
                    T * W * 8.0)
        pair(f"stream_add_t{T}", new, like)
        a, e = rand(2, T, W, dtype=torch.float32), rand(T, W,
                                                         dtype=torch.float32)
        h = torch.empty(T, W, dtype=dt, device=device)
        step = rand(W, dtype=torch.float32)
        new = _row(_time(lambda: gated._native().stream_enter(
            h, a[0], a[1], e, 1.0, step, norm.w, norm.b, 1e-5, x)),
            T * W * 18.0)
        pair(f"stream_enter_t{T}", new, like)
        del gu, a, e
    torch.cuda.empty_cache()
    return out
