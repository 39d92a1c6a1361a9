"""Throughput of a design's model beside a Llama of equal size, and each of
its kernels beside the like kernel of the Llama path (bench.py --design).

A kernel's distance is its time over the time its roofline allows (8 TB/s
HBM, 2.5 PFLOP/s dense bf16).
"""
from __future__ import annotations

import sys
import time
from typing import Callable, Dict, List

import torch

from helix_amd import ops
from helix_amd.engine.engine import EngineConfig, LLMEngine
from helix_amd.engine.sampling_params import SamplingParams
from helix_amd.models import registry
from helix_amd.models.llama import LlamaConfig, LlamaForCausalLM
from helix_amd.models.zederax import ZederaxConfig

HBM, FLOPS = 8.0e12, 2.5e15


def zederax_twin(z: ZederaxConfig) -> LlamaConfig:
    """Same width, depth, heads, vocabulary and window; the Llama
    feed-forward has three matrices, so two thirds of the ff."""
    m = z.layers[0].mixer
    return LlamaConfig(
        name=f"llama-as-{z.name}", vocab_size=z.vocab_size,
        hidden_size=z.hidden_size, num_layers=z.num_layers,
        intermediate_size=z.layers[0].ff * 2 // 3, num_heads=m.heads,
        num_kv_heads=m.kv_heads, head_dim=m.dim,
        max_position=z.max_position, sliding_window=m.window,
        tie_embeddings=True)


def _engine(cfg, device, batch: int, length: int) -> LLMEngine:
    model = registry.model_class(cfg)(cfg).to(torch.bfloat16).to(device)
    model.init_random(0)
    return LLMEngine(EngineConfig(
        model=cfg.name, max_num_seqs=batch, max_model_len=length,
        max_prefill_tokens=16384, eos_token_id=-1,
        kv_cache_blocks=batch * (length // 16 + 2),
        enable_prefix_caching=False), device=device, model=model)


def throughput(cfg, device, shapes, steps: int) -> List[dict]:
    """shapes: (batch, prompt length). The model is built once per shape
    set; prefill and decode run through the engine's own step()."""
    out = []
    top_b = max(b for b, _ in shapes)
    length = max(p for _, p in shapes) + 2 * steps + 64
    eng = _engine(cfg, device, top_b, -(-length // 16) * 16)
    for rnd, (b, p) in enumerate(shapes):
        g = torch.Generator().manual_seed(rnd)
        res = {}
        for rep in ("warm", "timed"):
            ids = torch.randint(3, cfg.vocab_size, (b, p),
                                generator=g).tolist()
            for i, t in enumerate(ids):
                eng.add_request(f"{rnd}-{rep}-{i}", t, SamplingParams(
                    max_tokens=steps + 8, ignore_eos=True))
            torch.cuda.synchronize()
            t0 = time.monotonic()
            while eng.waiting:
                eng.step()
            torch.cuda.synchronize()
            t1 = time.monotonic()
            for _ in range(4):
                eng.step()
            torch.cuda.synchronize()
            t2 = time.monotonic()
            for _ in range(steps):
                eng.step()
            torch.cuda.synchronize()
            t3 = time.monotonic()
            while eng.has_work:
                eng.step()
            res = {"batch": b, "prompt": p,
                   "prefill_tok_s": round(b * p / (t1 - t0)),
                   "decode_tok_s": round(b * steps / (t3 - t2)),
                   "decode_ms": round((t3 - t2) / steps * 1e3, 3)}
        out.append(res)
        print(f"{cfg.name}: {res}", file=sys.stderr, flush=True)
    del eng
    torch.cuda.empty_cache()
    return out


def _time(fn: Callable, reps: int = 20) -> float:
    """Median seconds of one call."""
    for _ in range(3):
        fn()
    ev = [(torch.cuda.Event(enable_timing=True),
           torch.cuda.Event(enable_timing=True)) for _ in range(reps)]
    for a, b in ev:
        a.record()
        fn()
        b.record()
    torch.cuda.synchronize()
    return sorted(a.elapsed_time(b) for a, b in ev)[reps // 2] * 1e-3


def _row(t: float, nbytes: float, flops: float = 0.0) -> dict:
    floor = max(nbytes / HBM, flops / FLOPS)
    return {"us": round(t * 1e6, 1), "roofline_us": round(floor * 1e6, 1),
            "distance": round(t / floor, 2)}


def zederax_kernels(z: ZederaxConfig, device, decode_batch: int = 256,
            decode_len: int = 1024, prompts: int = 8,
            prompt_len: int = 2048) -> Dict[str, dict]:
    """Each kernel of the new path and the like one, at one layer's size."""
    m, W, F = z.layers[0].mixer, z.hidden_size, z.layers[0].ff
    H, G, D, E, bs = m.heads, m.kv_heads, m.dim, m.vdim, 16
    dt = torch.bfloat16
    out = {}

    def rand(*s, dtype=dt):
        return torch.randn(*s, device=device, dtype=dtype)

    def i32(x):
        return torch.tensor(x, dtype=torch.int32, device=device)

    def pair(name, new, like):
        out[name] = {"new": new, "like": like,
                     "ratio": round(new["distance"] / like["distance"], 2)}

    tp = ops.TalkParams(m.scale, m.softcap, m.window,
                        torch.rand(H, device=device),
                        torch.randn(H, H, device=device) * 0.2)

    # --- decode attention: the visible K and V of every row once
    for B, L in ((decode_batch, decode_len), (64, 4096), (1, 4096)):
        nb = L // bs
        bt = torch.randperm(B * nb, device=device).int().view(B, nb)
        kc, vc = rand(B * nb, G, bs, D), rand(B * nb, G, E, bs)
        lens, q = i32([L] * B), rand(B, H, D)
        o, gate = rand(B, H * E), rand(B, H)
        ws = torch.empty(2 * ops.talk_scratch_floats(B, H, G, E, L),
                         device=device)
        t = _time(lambda: ops.talk_attn_rows(o, q, (kc, vc), bt, lens, L, tp,
                                             gate, workspace=ws))
        nbytes = 2.0 * B * tp.max_keys(L) * G * (D + E)
        new = _row(t, nbytes)
        vl = vc.view(B * nb, G, bs, E)
        lws = ops.decode_workspace(B, H, D, L, device)
        t = _time(lambda: ops.paged_attn_decode(q, kc, vl, bt, lens, m.scale,
                                                lws, L, window=m.window))
        pair(f"decode_attention_b{B}_l{L}", new, _row(t, nbytes))
        del kc, vc, vl

    # --- prefill attention: score and value products of the visible pairs
    for B, L in ((prompts, prompt_len), (1, 8192)):
        nb, T = L // bs, B * L
        bt = torch.randperm(B * nb, device=device).int().view(B, nb)
        kc, vc = rand(B * nb, G, bs, D), rand(B * nb, G, E, bs)
        q, o, gate = rand(T, H, D), rand(T, H * E), rand(T, H)
        cu, lens = i32([i * L for i in range(B + 1)]), i32([L] * B)
        win = min(m.window or L, L)
        pairs = B * (win * (win + 1) / 2 + (L - win) * win)
        flops = 2.0 * pairs * H * (D + E)
        nbytes = 2.0 * T * (H * (D + E) + G * (D + E))
        t = _time(lambda: ops.talk_attn_prefill(
            o, q, (kc, vc), bt, cu, lens, L, L, None, None, tp, gate),
            reps=5)
        new = _row(t, nbytes, flops)
        k, v = rand(T, G, D), rand(T, G, D)
        t = _time(lambda: ops.attn_prefill(q, k, v, cu, L, m.scale,
                                           window=m.window), reps=5)
        pair(f"prefill_attention_b{B}_l{L}", new, _row(t, nbytes, flops))
        del kc, vc, q, o

    # --- the rest: one pass over their operands
    for T in (decode_batch, prompts * prompt_len):
        qkv_w = H * D + G * (D + E)
        wide = qkv_w + F + 64
        zz = rand(T, wide)
        slots = torch.arange(T, device=device)
        npg = -(-T // bs)
        kc, vc = rand(npg, G, bs, D), rand(npg, G, E, bs)
        vf = rand(T, G * E)
        lam = torch.tensor(0.4, device=device)
        coef = torch.tensor([.8, .3, .2, .1], device=device)
        buf = rand(T, H * E + F)
        t = _time(lambda: ops.unit_qkv_cache(
            zz, [0, H * D, H * D + G * D], H, D, (kc, vc), slots, 1e-6, vf,
            lam))
        new = _row(t, 2.0 * T * (2 * qkv_w + G * E))
        cs = ops.make_cos_sin_cache(D, 4096, device=device)
        pos = slots % 4096
        qkv = rand(T, qkv_w)
        vl = vc.view(npg, G, bs, E)
        t = _time(lambda: ops.rope_qkv_cache(
            pos, qkv, cs, H, G, D, kv_cache=(kc, vl), slot_mapping=slots))
        pair(f"qkv_epilogue_t{T}", new, _row(t, 2.0 * T * 2 * qkv_w))
        t = _time(lambda: ops.poly_norm(zz[:, qkv_w:qkv_w + F], coef, 1e-6,
                                        buf[:, H * E:]))
        new = _row(t, 2.0 * T * 2 * F)
        gu = rand(T, 2 * (F * 2 // 3))
        t = _time(lambda: ops.silu_and_mul(gu))
        pair(f"activation_t{T}", new, _row(t, 2.0 * T * 3 * (F * 2 // 3)))
        n = z.num_layers // 2
        hist = torch.randn(n + 1, T, W, device=device)
        x, y = torch.randn(T, W, device=device), rand(T, W)
        dwa = torch.randn(n + 1, device=device)
        w32 = torch.ones(W, device=device)
        t = _time(lambda: ops.depth_norm(x, y, hist, n, dwa, w32, 1e-6,
                                         x_out=x))
        new = _row(t, T * W * (4.0 * n + 3 * 4 + 2 * 2))
        res, w16 = rand(T, W), torch.ones(W, device=device, dtype=dt)
        t = _time(lambda: ops.fused_add_rms_norm(y, res, w16, 1e-6))
        pair(f"residual_norm_t{T}", new, _row(t, T * W * 8.0))
        # both epilogues of the layer in their one launch
        t = _time(lambda: ops.unit_qkv_cache(
            zz, [0, H * D, H * D + G * D], H, D, (kc, vc), slots, 1e-6, vf,
            lam, ff=(zz[:, qkv_w:qkv_w + F], buf[:, H * E:], coef)))
        out[f"layer_epilogue_t{T}"] = {
            "new": _row(t, 2.0 * T * (2 * qkv_w + G * E + 2 * F))}
        del hist, zz, buf
    torch.cuda.empty_cache()
    return out


def _families():
    from helix_amd.engine import design_bench_gated as gated
    from helix_amd.engine import design_bench_hybrid as hybrid
    from helix_amd.engine import design_bench_routed as routed
    from helix_amd.models.dibizen import DibizenConfig
    from helix_amd.models.motolix import MotolixConfig
    from helix_amd.models.nibezen import NibezenConfig
    return {ZederaxConfig: ("zederax", zederax_twin, zederax_kernels),
            NibezenConfig: ("nibezen", hybrid.twin, hybrid.kernels),
            MotolixConfig: ("motolix", gated.twin, gated.kernels),
            DibizenConfig: ("dibizen", routed.twin, routed.kernels)}


def run(names: List[str], device: str, steps: int, what: str) -> dict:
    result = {}
    for name in names:
        z = registry.get_config(name)
        family, twin, kernels = _families()[type(z)]
        r = result[name] = {}
        if what in ("all", "throughput"):
            shapes = [(8, 2048), (64, 2048), (256, 1024)]
            r[family] = throughput(z, device, shapes, steps)
            r["llama"] = throughput(twin(z), device, shapes, steps)
            for a in ("prefill_tok_s", "decode_tok_s"):
                r[f"ratio_{a}"] = [
                    round(x[a] / y[a], 3)
                    for x, y in zip(r[family], r["llama"])]
        if what in ("all", "kernels"):
            r["kernels"] = kernels(z, device)
    return result
