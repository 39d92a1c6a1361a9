"""Nibezen against its plain full-sequence oracle: every mechanism alone,
then the model through the engine (portions, decoding, mixed batches, reused
pages and state slots, greedy generation). Each test runs on the CPU
reference ops and, marked gpu, on the HIP kernels."""
import io
import json
import math

import numpy as np
import pytest
import torch

import nibezen_oracle as no
from helix_amd import ops
from helix_amd.engine import replay
from helix_amd.engine.engine import EngineConfig, LLMEngine
from helix_amd.engine.kv_cache import KVCache
from helix_amd.engine.sampling_params import SamplingParams
from helix_amd.models import registry
from helix_amd.models.meta import (CONTEXT_TAIL, DecodeMeta, MixedMeta,
                                   PrefillMeta, StateLayer)
from helix_amd.models.latent import LatentAttention, LatentSpec
from helix_amd.models.nibezen import (PRESETS, NibezenConfig,
                                      NibezenForCausalLM)
from helix_amd.models.ssm import Mamba2Mixer, SSMSpec
from helix_amd.ops import hybrid

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F32, BF16 = torch.float32, torch.bfloat16
EPS = 1e-5


def tol(dtype):
    return 3e-5 if dtype == F32 else 3e-2


def close(got, want, dtype, scale=None):
    """Largest deviation, relative to the element plus the rms of all."""
    got, want = got.double().cpu(), want.double().cpu()
    ref = scale or max(float(want.pow(2).mean().sqrt()), 1e-6)
    err = float(((got - want).abs() / (ref + want.abs())).max())
    assert err < tol(dtype), err


def close_rows(got, want, dtype, rms):
    """A whole mixer. bf16 rounds several times in a row (projections, keys,
    weights), so there rows are judged by their root-mean-square error."""
    if dtype == F32:
        return close(got, want, dtype, rms)
    err = (got.double().cpu() - want.double()).pow(2).mean(-1).sqrt() / rms
    assert float(err.max()) < 0.06, float(err.max())


def rnd(g, *shape, dtype=F32, std=1.0):
    """Values exactly representable in dtype, as float64."""
    return (torch.randn(*shape, generator=g) * std).to(dtype).double()


def gen(seed):
    return torch.Generator().manual_seed(seed)


# ------------------------------------------------------------ stream and norms

@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,W", [(3, 64), (5, 250), (2, 1028), (600, 96),
                                 (1, 5120), (3, 77), (520, 2048)])
def test_residual_norm(dev, dtype, T, W):
    g = gen(T + W)
    x, ls, w, step = (rnd(g, *s) for s in ((T, W), (W,), (W,), (W,)))
    y, emb = rnd(g, T, W, dtype=dtype), rnd(g, 11, W, dtype=dtype)
    ids = torch.randint(0, 11, (T,), generator=g)

    def put(t, dt=F32):
        return t.to(dt).to(dev)

    for entry in (0, 1, 2):                   # none, step, embedding and step
        add = {}
        v = x + 0.7 * (ls * y)
        tapped = v
        if entry:
            add["step"] = put(step)
            if entry == 2:
                v = v + emb[ids]
                add.update(ids=ids.to(dev), embed=put(emb, dtype))
            v = v + step
        xd = put(x)
        tap = torch.empty_like(xd) if entry else None
        h = hybrid.residual_norm(xd, put(y, dtype), put(ls), 0.7, put(w),
                                 EPS, dtype, x_out=xd, tap=tap, **add)
        close(h, no.rms_norm(v, w, EPS), dtype)
        close(xd, v, F32)
        if entry:
            close(tap, tapped, F32)
    xd = torch.empty(T, W, device=dev)
    h = hybrid.residual_norm(None, None, None, 0.7, put(w), EPS, dtype,
                             ids=ids.to(dev), embed=put(emb, dtype),
                             step=put(step), x_out=xd)
    close(xd, emb[ids] + step, F32)
    close(h, no.rms_norm(emb[ids] + step, w, EPS), dtype)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,F", [(3, 64), (7, 50), (300, 1032)])
def test_silu_mul(dev, dtype, T, F):
    g = gen(F)
    up = -(-F // 8) * 8
    z = rnd(g, T, up + F, dtype=dtype, std=3.0)
    out = hybrid.silu_mul(z.to(dtype).to(dev), up, F)
    close(out, no.silu(z[:, :F]) * z[:, up:up + F], dtype)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,groups,size", [(3, 1, 64), (5, 3, 50),
                                           (40, 4, 24), (2, 2, 2100),
                                           (3, 2, 4096), (200, 8, 1024)])
def test_group_rms_norm(dev, dtype, T, groups, size):
    g = gen(size)
    # parts of very different size: each has its own root mean square
    y = rnd(g, T, groups, size)
    y = (y * torch.logspace(-2, 2, groups)[:, None]).flatten(1)
    y = y.to(dtype).double()
    w = rnd(g, groups * size)
    out = hybrid.group_rms_norm(y.to(dtype).to(dev), groups,
                                w.float().to(dev), EPS)
    want = no.group_norm(y, groups, w, EPS)
    close(out, want, dtype)


# ---------------------------------------------------------------- batch pieces

def prompt_meta(spans, tables, bs, dev, slots=None):
    """spans: (start, end) of each sequence's new tokens; tables: pages."""
    starts = np.array([s for s, _ in spans])
    ends = np.array([e for _, e in spans])
    lens = ends - starts
    which = np.repeat(np.arange(len(spans)), lens)
    pos = np.concatenate([np.arange(s, e) for s, e in spans])

    def put(a, dt):
        return torch.as_tensor(np.ascontiguousarray(a)).to(dt).to(dev)

    i32, i64 = torch.int32, torch.int64
    at = tables[which, pos // bs] * bs + pos % bs
    return PrefillMeta(
        cu_seqlens=put(np.concatenate([[0], np.cumsum(lens)]), i32),
        max_seqlen=int(lens.max()), slot_mapping=put(at, i64),
        positions=put(pos, i64), max_len=int(ends.max()),
        state_slots=put(np.arange(len(spans)) if slots is None else slots,
                        i32),
        starts=starts, ends=ends, block_size=bs, host_tables=tables,
        block_tables=put(tables, i32), seq_lens=put(ends, i32),
        row_seq=put(which, i32), row_len=put(pos + 1, i32))


def decode_meta(pos, tables, bs, dev, slots=None):
    pos = np.asarray(pos)

    def put(a, dt):
        return torch.as_tensor(np.ascontiguousarray(a)).to(dt).to(dev)

    at = tables[np.arange(len(pos)), pos // bs] * bs + pos % bs
    return DecodeMeta(
        block_tables=put(tables, torch.int32),
        seq_lens=put(pos + 1, torch.int32),
        slot_mapping=put(at, torch.int64), positions=put(pos, torch.int64),
        max_len=int(pos.max()) + 1,
        state_slots=put(np.arange(len(pos)) if slots is None else slots,
                        torch.int32))


def test_prompt_context_and_chunks():
    """Every portion's window in one aligned row list, in groups."""
    tables = np.arange(40).reshape(2, 20)[:, ::-1].copy()
    m = prompt_meta([(70, 130), (0, 33)], tables, 8, "cpu")
    for window, lows in ((0, (0, 0)), (1, (70, 0)), (50, (21, 0))):
        (c,) = m.context(window)
        assert (c.first, c.last) == (0, 2)
        for i, (lo, end) in enumerate(zip(lows, (130, 33))):
            a, n = int(c.start[i]), int(c.length[i])
            assert a % 8 == 0 and n == end - lo
            want = [tables[i, p // 8] * 8 + p % 8 for p in range(lo, end)]
            assert c.slots[a:a + n].tolist() == want
        assert len(c.slots) % 8 == 0
        assert len(c.slots) >= int(c.start[1] + c.length[1]) + CONTEXT_TAIL
    ch = m.chunks(32)
    assert ch.row.tolist() == [0, 32, 60, 92]
    assert ch.count.tolist() == [32, 28, 32, 1]
    assert ch.seq.tolist() == [0, 0, 1, 1] and ch.first.tolist() == [0, 2, 4]


def test_long_contexts_are_grouped(monkeypatch):
    from helix_amd.models import meta
    monkeypatch.setattr(meta, "CONTEXT_ROWS", 100)
    tables = np.arange(60).reshape(3, 20)
    m = prompt_meta([(0, 60), (0, 40), (90, 120)], tables, 8, "cpu")
    groups = [(c.first, c.last) for c in m.context(0)]
    assert groups == [(0, 1), (1, 2), (2, 3)]
    assert [(c.first, c.last) for c in m.context(20)] == [(0, 1), (1, 3)]


# ------------------------------------------------------------ latent attention

@pytest.mark.parametrize("scaling", [
    None, dict(factor=6.0, original=300, fast=16.0, slow=2.0),
    dict(factor=2.5, original=40, fast=4.0, slow=0.5),
    dict(factor=8.0, original=4096, fast=2.0, slow=2.0)])
@pytest.mark.parametrize("dims,base", [(12, 1e4), (64, 5e5), (2, 100.0),
                                       (6, 2e6)])
def test_yarn_frequencies(dims, base, scaling):
    f, amp = ops.yarn_frequencies(dims, base, scaling)
    want, want_amp = no.rotation_frequencies(dims, base, scaling)
    assert torch.allclose(f, torch.tensor(want, dtype=torch.float64),
                          rtol=1e-12, atol=0)
    assert abs(amp - want_amp) < 1e-12


ATTN = [
    # heads, dim, rot_dim, vdim, rank, window, rotated dims
    (5, 24, 8, 40, 48, 19, 8),
    (3, 20, 12, 36, 52, 33, 12),              # nothing a multiple of 8
    (6, 32, 16, 24, 64, 0, 8),                # part of the rotated dims
    (4, 16, 16, 16, 128, 1, 16),
    (16, 64, 32, 64, 128, 64, 32),
    (20, 96, 32, 96, 256, 50, 32),            # two tiles of heads
    (40, 128, 64, 128, 512, 70, 64),          # and three groups
    (32, 128, 64, 128, 256, 45, 64),
    (2, 200, 40, 200, 96, 31, 40),
    (1, 8, 2, 8, 8, 300, 2),
    (3, 48, 16, 72, 520, 40, 16),             # beyond the MFMA row kernel
    (2, 264, 16, 264, 72, 40, 16),            # beyond the MFMA prompt kernel
    (3, 24, 8, 13, 40, 25, 8),                # odd value size
]
YARN = dict(factor=3.0, original=64, fast=8.0, slow=0.5)


def latent_case(case, n, dtype, seed=0):
    """A mixer with random weights and one sequence's inputs in which keys
    stand out for late queries: a far one and those at the window's edge.
    -> (weights, mixer configuration, h, expected output)."""
    H, D, R, E, K, window, dims = case
    g = gen(seed + H * D + K)
    W = 64
    m = dict(heads=H, dim=D, rot_dim=R, vdim=E, kv_rank=K,
             scale=5.0 / math.sqrt(D + R), mask=dict(size=window),
             rot=dict(dims=dims, base=1e3, scaling=YARN))
    w = {}
    for name, shape in (("q", (H * (D + R), W)), ("dkv", (K + R, W)),
                        ("uk", (H * D, K)), ("uv", (H * E, K)),
                        ("g", (H, W)), ("o", (W, H * E))):
        w[name] = rnd(g, *shape, dtype=BF16, std=shape[1] ** -0.5)
    w["dkv.norm"] = (1 + rnd(g, K, std=0.2)).to(BF16).double()
    h = rnd(g, n, W, dtype=dtype)
    for i in (n - 1, n // 2):
        for j in ({i - window, i - window + 1, i - 1} if window else {0, 3}):
            if 0 <= j < n and j != i:
                h[j] = (h[i] + rnd(g, W, std=0.2)).to(dtype).double()
    return w, m, h


def build_latent(w, m, dtype, dev):
    mod = LatentAttention(LatentSpec.from_json(m), 64, EPS)
    for name, dst in mod.targets("").items():
        dst.copy_(w[name].float())
    return mod.to(dtype).to(dev)


def page_tables(lens, bs, g):
    """Shuffled page numbers, and how many pages the pool has."""
    need = [-(-n // bs) for n in lens]
    pool = sum(need) + 3
    perm = torch.randperm(pool, generator=g).numpy()
    t, at = np.zeros((len(lens), max(need)), dtype=np.int64), 0
    for i, n in enumerate(need):
        t[i, :n] = perm[at:at + n]
        at += n
    return t, pool


def want_latent(w, m, h):
    return no.latent_attention(w, m, h, EPS)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("case", ATTN, ids=str)
def test_latent_attention(dev, dtype, case):
    """Two sequences through the mixer: whole prompts, a late portion beside
    a short one, then single rows of unequal length. Pages are shuffled, free
    ones hold large values that must not show."""
    bs = 8 if case[1] == 24 else 16
    n = [150, 71]
    cases = [latent_case(case, k, dtype, seed=s) for s, k in enumerate(n)]
    w, m = cases[0][:2]
    hs = [c[2] for c in cases]
    want = [want_latent(w, m, h) for h in hs]
    mod = build_latent(w, m, dtype, dev)
    tables, pool = page_tables(n, bs, gen(3))
    kl = mod.spec.cache_layer()

    def run(meta, rows):
        x = torch.cat(rows).to(dtype).to(dev)
        with torch.inference_mode():
            return mod(x, cache, meta)

    def fresh():
        return (torch.full((pool, *kl.k_shape(bs)), 300.0, dtype=dtype,
                           device=dev),
                torch.empty(pool, *kl.v_shape(bs), dtype=dtype, device=dev))

    rms = float(want[0].pow(2).mean().sqrt())
    # whole prompts, then the same in portions
    for cuts in ([(0, 150)], [(0, 60), (60, 150)], [(0, 33), (33, 36),
                                                    (36, 118), (118, 150)]):
        cache = fresh()
        other = [(0, 71)] if len(cuts) == 1 else \
            [(0, 2), (2, 71)] + [None] * 2
        for a, b in zip(cuts, other):
            spans = [a] if b is None else [a, b]
            y = run(prompt_meta(spans, tables[:len(spans)], bs, dev),
                    [h[s:e] for h, (s, e) in zip(hs, spans)])
            close_rows(y, torch.cat([v[s:e] for v, (s, e) in zip(want, spans)]),
                  dtype, rms)
    # single rows over the cache that the last portions left
    for pos in ([149, 70], [0, 1], [15, 16], [32, 63], [100, 50]):
        y = run(decode_meta(pos, tables, bs, dev),
                [h[p:p + 1] for h, p in zip(hs, pos)])
        close_rows(y, torch.stack([v[p] for v, p in zip(want, pos)]), dtype, rms)
    # a row beside a portion
    d, p = decode_meta([149], tables[:1], bs, dev), \
        prompt_meta([(40, 71)], tables[1:], bs, dev)
    y = run(MixedMeta(decode=d, prefill=p, num_decode=1,
                      slot_mapping=torch.cat([d.slot_mapping,
                                              p.slot_mapping]),
                      positions=torch.cat([d.positions, p.positions])),
            [hs[0][149:], hs[1][40:]])
    close_rows(y, torch.cat([want[0][149:], want[1][40:]]), dtype, rms)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("window", [0, 700, 1000])
def test_long_rows_in_partitions(dev, dtype, window):
    """Rows that see several partitions, the last one partial."""
    case = (5, 24, 8, 40, 48, window, 8)
    n, bs = 1203, 16
    w, m, h = latent_case(case, n, dtype, seed=4)
    want = want_latent(w, m, h)
    mod = build_latent(w, m, dtype, dev)
    tables, pool = page_tables([n], bs, gen(5))
    kl = mod.spec.cache_layer()
    cache = (torch.zeros(pool, *kl.k_shape(bs), dtype=dtype, device=dev),
             None)
    with torch.inference_mode():
        y = mod(h.to(dtype).to(dev), cache,
                prompt_meta([(0, n)], tables, bs, dev))
        rms = float(want.pow(2).mean().sqrt())
        close_rows(y, want, dtype, rms)
        for pos in (n - 1, 1023, 1024, 899, 129, 3):
            meta = decode_meta([pos], tables, bs, dev)
            meta.max_len = 1500
            y = mod(h[pos:pos + 1].to(dtype).to(dev), cache, meta)
            close_rows(y, want[pos:pos + 1], dtype, rms)


def test_latent_cases_notice_mistakes():
    """Planted in the oracle: a window one token off, plain frequencies, the
    other pairing, a missing latent norm or gate."""
    case = ATTN[0]
    w, m, h = latent_case(case, 150, F32)
    good = want_latent(w, m, h)
    ref = float(good.pow(2).mean().sqrt())

    def off(w2=w, m2=m):
        return float((want_latent(w2, m2, h) - good).abs().max()) / ref

    assert off(m2={**m, "mask": {"size": 20}}) > 0.3
    assert off(m2={**m, "mask": {"size": 18}}) > 0.3
    assert off(m2={**m, "rot": {**m["rot"], "scaling": None}}) > 0.3
    assert off(m2={**m, "rot": None}) > 0.3
    assert off(w2={**w, "dkv.norm": torch.ones(48).double()}) > 0.1
    assert off(w2={**w, "g": w["g"] * 0.5}) > 0.1


# ------------------------------------------------------------------ state space

SSM = [
    # heads, vdim, state, groups, taps, norm groups
    (4, 24, 40, 2, 3, 4),
    (6, 48, 32, 3, 4, 2),
    (2, 64, 128, 1, 4, 1),
    (3, 13, 17, 3, 2, 3),                     # odd sizes
    (4, 80, 64, 4, 4, 4),                     # two blocks of values
    (8, 64, 256, 2, 5, 8),
    (2, 16, 300, 1, 4, 2),                    # beyond the chunk kernel
    (1, 24, 8, 1, 1, 1),                      # no history
]


def ssm_case(case, n, dtype, seed=0):
    """Weights and inputs; a few tokens are large, decays range from almost
    none to strong."""
    H, P, N, G, taps, ng = case
    g = gen(seed + H * P + N)
    W, inner, ch = 64, H * P, H * P + 2 * G * N
    m = dict(heads=H, vdim=P, state=N, groups=G, conv=taps, norm_groups=ng)
    w = {"in": rnd(g, inner + ch + H, W, dtype=BF16, std=W ** -0.5),
         "conv": rnd(g, ch, taps, dtype=BF16, std=0.7),
         "conv.b": rnd(g, ch, dtype=BF16, std=0.3),
         "dt_bias": (rnd(g, H) - 2.0).to(BF16).double(),
         "A_log": (rnd(g, H) * 1.5).to(BF16).double(),
         "D": rnd(g, H, dtype=BF16), "o": rnd(g, W, inner, dtype=BF16,
                                              std=inner ** -0.5),
         "norm": (1 + rnd(g, inner, std=0.2)).to(BF16).double()}
    h = rnd(g, n, W, dtype=dtype)
    for i in (0, 2, n // 3, n // 2):
        h[i] *= 3.0
    return w, m, h.to(dtype).double()


def build_ssm(w, m, dtype, dev):
    mod = Mamba2Mixer(SSMSpec.from_json(m), 64, EPS)
    for name, dst in mod.targets("").items():
        dst.copy_(w[name].float())
    return mod.to(dtype).to(dev)


def fresh_state(mod, slots, dtype, dev, value=7.0):
    """What an earlier sequence may have left in the slots."""
    return tuple(torch.full((slots, *s), value, dtype=dt or dtype,
                            device=dev)
                 for s, dt in mod.spec.cache_layer().tensors)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("case", SSM, ids=str)
def test_mamba2(dev, dtype, case):
    """Whole prompts, portions and single tokens of two sequences in stale
    slots; the slots are not the batch rows."""
    n = [150, 75]
    cases = [ssm_case(case, k, dtype, seed=s) for s, k in enumerate(n)]
    w, m = cases[0][:2]
    hs = [c[2] for c in cases]
    want = [no.mamba2(w, m, h, EPS) for h in hs]
    rms = float(want[0].pow(2).mean().sqrt())
    mod = build_ssm(w, m, dtype, dev)
    tables = np.zeros((2, 20), dtype=np.int64)
    slots = [3, 1]

    def run(meta, rows):
        x = torch.cat(rows).to(dtype).to(dev)
        with torch.inference_mode():
            return mod(x, state, meta)

    # (spans of sequence 0, spans of sequence 1); None = sits out
    for a, b in (([(0, 150)], [(0, 75)]),
                 ([(0, 64), (64, 150)], [(0, 2), (2, 75)]),
                 ([(0, 1), (1, 3), (3, 70), (70, 150)],
                  [None, (0, 3), (3, 5), (5, 75)])):
        state = fresh_state(mod, 4, dtype, dev)
        keep = [t[[0, 2]].clone() for t in state]
        for sa, sb in zip(a, b):
            live = [i for i, s in enumerate((sa, sb)) if s is not None]
            spans = [(sa, sb)[i] for i in live]
            y = run(prompt_meta(spans, tables[live], 16, dev,
                                [slots[i] for i in live]),
                    [hs[i][s:e] for i, (s, e) in zip(live, spans)])
            close_rows(y, torch.cat([want[i][s:e]
                                for i, (s, e) in zip(live, spans)]), dtype,
                  rms)
        for t, k in zip(state, keep):         # nobody else's slot
            assert torch.equal(t[[0, 2]], k)
    # single tokens: from the start, and on top of portions
    for first in (0, 1, 40):
        state = fresh_state(mod, 4, dtype, dev)
        if first:
            run(prompt_meta([(0, first), (0, first + 2)], tables, 16, dev,
                            slots), [hs[0][:first], hs[1][:first + 2]])
        for t in range(30):
            pos = [first + t, first + 2 + t] if first else [t, t]
            y = run(decode_meta(pos, tables, 16, dev, slots),
                    [h[p:p + 1] for h, p in zip(hs, pos)])
            close_rows(y, torch.stack([v[p] for v, p in zip(want, pos)]), dtype,
                  rms)
        # a portion after single tokens, beside a single token
        at = pos[0] + 1
        d = decode_meta([pos[1] + 1], tables[:1], 16, dev, slots[1:])
        p = prompt_meta([(at, at + 5)], tables[:1], 16, dev, slots[:1])
        y = run(MixedMeta(decode=d, prefill=p, num_decode=1,
                          slot_mapping=torch.cat([d.slot_mapping,
                                                  p.slot_mapping]),
                          positions=torch.cat([d.positions, p.positions])),
                [hs[1][pos[1] + 1:pos[1] + 2], hs[0][at:at + 5]])
        close_rows(y, torch.cat([want[1][pos[1] + 1:pos[1] + 2],
                            want[0][at:at + 5]]), dtype, rms)


@pytest.mark.parametrize("dev", DEVICES)
def test_rows_without_a_slot_leave_states_alone(dev):
    w, m, h = ssm_case(SSM[0], 4, BF16)
    mod = build_ssm(w, m, BF16, dev)
    state = fresh_state(mod, 2, BF16, dev)
    keep = [t.clone() for t in state]
    with torch.inference_mode():
        mod(h[:2].to(BF16).to(dev), state, decode_meta(
            [0, 5], np.zeros((2, 4), dtype=np.int64), 16, dev, [-1, -1]))
    for t, k in zip(state, keep):
        assert torch.equal(t, k)


def test_state_carries_far():
    """With slow decays a token from the first chunk still shows at the end:
    the cases above see a state that is lost between chunks."""
    w, m, h = ssm_case(SSM[1], 150, F32)
    good = no.mamba2(w, m, h, EPS)
    cut = no.mamba2(w, m, h[64:], EPS)
    ref = float(good.pow(2).mean().sqrt())
    assert float((cut[40:] - good[104:]).abs().max()) / ref > 0.1


def test_ssm_cases_notice_mistakes():
    w, m, h = ssm_case(SSM[1], 100, F32)
    good = no.mamba2(w, m, h, EPS)
    ref = float(good.pow(2).mean().sqrt())

    def off(w2=w, m2=m):
        return float((no.mamba2(w2, m2, h, EPS) - good).abs().max()) / ref

    for name in ("A_log", "D", "dt_bias", "conv.b", "norm", "conv"):
        assert off({**w, name: w[name] * 0.5}) > 0.05, name
    assert off({**w, "conv": w["conv"].flip(1)}) > 0.3
    assert off(m2={**m, "norm_groups": 1}) > 0.05
    assert off(m2={**m, "groups": 3, "heads": 6}) == 0


# ----------------------------------------------------------------------- model

def attn(heads, dim, rot, vdim, rank, size, ff, scale=None, base=1e3,
         scaling=YARN):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot,
                      "vdim": vdim, "kv_rank": rank,
                      "scale": scale or 3.0 / math.sqrt(dim + rot),
                      "mask": {"size": size},
                      "rot": {"dims": rot, "base": base,
                              "scaling": scaling}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def mamba(heads, vdim, state, groups, conv, norm_groups, ff):
    return {"type": "mamba2",
            "mixer": {"heads": heads, "vdim": vdim, "state": state,
                      "groups": groups, "conv": conv,
                      "norm_groups": norm_groups},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


CONFIGS = {
    # layers of different shapes, one without a feed-forward, a loop in the
    # middle that begins with a Mamba-2 layer
    "varied": {"architecture": "Nibezen", "vocab": 97, "width": 72,
               "norm": {"eps": 1e-5}, "residual_mult": 0.8,
               "loop": {"start": 1, "stop": 3, "times": 2}, "layers": [
                   attn(3, 24, 8, 40, 36, 21, 96),
                   mamba(4, 20, 24, 2, 3, 4, 0),
                   attn(5, 16, 12, 24, 64, 50, 130, scaling=None),
                   mamba(2, 48, 40, 1, 4, 1, 52),
                   attn(2, 20, 4, 12, 20, 9, 0, base=50.0)]},
    # the loop from the first layer to the last
    "wide": {"architecture": "Nibezen", "vocab": 300, "width": 128,
             "norm": {"eps": 3e-6}, "residual_mult": 0.5,
             "loop": {"start": 0, "stop": 2, "times": 3}, "layers": [
                 attn(16, 64, 32, 64, 128, 70, 264),
                 mamba(4, 64, 128, 2, 4, 2, 264)]},
    # sizes of one, the window of one token, a loop of one pass
    "single": {"architecture": "Nibezen", "vocab": 33, "width": 20,
               "norm": {"eps": 1e-6}, "residual_mult": 1.0,
               "loop": {"start": 1, "stop": 2, "times": 1}, "layers": [
                   attn(1, 12, 2, 20, 8, 1, 28),
                   mamba(1, 8, 8, 1, 1, 1, 0),
                   attn(1, 8, 6, 20, 12, 300, 0)]},
    # recurrent layers only, no loop
    "recurrent": {"architecture": "Nibezen", "vocab": 50, "width": 48,
                  "norm": {"eps": 1e-5}, "residual_mult": 0.9,
                  "loop": None, "layers": [
                      mamba(3, 32, 16, 3, 2, 3, 64),
                      mamba(2, 16, 32, 1, 4, 1, 40)]},
}


def make_weights(cfg, seed=0):
    """bf16 tensors under their checkpoint names; queries and keys are
    large enough for single keys to stand out."""
    g = gen(seed)
    W, out = cfg["width"], {}

    def add(name, *shape, std=None, mean=0.0):
        std = std if std is not None else 1.0 / math.sqrt(shape[-1])
        out[name] = (torch.randn(shape, generator=g) * std + mean).to(BF16)

    add("embed", cfg["vocab"], W, std=1.0)
    add("head", cfg["vocab"], W)
    add("final.norm", W, std=0.2, mean=1.0)
    if cfg["loop"]:
        add("loop.step", cfg["loop"]["times"], W, std=0.5)
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        add(p + "norm1", W, std=0.2, mean=1.0)
        add(p + "ls1", W, std=0.3, mean=0.8)
        H = m["heads"]
        if l["type"] == "latent_attention":
            D, R, E, K = (m[k] for k in ("dim", "rot_dim", "vdim", "kv_rank"))
            for n, rows, cols in (("q", H * (D + R), W), ("dkv", K + R, W),
                                  ("uk", H * D, K), ("uv", H * E, K),
                                  ("g", H, W), ("o", W, H * E)):
                add(p + "mix." + n, rows, cols)
            add(p + "mix.dkv.norm", K, std=0.2, mean=1.0)
        else:
            inner = H * m["vdim"]
            ch = inner + 2 * m["groups"] * m["state"]
            add(p + "mix.in", inner + ch + H, W)
            add(p + "mix.conv", ch, m["conv"], std=0.6)
            add(p + "mix.conv.b", ch, std=0.3)
            add(p + "mix.dt_bias", H, std=0.7, mean=-2.0)
            add(p + "mix.A_log", H, std=1.0)
            add(p + "mix.D", H, std=1.0)
            add(p + "mix.norm", inner, std=0.2, mean=1.0)
            add(p + "mix.o", W, inner)
        if l["mlp"]:
            F = l["mlp"]["ff"]
            add(p + "norm2", W, std=0.2, mean=1.0)
            add(p + "ls2", W, std=0.3, mean=0.8)
            add(p + "mlp.gate", F, W)
            add(p + "mlp.up", F, W)
            add(p + "mlp.down", W, F)
    return out


@pytest.fixture(scope="session")
def folders(tmp_path_factory):
    from safetensors.torch import save_file
    made = {}
    for name, cfg in CONFIGS.items():
        d = tmp_path_factory.mktemp(name)
        (d / "config.json").write_text(json.dumps(cfg))
        w = make_weights(cfg)
        save_file(w, str(d / "model.safetensors"))
        made[name] = (str(d), cfg, w)
    return made


def prompt(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=gen(seed)).tolist()


_WANT = {}


def want_logits(name, cfg, w, ids):
    key = (name, tuple(ids))
    if key not in _WANT:
        _WANT[key] = no.forward(cfg, w, ids)
    return _WANT[key]


def engine_for(folder, dev, dtype, blocks=64, seqs=4, **kw):
    return LLMEngine(EngineConfig(
        model=folder, dtype=dtype, max_num_seqs=seqs, kv_cache_blocks=blocks,
        max_model_len=640, eos_token_id=-1, **kw), device=dev)


MODEL_TOL = {"float32": 2e-4, "bfloat16": 0.08}


def check_rows(got, want, dtype):
    """Root-mean-square error of every position's logits over the spread of
    all of them."""
    got, want = got.double().cpu(), want.double()
    err = (got - want).pow(2).mean(-1).sqrt() / want.std()
    assert float(err.max()) < MODEL_TOL[dtype], err


def run_cut(eng, sid, ids, cuts):
    """Feed ids in portions of the given sizes; all positions' logits."""
    out, at = [], 0
    for n in cuts:
        part = ids[at:at + n]
        out.append(eng.extend([(sid, part, list(range(len(part))))])
                   .float().cpu())
        at += len(part)
    assert at == len(ids)
    return torch.cat(out)


def cuts_of(total, sizes):
    out, i = [], 0
    while sum(out) < total:
        out.append(min(sizes[i % len(sizes)], total - sum(out)))
        i += 1
    return out


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_portions_and_decode(folders, dev, dtype, name):
    folder, cfg, w = folders[name]
    eng = engine_for(folder, dev, dtype)
    ids = prompt(cfg, 139, 5)
    want = want_logits(name, cfg, w, ids)
    free = eng.num_free_blocks()
    for k, sizes in enumerate(([139], [2], [3, 16, 2, 33], [64], [17, 1],
                               [100] + [1] * 39)):
        got = run_cut(eng, f"s{k}", ids, cuts_of(139, sizes))
        check_rows(got, want, dtype)
        eng.release(f"s{k}")
    assert eng.num_free_blocks() == free


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("name", ["varied", "wide"])
def test_token_by_token(folders, dev, name):
    folder, cfg, w = folders[name]
    eng = engine_for(folder, dev, "float32")
    ids = prompt(cfg, 90, 6)
    got = run_cut(eng, "a", ids, [1] * 90)
    check_rows(got, want_logits(name, cfg, w, ids), "float32")


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("name", ["varied", "single"])
def test_layers_one_by_one(folders, dev, name):
    folder, cfg, w = folders[name]
    eng = engine_for(folder, dev, "float32", enforce_eager=True)
    ids = prompt(cfg, 60, 7)
    want, tap = [], []
    no.forward(cfg, w, ids, layers_out=want)
    eng.model.layer_tap = tap
    eng.extend([("a", ids, [])])
    assert len(tap) == len(want)
    for a, b in zip(tap, want):
        close(a, b, F32)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_and_reused_slots(folders, dev, dtype):
    """Portions beside single tokens, requests left out of steps, and a pool
    so small that pages and state slots are used again."""
    name = "varied"
    folder, cfg, w = folders[name]
    eng = engine_for(folder, dev, dtype, blocks=20, seqs=3)
    lens = {"a": 130, "b": 41, "c": 77, "d": 102, "e": 1, "f": 64}
    ids = {s: prompt(cfg, n, 20 + i) for i, (s, n) in enumerate(lens.items())}
    got = {s: [] for s in ids}
    at = dict.fromkeys(ids, 0)
    sizes = {"a": [29, 1, 2, 1, 40, 1, 1], "b": [2, 1, 1, 7], "c": [1, 33, 2],
             "d": [64, 1, 3], "e": [1], "f": [1, 1, 62]}
    live, queue, turn = ["a", "b"], ["c", "d", "e", "f"], 0
    while live:
        turn += 1
        if queue and len(live) < 3 and sum(
                -(-lens[s] // 16) for s in live + queue[:1]) <= 20:
            live.append(queue.pop(0))
        entries = []
        for j, s in enumerate(live):
            if (turn + j) % 4 == 0 and len(live) > 1:
                continue                       # sits this step out
            k = len(got[s]) % len(sizes[s])
            n = min(sizes[s][k], lens[s] - at[s])
            entries.append((s, ids[s][at[s]:at[s] + n], list(range(n))))
        out = eng.extend(entries)
        row = 0
        for s, part, _ in entries:
            got[s].append(out[row:row + len(part)].float().cpu())
            row += len(part)
            at[s] += len(part)
            if at[s] == lens[s]:
                eng.release(s)
                live.remove(s)
    assert eng.num_free_blocks() == 20
    for s in ids:
        check_rows(torch.cat(got[s]), want_logits(name, cfg, w, ids[s]),
                   dtype)


def oracle_greedy(cfg, w, ids, n):
    ids = list(ids)
    for _ in range(n):
        ids.append(int(no.forward(cfg, w, ids)[-1].argmax()))
    return ids[-n:]


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("mixed", [False, True])
def test_greedy_generation(folders, dev, mixed):
    """Through generate(): chunked prompts, a shared prefix (which a model
    with recurrent state must compute again), preemption."""
    folder, cfg, w = folders["varied"]
    prompts = [prompt(cfg, n, 40 + n) for n in (50, 3, 61)]
    prompts.append(prompts[0][:32] + prompt(cfg, 9, 3))     # shared prefix
    if "want" not in _GREEDY:
        _GREEDY["want"] = [oracle_greedy(cfg, w, p, 14) for p in prompts]
    want = _GREEDY["want"]
    sp = SamplingParams(temperature=0.0, max_tokens=14, ignore_eos=True)
    for kw in (dict(max_prefill_tokens=4096),
               dict(max_prefill_tokens=24),
               dict(max_prefill_tokens=24, blocks=10)):
        eng = engine_for(folder, dev, "float32", mixed_steps=mixed, **kw)
        eng.generate(prompts, sp)
        full = [eng.seqs[f"gen-1-{i}"] for i in range(4)]
        outs = [(s.prompt_ids + s.output_ids)[len(p):]
                for s, p in zip(full, prompts)]
        assert outs == want, kw


_GREEDY = {}


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("name,dtype,n,cuts", [
    ("varied", "float32", 300, [5] + [1] * 295),
    ("varied", "bfloat16", 300, [5] + [1] * 295),
    ("wide", "bfloat16", 560, [2, 300, 198] + [1] * 60),
    ("wide", "float32", 560, [500] + [1] * 60)])
def test_long_decode(folders, dev, name, dtype, n, cuts):
    """Far past every window, page by page."""
    folder, cfg, w = folders[name]
    ids = prompt(cfg, n, 8)
    eng = engine_for(folder, dev, dtype)
    got = run_cut(eng, "a", ids, cuts)
    check_rows(got, want_logits(name, cfg, w, ids), dtype)


def test_model_tests_notice_mistakes(folders):
    """Planted in the oracle: the tolerances above would catch each."""
    folder, cfg, w = folders["varied"]
    ids = prompt(cfg, 139, 5)
    good = want_logits("varied", cfg, w, ids)

    def off(c2, w2):
        bad = no.forward(c2, w2, ids)
        return float(((bad - good).pow(2).mean(-1).sqrt()
                      / good.std()).max())

    for i in (0, 2, 4):
        c2 = json.loads(json.dumps(cfg))
        c2["layers"][i]["mixer"]["mask"]["size"] += 1
        assert off(c2, w) > 10 * MODEL_TOL["float32"], i
    assert off({**cfg, "residual_mult": 0.9}, w) > 0.08
    swapped = {**w, "loop.step": w["loop.step"].flip(0)}
    assert off(cfg, swapped) > 0.08
    for n in ("l0.ls1", "l2.ls2", "l1.mix.dt_bias", "l3.mix.A_log",
              "l1.mix.conv.b", "l3.mix.D", "l2.mix.g", "l4.mix.dkv.norm"):
        assert off(cfg, {**w, n: w[n] * 0.5}) > 10 * MODEL_TOL["float32"], n


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_graph_replays_match_eager(folders, dtype):
    """Captured decode, replayed many times with eager prompts between; the
    captures' warm-up leaves states alone."""
    folder, cfg, w = folders["wide"]
    outs = []
    for eager in (True, False):
        eng = engine_for(folder, "cuda", dtype, enforce_eager=eager)
        got = []
        for sid in "abc":
            eng.extend([(sid, prompt(cfg, 40 + ord(sid) % 7, 3), [])])
        for i in range(12):
            ent = [(s, [(7 * i + ord(s)) % cfg["vocab"]], [0])
                   for s in "abc"[:1 + i % 3]]
            out = eng.extend(ent)
            got.append(out.float().cpu())
            if i % 4 == 3:
                eng.extend([("p%d" % i, prompt(cfg, 33, i), [])])
                eng.release("p%d" % i)
        outs.append(torch.cat(got))
    check_rows(outs[1], outs[0], dtype)


# ------------------------------------------------------------------- framework

def test_config_reader():
    cfg = NibezenConfig.from_json(CONFIGS["varied"], "x")
    assert [l.ff for l in cfg.layers] == [96, 0, 130, 52, 0]
    assert [r.layer for r in cfg.runs()] == [0, 1, 2, 1, 2, 3, 4]
    assert [r.loop_pass for r in cfg.runs()] == [-1, 0, -1, 1, -1, -1, -1]
    kinds = [isinstance(l, StateLayer) for l in cfg.kv_layers()]
    assert kinds == [False, True, False, True, False, True, False]
    assert cfg.kv_layers()[0].k_dim == 40 + 8
    assert cfg.layers[2].mixer.rotary.scaling is None
    assert len(NibezenConfig.from_json(CONFIGS["recurrent"]).runs()) == 2
    for path, value in ((("layers", 0, "type"), "other"),
                        (("layers", 0, "mlp", "kind"), "other"),
                        (("layers", 1, "mixer", "groups"), 3),
                        (("layers", 1, "mixer", "norm_groups"), 7),
                        (("layers", 0, "mixer", "rot", "dims"), 7),
                        (("loop", "stop"), 9)):
        bad = json.loads(json.dumps(CONFIGS["varied"]))
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ValueError):
            NibezenConfig.from_json(bad)
    with pytest.raises(ValueError):
        NibezenForCausalLM(cfg, tp_size=2)


def test_small_tensors_keep_their_bits():
    m = NibezenForCausalLM(PRESETS["tiny-nibezen"]).to(BF16)
    a, s = m.layers[0], m.layers[1]
    assert m.embed_tokens.weight.dtype == a.mixer.uk.dtype == BF16
    for t in (a.norm1_w, a.ls1, a.norm2_w, a.mixer.kv_norm_w, s.mixer.conv_w,
              s.mixer.dt_bias, s.mixer.A_log, s.mixer.D, s.mixer.norm_w,
              m.final_norm_w, m.loop_step):
        assert t.dtype == F32
    assert a.mixer.freqs.dtype == torch.float64


def test_registry(tmp_path, folders):
    folder, cfg, w = folders["varied"]
    assert registry.get_config(folder).vocab_size == 97
    assert registry.get_config("tiny-nibezen") is PRESETS["tiny-nibezen"]
    assert registry.model_class(registry.get_config(folder)) \
        is NibezenForCausalLM
    from safetensors.torch import save_file
    for change in ("missing", "shape"):
        d = tmp_path / change
        d.mkdir()
        (d / "config.json").write_text(json.dumps(cfg))
        w2 = dict(w)
        if change == "missing":
            del w2["l1.mix.A_log"]
        else:
            w2["l0.mix.q"] = w2["l0.mix.q"][:-1].contiguous()
        save_file(w2, str(d / "model.safetensors"))
        with pytest.raises(ValueError):
            registry.build_model(str(d), F32, torch.device("cpu"))


def test_state_in_the_cache_manager(folders):
    folder, cfg, w = folders["varied"]
    eng = engine_for(folder, "cpu", "bfloat16", seqs=3)
    layers = eng.model_cfg.kv_layers()
    for l, c in zip(layers, eng.kv.caches):
        if isinstance(l, StateLayer):
            assert c[0].shape[0] == c[1].shape[0] == 3
            assert c[0].dtype == BF16 and c[1].dtype == F32
        else:
            assert c[0].shape[0] == 64
    want = sum(t.numel() * t.element_size() for l, c in
               zip(layers, eng.kv.caches) if isinstance(l, StateLayer)
               for t in c)
    assert KVCache.state_bytes(layers, 3, BF16) == want
    # a cached page has no state to go with it
    assert eng.cfg.enable_prefix_caching and not eng.prefix_caching
    assert KVCache.block_bytes(0, 0, 0, 16, BF16, layers) == sum(
        2 * 16 * l.k_dim for l in layers if not isinstance(l, StateLayer))


def test_sizes_for_the_planner():
    cfg = registry.get_config("nibezen-1b")
    emb, rest = cfg.num_weights()
    with torch.device("meta"):
        n = sum(p.numel() for p in NibezenForCausalLM(cfg).parameters())
    # the transposed copy of W_uk and padding are extra
    assert 1.0 <= n / (emb + rest) < 1.06
    assert cfg.activation_bytes(10) > 0


@pytest.mark.parametrize("dev", DEVICES)
def test_replay(folders, tmp_path, monkeypatch, capsys, dev):
    """The replay program end to end; ended requests give their slots back."""
    folder, cfg, w = folders["varied"]
    a, b = prompt(cfg, 20, 1), prompt(cfg, 9, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:12],
                                      "want": [11, 0]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b, "want": []},
                                     {"id": "a", "tokens": a[12:13],
                                      "want": []}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "b2", "tokens": b, "want": [8]},
                                     {"id": "a", "tokens": a[13:],
                                      "want": [0, 6]}], "end": ["a", "b2"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO(
        "\n".join(json.dumps(s) for s in steps) + "\n"))
    assert replay.main(["--model", folder, "--dtype", "float32", "--out",
                        str(tmp_path), "--max-tokens", "64", "--device",
                        "cuda:0" if dev == "cuda" else dev]) == 0
    said = capsys.readouterr().out.splitlines()
    assert [s for s in said if s.startswith("done")] == \
        ["done 0", "done 1", "done 2"]
    wa, wb = (want_logits("varied", cfg, w, t) for t in (a, b))
    assert not (tmp_path / "1.f32").exists()
    for step, want in ((0, [wa[11], wa[0]]), (2, [wb[8], wa[13], wa[19]])):
        got = np.fromfile(tmp_path / f"{step}.f32", dtype="<f4")
        check_rows(torch.from_numpy(got).view(len(want), 97),
                   torch.stack(want), "float32")
