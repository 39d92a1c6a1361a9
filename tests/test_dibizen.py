"""Dibizen against its plain full-sequence oracle: every mechanism alone,
then the model through the engine (portions, decoding, mixed batches, reused
pages and state slots, greedy generation). Each test runs on the CPU
reference ops and, marked gpu, on the HIP kernels."""
import io
import json
import math

import numpy as np
import pytest
import torch

import dibizen_oracle as do
from helix_amd.engine import replay
from helix_amd.engine.kv_cache import KVCache
from helix_amd.engine.sampling_params import SamplingParams
from helix_amd.models import registry
from helix_amd.models.dibizen import (MIXERS, PRESETS, DibizenConfig,
                                      DibizenForCausalLM, LayerSpec)
from helix_amd.models.gla import LightningSpec
from helix_amd.models.meta import MixedMeta, StateLayer
from helix_amd.models.mixer_group import MixerGroup
from helix_amd.models.moe import Mixture, MixtureSpec
from helix_amd.models.rotary_attention import (QueryTemperature,
                                               RotaryTables)
from helix_amd.models.selective import SelectiveSpec
from helix_amd.ops import build, routed
from helix_amd.ops.routed import RouterParams
from test_nibezen import (BF16, DEVICES, F32, MODEL_TOL, check_rows, close,
                          cuts_of, decode_meta, engine_for, gen, prompt,
                          prompt_meta, rnd, run_cut)

EPS = 1e-5


def close_rows(got, want, dtype, rms):
    """A whole mixer; in bf16 rows are judged by their rms error."""
    if dtype == F32:
        return close(got, want, dtype, rms)
    err = (got.double().cpu() - want.double()).pow(2).mean(-1).sqrt() / rms
    assert float(err.max()) < 0.06, err


def bf16_exact(g, *shape, std=None, mean=0.0):
    std = std if std is not None else shape[-1] ** -0.5
    return (torch.randn(shape, generator=g) * std + mean).to(BF16).double()


# -------------------------------------------------------------------- streams

def hyper_case(g, T, S, W):
    c = dict(into=rnd(g, S), mix=rnd(g, S, S), out=rnd(g, S))
    norm = {"n": 1 + rnd(g, W, std=0.3), "n.b": rnd(g, W, std=0.3),
            "n.alpha": torch.tensor(0.7, dtype=torch.float64)}
    return c, norm, rnd(g, T, S, W)


def on(dev, t, dt=F32):
    return t.to(dt).to(dev).contiguous()


def tanh_norm(norm, dev):
    return routed.TanhNorm(on(dev, norm["n.alpha"].reshape(1)),
                           on(dev, norm["n"]), on(dev, norm["n.b"]))


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,S,W", [(3, 3, 64), (5, 1, 250), (2, 2, 1028),
                                   (600, 4, 96), (1, 5, 77), (9, 8, 40),
                                   (2, 6, 33), (4, 7, 64)])
def test_streams(dev, dtype, T, S, W):
    g = gen(T + S + W)
    c, norm, x = hyper_case(g, T, S, W)
    tn = tanh_norm(norm, dev)
    back = routed.Return(on(dev, c["mix"]), on(dev, c["out"]))
    into = on(dev, c["into"])
    # a sublayer's result
    y = rnd(g, T, W, dtype=dtype)
    want = torch.stack(do.write_streams(list(x.unbind(1)), y, c["mix"],
                                        c["out"]), 1)
    h_want = do.dyn_tanh(do.read_streams(list(want.unbind(1)), c["into"]),
                         norm, "n")
    xd, tap = on(dev, x), torch.empty(T, W, device=dev)
    h = routed.hyper_step(xd, on(dev, y, dtype), back, into, tn, tap)
    close(xd, want, F32)
    close(tap, want.sum(1), F32)
    close(h, h_want, dtype)
    # a mixture's rows: two experts, one identity; row 0 is nobody's
    K = 3
    rows, self = rnd(g, T * K + 1, W, dtype=dtype), rnd(g, T, W, dtype=dtype)
    rows[0] = float("nan")
    slot = 1 + torch.randperm(T * K, generator=g).int().view(T, K)
    slot[:, 1] = -1
    wt = rnd(g, T, K)
    y = sum(wt[:, k, None] * (self if k == 1 else rows[slot[:, k].long()])
            for k in range(K))
    want = torch.stack(do.write_streams(list(x.unbind(1)), y, c["mix"],
                                        c["out"]), 1)
    xd = on(dev, x)
    h = routed.hyper_step(xd, routed.RoutedRows(
        on(dev, rows, dtype), slot.to(dev), on(dev, wt),
        on(dev, self, dtype)), back, into, tn)
    close(xd, want, F32)
    close(h, do.dyn_tanh(do.read_streams(list(want.unbind(1)), c["into"]),
                         norm, "n"), dtype)
    # the beginning
    emb, places = rnd(g, 11, W, dtype=dtype), rnd(g, 40, W, dtype=dtype)
    ids = torch.randint(0, 11, (T,), generator=g)
    pos = torch.randint(0, 40, (T,), generator=g)
    xd = torch.empty(T, S, W, device=dev)
    h = routed.hyper_embed(xd, ids.to(dev), pos.to(dev), on(dev, emb, dtype),
                           on(dev, places, dtype), into, tn)
    e = emb[ids] + places[pos]
    close(xd, e[:, None].expand(T, S, W), F32)
    close(h, do.dyn_tanh(e * c["into"].sum(), norm, "n"), dtype)


def test_mix_is_from_to():
    """Planted in the oracle: a transposed mixing matrix shows."""
    c, _, x = hyper_case(gen(0), 4, 3, 16)
    xs, y = list(x.unbind(1)), rnd(gen(1), 4, 16)
    a = do.write_streams(xs, y, c["mix"], c["out"])
    b = do.write_streams(xs, y, c["mix"].T, c["out"])
    assert float((a[0] - b[0]).abs().max()) > 0.1


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("shape", [(3, 450), (1, 5), (7, 1001)])
def test_softcap(dev, shape):
    x = rnd(gen(2), *shape, std=40.0)
    got = routed.softcap(on(dev, x), 12.0)
    close(got, 12.0 * torch.tanh(x / 12.0), F32)


# ----------------------------------------------------------- mixture of experts

ROUTERS = [RouterParams(18, 5, 2, 5, 3), RouterParams(6, 2, 2, 4, 2),
           RouterParams(5, 3), RouterParams(1, 1), RouterParams(3, 2, 5, 2, 1),
           RouterParams(60, 6, 4, 8, 1), RouterParams(250, 9, 50, 10, 4),
           RouterParams(7, 8, 1, 4, 4), RouterParams(640, 12, 0, 5, 2)]


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("p", ROUTERS, ids=str)
@pytest.mark.parametrize("T", [1, 7, 300])
def test_choice_of_experts(dev, p, T):
    g, n = gen(T), p.outputs
    z, corr = rnd(g, T, n, std=2.0), rnd(g, n, std=0.1)
    # all choice scores negative: what is shut out must not come back as zero
    corr = corr - 2.0
    ids, w = routed.choose_experts(on(dev, z), on(dev, corr), p)
    r = dict(top=p.top, experts=p.experts,
             groups=dict(count=p.groups, keep=p.keep))
    for t in range(T):
        s = do.softmax(z[t])
        want = do.choose(s, corr, r)
        assert sorted(ids[t].tolist()) == sorted(want)
        total = sum(float(s[e]) for e in want) + 1e-20
        for e, v in zip(ids[t].tolist(), w[t].tolist()):
            assert abs(v - float(s[e]) / total) < 2e-6


def test_choice_notices_mistakes():
    """Planted in the oracle: correction, groups and the weights' scores each
    change the result of the cases above."""
    p = ROUTERS[0]
    g = gen(300)
    z, corr = rnd(g, 300, 20, std=2.0), rnd(g, 20, std=0.1)
    r = dict(top=p.top, experts=p.experts, groups=dict(count=5, keep=3))
    flat = {**r, "groups": dict(count=5, keep=5)}
    s = [do.softmax(row) for row in z]
    good = [do.choose(x, corr, r) for x in s]
    assert any(sorted(a) != sorted(do.choose(x, 0 * corr, r))
               for a, x in zip(good, s))
    assert any(sorted(a) != sorted(do.choose(x, corr, flat))
               for a, x in zip(good, s))
    assert any(max(e) >= p.experts for e in good)


def mixture_case(W, F, p, T, dtype, seed=0):
    g = gen(seed + W + T)
    w = {"router": bf16_exact(g, p.outputs, W, std=2.0 * W ** -0.5),
         "correction": bf16_exact(g, p.outputs, std=0.05)}
    for e in range(p.experts):
        w[f"e{e}.up"] = bf16_exact(g, F, W)
        w[f"e{e}.down"] = bf16_exact(g, W, F)
    h = rnd(g, T, W, dtype=dtype)
    return w, h


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("W,F,p,T", [
    (40, 24, ROUTERS[0], 33),                  # inner sizes between the tiles
    (72, 130, ROUTERS[1], 50),                 # not in 16-byte pieces
    (20, 28, ROUTERS[2], 9),
    (8, 8, ROUTERS[3], 3),
    (64, 64, ROUTERS[4], 1),
    (176, 112, ROUTERS[0], 60),                # streams of few rows, of many
    (136, 160, ROUTERS[2], 70),
    (64, 128, ROUTERS[0], 25),                 # tiles of 32, 128, 256 rows
    (128, 192, ROUTERS[1], 420),
    (64, 320, ROUTERS[7], 600),
    (320, 64, ROUTERS[3], 129),
    (64, 72, ROUTERS[6], 130),                 # most experts have few rows
])
def test_mixture(dev, dtype, W, F, p, T):
    w, h = mixture_case(W, F, p, T, dtype)
    r = dict(experts=p.experts, top=p.top, identity=p.identity,
             groups=dict(count=p.groups, keep=p.keep))
    mod = Mixture(MixtureSpec(F, p), W).to(dtype)
    with torch.inference_mode():
        targets = mod.targets("")
        assert set(targets) == set(w)
        for n, t in targets.items():
            t.copy_(w[n].to(t.dtype))
        mod = mod.to(dev)
        out = mod(on(dev, h, dtype))
        streams = torch.zeros(T, 1, W, device=dev)
        one = torch.ones(1, device=dev)
        routed.hyper_step(streams, out, routed.Return(one.view(1, 1), one),
                          one, routed.TanhNorm(one, torch.ones(W, device=dev),
                                               torch.zeros(W, device=dev)))
    want = do.mixture(h, w, "", {"router": r})
    close_rows(streams[:, 0], want, dtype, float(want.pow(2).mean().sqrt()))


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T", [1, 9])
def test_identity_experts_alone(dev, dtype, T):
    """No expert with weights is chosen, so no row of theirs is written, and
    what lies in that memory must not show."""
    W, p = 48, RouterParams(4, 2, 4, 2, 1)
    w, h = mixture_case(W, 16, p, T, dtype)
    w["correction"][4:] = 3.0
    mod = Mixture(MixtureSpec(16, p), W).to(dtype)
    with torch.inference_mode():
        for n, t in mod.targets("").items():
            t.copy_(w[n].to(t.dtype))
        mod = mod.to(dev)
        out = mod(on(dev, h, dtype))
        assert (out.slot == -1).all()
        out.rows.fill_(float("nan"))
        x, one = torch.zeros(T, 1, W, device=dev), torch.ones(1, device=dev)
        routed.hyper_step(x, out, routed.Return(one.view(1, 1), one), one,
                          routed.TanhNorm(one, torch.ones(W, device=dev),
                                          torch.zeros(W, device=dev)))
    close(x[:, 0], h, F32)


@pytest.mark.gpu
@pytest.mark.parametrize("T", [1, 5, 64, 1500])
@pytest.mark.parametrize("p", [ROUTERS[0], ROUTERS[5], ROUTERS[8]], ids=str)
@pytest.mark.parametrize("height", [16, 64, 128])
def test_expert_lists(T, p, height):
    """Every pair once, tiles cover each expert's rows, and no others."""
    z = rnd(gen(T), T, p.outputs, std=2.0).float().cuda()
    corr = torch.zeros(p.outputs, device="cuda")
    ids, _, rank, hist = routed._route(z, corr, p)
    l = routed.expert_lists(ids, rank, hist, p, height, "tile")
    ids, slot = ids.cpu().flatten(), l.slot.cpu().flatten()
    order, tiles = l.order.cpu(), l.tiles.cpu().tolist()
    real = (ids < p.experts).nonzero().flatten()
    assert (slot[ids >= p.experts] == -1).all()
    assert sorted(slot[real].tolist()) == list(range(len(real)))
    assert (order[slot[real].long()] == real.int()).all()
    seen = []
    for e, row, rows, _ in tiles:
        if e < 0:
            continue
        assert 1 <= rows <= height
        assert (ids[order[row:row + rows].long()] == e).all()
        seen += range(row, row + rows)
    assert sorted(seen) == list(range(len(real)))


# ------------------------------------------------------------- mixers as a whole

def attn(heads, kv_heads, dim, vdim, coef=0.35, every=16, scale=None,
         kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim,
             scale=scale or 3.0 / math.sqrt(dim),
             q_temp=dict(coef=coef, every=every))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def lightning(dim, vdim, *decay):
    return {"type": "lightning", "mixer": dict(
        heads=len(decay), dim=dim, vdim=vdim, decay=list(decay))}


def mamba(inner, state, conv, dt_rank):
    return {"type": "mamba1", "mixer": dict(inner=inner, state=state,
                                            conv=conv, dt_rank=dt_rank)}


def mixer_weights(layer, W, seed=0):
    """bf16-exact weights; the keys' projection is that of the group's first
    query head for rows shifted by one column, so a row that is another one
    shifted meets it with a score that stands out, and not itself."""
    g, m, out = gen(seed), layer["mixer"], {}

    def add(name, *shape, std=None, mean=0.0):
        out[name] = bf16_exact(g, *shape, std=std, mean=mean)

    if layer["type"] == "mamba1":
        I, N, R = m["inner"], m["state"], m["dt_rank"]
        add("in", 2 * I, W)
        add("conv", I, m["conv"])
        add("conv.b", I, std=0.2)
        add("x", R + 2 * N, I, std=2.0 * I ** -0.5)
        add("dt", I, R, std=0.7 * R ** -0.5)
        add("dt.b", I, std=1.0, mean=-3.0)
        # decays from almost none to several bits a token
        add("A_log", I, N, std=1.5, mean=-0.5)
        add("D", I, std=0.3, mean=1.0)
        add("o", W, I)
        return out
    H, D, E = m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads", H)
    add("q", H * D, W)
    if "kv_from" not in m:
        if layer["type"] == "attention":
            out["k"] = out["q"].view(G, H // G, D, W)[:, 0].reshape(
                G * D, W).roll(-1, 1)
        else:
            add("k", G * D, W)
        add("v", G * E, W)
    add("g", H * E, W)
    add("o", W, H * E)
    if layer["type"] == "lightning":
        add("norm", H * E, std=0.2, mean=1.0)
    return out


def oracle_mixer(layer, h, w, kv=None):
    m = layer["mixer"]
    if layer["type"] == "attention":
        return do.attention(h, w, "", m, kv or do.keys_values(h, w, "", m))
    if layer["type"] == "lightning":
        return do.lightning(h, w, "", m, EPS)
    return do.mamba1(h, w, "", m)


def build_mixer(layer, w, W, dtype, dev):
    spec = LayerSpec.of(MIXERS[layer["type"]](layer["mixer"])).mixer
    mod = MixerGroup(spec, W, EPS).to(dtype)
    with torch.inference_mode():
        targets = mod.targets("")
        assert set(targets) == set(w)
        for n, t in targets.items():
            assert tuple(t.shape) == tuple(w[n].shape), n
            src = w[n] if not isinstance(t, torch.Tensor) else w[n].to(t.dtype)
            t.copy_(src)
    return mod.to(dev)


def rows(n, W, dtype, seed=1):
    """One sequence's inputs, in which some late rows are far ones, shifted
    by a column."""
    g = gen(seed)
    h = rnd(g, n, W, dtype=dtype)
    for i, j in ((n // 2, 1), (n - 1, 0), (n - 2, n - 3)):
        if 0 <= j < i:
            h[i] = (h[j].roll(1) + rnd(g, W, std=0.1)).to(dtype).double()
    return h


def caches_of(mod, blocks, bs, dtype, dev, slots=3):
    kv = KVCache.for_layers(mod.spec.cache_layers(), bs, blocks, dev, dtype,
                            state_slots=slots)
    for c in kv.caches:
        for t in c:
            t.uniform_(-3, 3)        # what an earlier sequence left behind
    return kv.caches


def run(mod, h, caches, meta, dtype, dev):
    with torch.inference_mode():
        return mod(torch.cat(h).to(dtype).to(dev), caches, meta,
                   RotaryTables(meta.positions))


LAYERS = {
    "attention": attn(6, 2, 24, 40),
    "attention one head": attn(1, 1, 8, 8, 0.5, 1),
    "attention odd": attn(5, 5, 13, 11, 0.4, 7),
    "attention many": attn(40, 2, 64, 64, 0.2, 33),   # two tiles of heads
    "attention wide": attn(4, 1, 128, 96),
    "attention large": attn(2, 1, 200, 256, 0.25, 60),
    "attention plain": attn(2, 2, 264, 264),
    "lightning": lightning(24, 20, 0.9, 0.5, 0.999),
    "lightning one head": lightning(4, 3, 0.95),
    "lightning odd": lightning(37, 51, 0.97, 0.01),
    "lightning 64": lightning(64, 96, 0.62, 0.99),
    "lightning 128": lightning(128, 128, 0.9, 0.98, 0.999, 1.0),
    "lightning large": lightning(200, 256, 0.99),
    "lightning forgets": lightning(32, 16, 0.0, 1e-6, 1.0),
    "mamba": mamba(96, 16, 4, 6),
    "mamba odd": mamba(77, 5, 3, 1),
    "mamba one": mamba(1, 1, 1, 1),
    "mamba states": mamba(72, 20, 4, 12),
    "mamba many states": mamba(40, 100, 2, 8),
    "mamba taps": mamba(130, 33, 9, 12),
    "mamba wide": mamba(1032, 8, 4, 40),
}
WIDTH = 40
_CASES = {}


def cached_case(name, n, dtype):
    key = (name, n, dtype)
    if key not in _CASES:
        layer = LAYERS[name]
        w = mixer_weights(layer, WIDTH)
        h = rows(n, WIDTH, dtype)
        want = oracle_mixer(layer, h, w)
        _CASES[key] = (layer, w, h, want, float(want.pow(2).mean().sqrt()))
    return _CASES[key]


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", list(LAYERS))
def test_mixer_prompts(dev, dtype, name):
    """Whole prompts, portions down to two tokens, on scattered pages."""
    layer, w, h, want, rms = cached_case(name, 150, dtype)
    mod = build_mixer(layer, w, WIDTH, dtype, dev)
    tables = np.random.RandomState(0).permutation(40).reshape(2, 20)
    for cuts in ([150], [2, 21, 2, 64, 61], [17, 128, 5]):
        caches, at = caches_of(mod, 40, 8, dtype, dev), 0
        for n in cuts:
            meta = prompt_meta([(at, at + n)], tables[1:], 8, dev, [2])
            y = run(mod, [h[at:at + n]], caches, meta, dtype, dev)
            close_rows(y, want[at:at + n], dtype, rms)
            at += n


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", list(LAYERS))
def test_mixer_batches_and_single_tokens(dev, dtype, name):
    """Two sequences of unequal length: prompts together, then single tokens,
    then a portion beside a single token."""
    layer, w, h, want, rms = cached_case(name, 150, dtype)
    hs, wants = [h, h[:90]], [want, want[:90]]
    mod = build_mixer(layer, w, WIDTH, dtype, dev)
    tables = np.random.RandomState(1).permutation(24).reshape(2, 12)
    slots = [2, 0]
    for first in ((0, 0), (33, 40), (100, 45)):
        caches = caches_of(mod, 24, 16, dtype, dev)
        if first[0]:
            y = run(mod, [x[:n] for x, n in zip(hs, first)], caches,
                    prompt_meta([(0, n) for n in first], tables, 16, dev,
                                slots), dtype, dev)
            close_rows(y, torch.cat([x[:n] for x, n in zip(wants, first)]),
                       dtype, rms)
        pos = list(first)
        for _ in range(20):
            y = run(mod, [x[p:p + 1] for x, p in zip(hs, pos)], caches,
                    decode_meta(pos, tables, 16, dev, slots), dtype, dev)
            close_rows(y, torch.stack([x[p] for x, p in zip(wants, pos)]),
                       dtype, rms)
            pos = [p + 1 for p in pos]
        d = decode_meta([pos[1]], tables[1:], 16, dev, slots[1:])
        p = prompt_meta([(pos[0], pos[0] + 25)], tables[:1], 16, dev,
                        slots[:1])
        meta = MixedMeta(
            decode=d, prefill=p, num_decode=1,
            slot_mapping=torch.cat([d.slot_mapping, p.slot_mapping]),
            positions=torch.cat([d.positions, p.positions]))
        y = run(mod, [hs[1][pos[1]:pos[1] + 1], hs[0][pos[0]:pos[0] + 25]],
                caches, meta, dtype, dev)
        close_rows(y, torch.cat([wants[1][pos[1]:pos[1] + 1],
                                 wants[0][pos[0]:pos[0] + 25]]), dtype, rms)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", ["attention", "attention odd",
                                  "attention wide", "attention many"])
def test_long_rows_in_partitions(dev, dtype, name):
    """A single token far into a sequence: its keys are cut into partitions
    on the GPU, and only a far one stands out."""
    n = 700
    layer, w, h, want, rms = cached_case(name, n, dtype)
    mod = build_mixer(layer, w, WIDTH, dtype, dev)
    tables = np.random.RandomState(2).permutation(88).reshape(2, 44)
    caches = caches_of(mod, 88, 16, dtype, dev)
    run(mod, [h[:n - 1]], caches, prompt_meta([(0, n - 1)], tables[:1], 16,
                                              dev, [1]), dtype, dev)
    y = run(mod, [h[n - 1:]], caches, decode_meta([n - 1], tables[:1], 16,
                                                  dev, [1]), dtype, dev)
    close_rows(y, want[n - 1:], dtype, rms)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("sizes,heads", [((24, 40), 4), ((13, 11), 2),
                                         ((64, 64), 8)])
def test_shared_keys_and_values(dev, dtype, sizes, heads):
    """A layer that reads another's cache, with other heads, scale and
    temperature; both see the same rows here."""
    own, other = attn(6 if heads == 4 else 2 * heads, 2, *sizes), \
        attn(heads, 2, *sizes, 0.7, 5, 1.3, kv_from=0)
    n = 100
    w, w2 = mixer_weights(own, WIDTH), mixer_weights(other, WIDTH, 4)
    h, h2 = rows(n, WIDTH, dtype), rows(n, WIDTH, dtype, 6)
    kv = do.keys_values(h, w, "", own["mixer"])
    want = oracle_mixer(other, h2, w2, kv)
    rms = float(want.pow(2).mean().sqrt())
    a, b = (build_mixer(l, x, WIDTH, dtype, dev)
            for l, x in ((own, w), (other, w2)))
    assert b.spec.cache_layers() == []
    caches = caches_of(a, 12, 16, dtype, dev)
    tables = np.random.RandomState(3).permutation(12)[None]
    at = 0
    for k in (30, 2, 1, 1, 40, 1, 25):
        meta = decode_meta([at], tables, 16, dev, [1]) if k == 1 else \
            prompt_meta([(at, at + k)], tables, 16, dev, [1])
        run(a, [h[at:at + k]], caches, meta, dtype, dev)
        y = run(b, [h2[at:at + k]], caches, meta, dtype, dev)
        close_rows(y, want[at:at + k], dtype, rms)
        at += k


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("name", ["attention", "lightning", "mamba"])
def test_rows_without_a_slot_leave_caches_alone(dev, name):
    layer, w, h, _, _ = cached_case(name, 150, BF16)
    mod = build_mixer(layer, w, WIDTH, BF16, dev)
    caches = caches_of(mod, 4, 16, BF16, dev)
    keep = [[t.clone() for t in c] for c in caches]
    meta = decode_meta([0, 5], np.zeros((2, 4), dtype=np.int64), 16, dev,
                       [-1, -1])
    meta.slot_mapping.fill_(-1)
    run(mod, [h[:2]], caches, meta, BF16, dev)
    for a, b in zip(caches, keep):
        for t, k in zip(a, b):
            assert torch.equal(t, k)


def test_mixer_cases_notice_mistakes():
    """Planted in the oracle: what the cases above would catch."""
    for name in ("attention", "lightning", "mamba"):
        layer, w, h, good, rms = cached_case(name, 150, F32)

        def off(w2=w, layer2=layer, h2=h, at=slice(None)):
            bad = oracle_mixer(layer2, h2, w2)
            return float((bad - good)[at].pow(2).mean(-1).sqrt().max()) / rms

        for n in w:
            if name == "lightning" and n in ("q", "k", "v"):
                continue             # the norm undoes most of their size
            assert off({**w, n: w[n] * 0.6}) > 0.06, n
        if name == "attention":      # one far key, seen from the last row
            gone = h.clone()
            gone[0] = 0
            assert off(h2=gone, at=slice(149, 150)) > 0.07
    for name, key, value in (
            ("attention", "scale", 0.3),
            ("attention", "q_temp", dict(coef=0.0, every=16)),
            ("attention", "q_temp", dict(coef=0.35, every=17)),
            ("lightning", "decay", [0.9, 0.5, 0.99])):
        layer, w, h, good, rms = cached_case(name, 150, F32)
        l2 = {**layer, "mixer": {**layer["mixer"], key: value}}
        bad = oracle_mixer(l2, h, w)
        assert float((bad - good).pow(2).mean(-1).sqrt().max()) / rms > 1e-3
    for name, start in (("lightning", 64), ("mamba", 64)):
        # with slow decays the first chunk still shows at the end
        layer, w, h, good, rms = cached_case(name, 150, F32)
        cut = oracle_mixer(layer, h[start:], w)
        assert float((cut[60:] - good[start + 60:]).abs().max()) / rms > 0.1


# --------------------------------------------------------------- temperature

@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("coef,every", [(0.45, 48), (1.5, 1), (0.1, 8192)])
def test_query_temperature(dev, coef, every):
    pos = torch.tensor([0, 1, every - 2 if every > 1 else 3, every - 1, every,
                        2 * every - 2 if every > 1 else 4, 2 * every - 1,
                        7 * every, (1 << 30) - 1])
    t = RotaryTables(pos.to(dev))
    got = t.temperature(QueryTemperature(coef, every))
    want = [do.query_temperature(int(p), coef, every) for p in pos]
    close(got, torch.tensor(want, dtype=torch.float64), F32)
    assert got is t.temperature(QueryTemperature(coef, every))
    assert t.temperature(None) is None


# ------------------------------------------------------------------ recurrences

@pytest.mark.gpu
@pytest.mark.parametrize("decay", [0.999, 0.7, 1.0])
def test_chunk_form_keeps_seventeen_bits(decay):
    """The state after a long bf16 prompt beside the recurrence in fp64 from
    the same bf16 inputs: chunking costs no precision."""
    layer = lightning(64, 64, decay, decay)
    w = mixer_weights(layer, WIDTH)
    mod = build_mixer(layer, w, WIDTH, BF16, "cuda")
    h = rows(500, WIDTH, BF16)
    caches = caches_of(mod, 1, 8, BF16, "cuda")
    run(mod, [h], caches, prompt_meta([(0, 500)], np.zeros((1, 63), int), 8,
                                      "cuda", [1]), BF16, "cuda")
    p = mod.cores[0].params
    with torch.inference_mode():
        z = mod.in_proj(h.to(BF16).cuda()).double().cpu()
    k, v = (do.silu(z[:, at:at + 128]).to(BF16).double().view(500, 2, 64)
            for at in (p.k_at, p.v_at))
    S = torch.zeros(2, 64, 64, dtype=torch.float64)
    a = float(np.float32(decay))
    for t in range(500):
        S = a * S + k[t][:, :, None] * v[t][:, None, :]
    got = caches[0][0][1].double().cpu()
    err = (got - S).abs().amax((0, 2)) / S.pow(2).mean().sqrt()
    # one bf16 step of some silu may fall the other way
    assert float(err.max()) < 5e-3 and float(err.median()) < 3e-4, err


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("inner,state", [(200, 16), (64, 100), (520, 5)])
def test_scan_in_chunks(dtype, inner, state):
    """Sequences cut into chunks beside the same whole, results and states;
    step sizes from tiny to large."""
    g, T = gen(inner), 700
    lens = [413, 1, 286]
    put = lambda t, dt=F32: t.to(dt).cuda().contiguous()  # noqa: E731
    w = routed.ScanWeights(
        None, None, None, None, put(rnd(g, inner, std=2.0) - 4.0),
        put(-torch.exp(rnd(g, state, inner)) * math.log2(math.e)),
        put(rnd(g, inner)))
    at = 8 + routed.state_columns(state)
    p = routed.ScanParams(inner, state, 4, 1, 0, 0, 8, at)
    x, z = (put(rnd(g, T, inner), dtype) for _ in range(2))
    dt, bc = put(rnd(g, T, inner, std=3.0)), put(rnd(g, T, p.columns))
    bc[:, 8 + state:at] = bc[:, at + state:] = 0
    cu = np.concatenate([[0], np.cumsum(lens)])
    meta = prompt_meta([(0, 413), (50, 51), (7, 293)],
                       np.zeros((3, 60), int), 8, "cuda", [2, 0, 1])
    start = torch.randn(3, state, inner, device="cuda")
    want, states = torch.zeros(T, inner, dtype=torch.float64), []
    A = w.A.double().cpu() * math.log(2)
    for b in range(3):
        s = slice(int(cu[b]), int(cu[b + 1]))
        d = do.softplus(dt[s].double().cpu() + w.dt_b.double().cpu())
        S = start[[2, 0, 1][b]].double().cpu() if b else \
            torch.zeros(state, inner, dtype=torch.float64)
        for t, (xt, dd, q) in enumerate(zip(x[s].double().cpu(), d,
                                            bc[s].double().cpu())):
            S = torch.exp(dd * A) * S + (dd * xt) * q[8:8 + state, None]
            want[int(cu[b]) + t] = (S * q[at:at + state, None]).sum(0) \
                + w.D.double().cpu() * xt
        states.append(S)
    want = want * do.silu(z.double().cpu())
    for size in (0, 64, 96, 512):
        state_t, y = start.clone(), torch.empty_like(x)
        real, routed.scan_chunk = routed.scan_chunk, lambda *a: size
        try:
            routed.scan_prompt(y, x, z, p, w, state_t, dt, bc, meta)
        finally:
            routed.scan_chunk = real
        close(y, want, dtype)
        for b, slot in enumerate([2, 0, 1]):
            close(state_t[slot], states[b], F32)


# ----------------------------------------------------------------------- model

def moe(ff, experts, top, identity=0, groups=1, keep=1):
    return {"kind": "moe", "expert": {"ff": ff}, "router": dict(
        experts=experts, top=top, identity=identity,
        groups=dict(count=groups, keep=keep))}


def with_ff(layer, mlp):
    return {**layer, "mlp": mlp}


def config(vocab, width, streams, cap, layers, places=640, eps=1e-5):
    return {"architecture": "Dibizen", "vocab": vocab, "width": width,
            "streams": streams, "logit_softcap": cap,
            "max_positions": places, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # layers of different shapes and order, one without a feed-forward, keys
    # and values read by two later layers
    "varied": config(97, 72, 3, 9.0, [
        with_ff(mamba(88, 6, 3, 5), moe(40, 6, 2, 2, 4, 2)),
        with_ff(attn(4, 2, 24, 40), moe(33, 5, 3)),
        with_ff(lightning(20, 28, 0.9, 0.5, 0.99), None),
        with_ff(attn(6, 2, 24, 40, 0.5, 9, 0.8, kv_from=1),
                moe(48, 3, 2, 3, 2, 1)),
        with_ff(attn(2, 2, 24, 40, 0.2, 30, kv_from=1), moe(24, 4, 4))]),
    # whole tiles everywhere
    "wide": config(300, 128, 4, 20.0, [
        with_ff(lightning(64, 64, 0.97, 0.8), moe(128, 6, 2, 2, 2, 1)),
        with_ff(attn(8, 2, 64, 64, 0.1, 40), moe(64, 8, 3)),
        with_ff(mamba(256, 16, 4, 8), moe(192, 4, 2))], eps=3e-6),
    # sizes of one
    "single": config(33, 20, 1, 3.0, [
        with_ff(attn(1, 1, 8, 8, 0.5, 1), moe(12, 1, 1)),
        with_ff(lightning(4, 6, 0.9), None),
        with_ff(mamba(5, 1, 1, 1), moe(8, 1, 1, 1))]),
    # attention only
    "flat": config(50, 48, 2, 12.0, [
        with_ff(attn(4, 2, 16, 16), moe(32, 4, 2)),
        with_ff(attn(4, 2, 16, 16, 0.4, 5, 1.1, kv_from=0),
                moe(24, 3, 2, 1, 2, 2))]),
}
CODE = 12            # columns that routing reads


def make_weights(cfg, seed=0):
    """bf16 tensors under their checkpoint names. Routers read a few columns
    that hold a sign per token, which nothing but identity experts writes to,
    so that rounding moves no choice (margin())."""
    g = gen(seed)
    W, S, out = cfg["width"], cfg["streams"], {}

    def add(name, *shape, std=None, mean=0.0):
        out[name] = bf16_exact(g, *shape, std=std, mean=mean).to(BF16)

    def norm(name):
        add(name, W, std=0.2, mean=1.0)
        add(name + ".b", W, std=0.2)
        out[name][:CODE], out[name + ".b"][:CODE] = 1.0, 0.0
        out[name + ".alpha"] = torch.tensor(0.8).to(BF16)

    def hyper(name):
        add(name + ".in", S, std=0.2, mean=1.0 / S)
        add(name + ".out", S, std=0.3, mean=1.0)
        add(name + ".mix", S, S, std=0.1)
        out[name + ".mix"] += torch.eye(S, dtype=BF16)
        for n in ("in", "out", "mix"):           # signs stay signs
            out[f"{name}.{n}"] = out[f"{name}.{n}"].abs()

    add("embed", cfg["vocab"], W, std=1.0)
    add("pos", cfg["max_positions"], W, std=0.5)
    add("head", cfg["vocab"], W, std=3.0 * W ** -0.5)
    out["pos"][:, :CODE] = 0
    norm("final.norm")
    for i, l in enumerate(cfg["layers"]):
        p = f"l{i}."
        for q in (1, 2) if l["mlp"] else (1,):
            norm(f"{p}norm{q}")
            hyper(f"{p}hc{q}")
        for k, v in mixer_weights(l, W, seed=seed + i).items():
            out[f"{p}mix.{k}"] = v.to(BF16)
        out[p + "mix.o"][:CODE] = 0
        if l["mlp"]:
            F, r = l["mlp"]["expert"]["ff"], l["mlp"]["router"]
            n = r["experts"] + r["identity"]
            add(p + "mlp.router", n, W, std=0.002)
            out[p + "mlp.router"][:, :CODE] = bf16_exact(
                g, n, CODE, std=0.6).to(BF16)
            add(p + "mlp.correction", n, std=0.02)
            for e in range(r["experts"]):
                add(f"{p}mlp.e{e}.up", F, W)
                add(f"{p}mlp.e{e}.down", W, F)
                out[f"{p}mlp.e{e}.down"][:CODE] = 0
    # signs for every token whose choices are clear in all layers
    w = {k: v.double() for k, v in out.items()}
    for t in range(cfg["vocab"]):
        for _ in range(400):
            code = torch.randint(0, 2, (CODE,), generator=g) * 8.0 - 4.0
            w["embed"][t, :CODE] = code
            if margin(cfg, w, t) > 0.02:
                break
        else:
            raise AssertionError("no clear choices")
        out["embed"][t, :CODE] = code.to(BF16)
    return out


def margin(cfg, w, token):
    """Least distance between what is chosen and what is not, over all
    layers, for a token on its own (the columns that count are the same at
    any place)."""
    worst = [1.0]
    choose = do.choose

    def watched(s, corr, r):
        picked = choose(s, corr, r)
        c, g = s + corr, r["groups"]
        size = len(c) // g["count"]
        best = sorted((float(c[k * size:(k + 1) * size].max())
                       for k in range(g["count"])), reverse=True)
        if g["keep"] < g["count"]:
            worst.append(best[g["keep"] - 1] - best[g["keep"]])
        # in the order of choice scores, the open ones alone
        more = choose(s, corr, {**r, "top": r["top"] + 1})
        if len(more) > r["top"]:
            worst.append(float(c[more[-2]] - c[more[-1]]))
        return picked

    do.choose = watched
    try:
        do.run(cfg, w, [token])
    finally:
        do.choose = choose
    return min(worst)


@pytest.fixture(scope="session")
def folders(tmp_path_factory):
    from safetensors.torch import save_file
    made = {}
    for name, cfg in CONFIGS.items():
        d = tmp_path_factory.mktemp("dibizen-" + name)
        (d / "config.json").write_text(json.dumps(cfg))
        w = make_weights(cfg)
        save_file(w, str(d / "model.safetensors"))
        made[name] = (str(d), cfg, {k: v.double() for k, v in w.items()})
    return made


_WANT = {}


def want_logits(name, cfg, w, ids):
    """Of the longest sequence asked for with this beginning."""
    for (n, seen), want in _WANT.items():
        if n == name and seen[:len(ids)] == tuple(ids):
            return want[:len(ids)]
    _WANT[name, tuple(ids)] = do.run(cfg, w, ids)[0]
    return _WANT[name, tuple(ids)]


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_portions_and_decode(folders, dev, dtype, name):
    folder, cfg, w = folders[name]
    eng = engine_for(folder, dev, dtype)
    ids = prompt(cfg, 139, 5)
    want = want_logits(name, cfg, w, ids)
    free = eng.num_free_blocks()
    for k, cut in enumerate(([139], [2], [3, 16, 2, 33], [64], [17, 1],
                             [100] + [1] * 39)):
        if dev == "cpu" and dtype == "bfloat16" and k in (1, 2, 4):
            continue
        got = run_cut(eng, f"s{k}", ids, cuts_of(139, cut))
        check_rows(got, want, dtype)
        eng.release(f"s{k}")
    assert eng.num_free_blocks() == free


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("name", ["varied", "wide"])
def test_token_by_token(folders, dev, name):
    folder, cfg, w = folders[name]
    eng = engine_for(folder, dev, "float32")
    ids = prompt(cfg, 139, 5)[:80]
    got = run_cut(eng, "a", ids, [1] * 80)
    check_rows(got, want_logits(name, cfg, w, ids), "float32")


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("name", ["varied", "wide", "single"])
def test_layers_one_by_one(folders, dev, name):
    folder, cfg, w = folders[name]
    eng = engine_for(folder, dev, "float32", enforce_eager=True)
    ids = prompt(cfg, 60, 7)
    _, want = do.run(cfg, w, ids)
    tap = eng.model.layer_tap = []
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
    cuts = {"a": [29, 1, 2, 1, 40, 1, 1], "b": [2, 1, 1, 7], "c": [1, 33, 2],
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
            k = len(got[s]) % len(cuts[s])
            n = min(cuts[s][k], lens[s] - at[s])
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
        ids.append(int(do.run(cfg, w, ids)[0][-1].argmax()))
    return ids[-n:]


_GREEDY = {}


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("mixed", [False, True])
@pytest.mark.parametrize("name", ["varied", "flat"])
def test_greedy_generation(folders, dev, mixed, name):
    """Through generate(): chunked prompts, a shared prefix (cached where
    there is no recurrent state), preemption."""
    folder, cfg, w = folders[name]
    prompts = [prompt(cfg, n, 40 + n) for n in (50, 3, 41)]
    prompts.append(prompts[0][:32] + prompt(cfg, 9, 3))     # shared prefix
    if name not in _GREEDY:
        _GREEDY[name] = [oracle_greedy(cfg, w, p, 8) for p in prompts]
    sp = SamplingParams(temperature=0.0, max_tokens=8, ignore_eos=True)
    for kw in (dict(max_prefill_tokens=4096), dict(max_prefill_tokens=24),
               dict(max_prefill_tokens=24, blocks=8)):
        eng = engine_for(folder, dev, "float32", mixed_steps=mixed, **kw)
        assert eng.prefix_caching == (name == "flat")
        eng.generate(prompts, sp)
        full = [eng.seqs[f"gen-1-{i}"] for i in range(4)]
        outs = [(s.prompt_ids + s.output_ids)[len(p):]
                for s, p in zip(full, prompts)]
        assert outs == _GREEDY[name], kw


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("name,dtype,n,cuts", [
    ("varied", "float32", 300, [5] + [1] * 295),
    ("varied", "bfloat16", 300, [5] + [1] * 295),
    ("wide", "bfloat16", 560, [2, 300, 198] + [1] * 60)])
def test_long_decode(folders, dev, name, dtype, n, cuts):
    """Hundreds of tokens, page by page."""
    folder, cfg, w = folders[name]
    ids = prompt(cfg, n, 8)
    eng = engine_for(folder, dev, dtype)
    got = run_cut(eng, "a", ids, cuts)
    check_rows(got, want_logits(name, cfg, w, ids), dtype)


def test_model_tests_notice_mistakes(folders):
    """Planted in the oracle: the tolerances above would catch each."""
    folder, cfg, w = folders["varied"]
    ids = prompt(cfg, 139, 5)[:60]
    good = want_logits("varied", cfg, w, ids)

    def off(c2, w2):
        bad, _ = do.run(c2, w2, ids)
        return float(((bad - good).pow(2).mean(-1).sqrt()
                      / good.std()).max())

    assert off({**cfg, "logit_softcap": 6.0}, w) > 0.08
    assert off(cfg, {**w, "pos": w["pos"].roll(1, 0)}) > 0.08
    # another layer's keys and values
    assert off({**cfg, "layers": cfg["layers"][:3] + [
        with_ff(attn(6, 2, 24, 40, 0.5, 90, 0.8, kv_from=1),
                cfg["layers"][3]["mlp"])] + cfg["layers"][4:]}, w) > \
        10 * MODEL_TOL["float32"]
    for n in w:
        if n == "embed" or ".e" in n or n.endswith("router") or \
                n == "l4.mlp.correction":
            continue         # some experts never chosen, layer 4 takes all
        if n.endswith("correction"):
            change = w[n] * 0 + torch.arange(len(w[n])) * 0.2
        elif n.endswith("mix"):
            change = w[n].T
        else:
            change = w[n] * 0.5
        assert off(cfg, {**w, n: change}) > 10 * MODEL_TOL["float32"], n


def test_choices_are_clear(folders):
    """What lets the bf16 tests stand: no token is near another choice."""
    for name, (_, cfg, w) in folders.items():
        assert min(margin(cfg, w, t) for t in range(0, cfg["vocab"], 3)) \
            > 0.02, name


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
    cfg = DibizenConfig.from_json(CONFIGS["varied"], "x")
    assert [l.ff.ff if l.ff else 0 for l in cfg.layers] == [40, 33, 0, 48, 24]
    assert cfg.layers[0].ff.router == RouterParams(6, 2, 2, 4, 2)
    assert cfg.layers[1].ff.router == RouterParams(5, 3)
    kinds = [isinstance(l, StateLayer) for l in cfg.kv_layers()]
    assert kinds == [True, False, True]
    assert cfg.cache_entries() == [0, 1, 2, 1, 1]
    assert (cfg.streams, cfg.logit_softcap, cfg.position_limit) == \
        (3, 9.0, 640)
    s = [l.mixer.members[0].spec for l in cfg.layers]
    assert s[0] == SelectiveSpec(88, 6, 3, 5)
    assert s[2] == LightningSpec(3, 20, 28, (0.9, 0.5, 0.99))
    assert s[3].shared_kv and s[3].q_temp == QueryTemperature(0.5, 9.0)
    plain = json.loads(json.dumps(CONFIGS["varied"]))
    del plain["layers"][1]["mixer"]["q_temp"]
    del plain["layers"][1]["mlp"]["router"]["groups"]
    del plain["layers"][1]["mlp"]["router"]["identity"]
    cfg = DibizenConfig.from_json(plain)
    assert cfg.layers[1].mixer.members[0].spec.q_temp is None
    assert cfg.layers[1].ff.router == RouterParams(5, 3)
    for path, value in ((("layers", 0, "type"), "other"),
                        (("layers", 0, "mlp", "kind"), "other"),
                        (("layers", 1, "mixer", "kv_heads"), 3),
                        (("layers", 3, "mixer", "vdim"), 24),
                        (("layers", 3, "mixer", "kv_from"), 0),
                        (("layers", 3, "mixer", "kv_from"), 4),
                        (("layers", 4, "mixer", "kv_from"), 3),
                        (("layers", 2, "mixer", "decay"), [0.5]),
                        (("layers", 0, "mlp", "router", "top"), 5),
                        (("layers", 0, "mlp", "router", "identity"), 1),
                        (("layers", 0, "mixer", "state"), 200),
                        (("layers", 1, "mixer", "q_temp", "every"), 0),
                        (("logit_softcap",), 0), (("streams",), 9)):
        bad = json.loads(json.dumps(CONFIGS["varied"]))
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ValueError):
            DibizenConfig.from_json(bad, "x")
    with pytest.raises(ValueError):
        DibizenForCausalLM(cfg, tp_size=2)


def test_small_tensors_keep_their_bits():
    m = DibizenForCausalLM(PRESETS["tiny-dibizen"]).to(BF16)
    light, scan = m.layers[0].mixer.cores[0], m.layers[2].mixer.cores[0]
    assert m.embed_tokens.weight.dtype == m.places.dtype == BF16
    assert m.layers[0].ff.ups.dtype == scan.x_w.dtype == BF16
    a = m.layers[0].around[1]
    for t in (a.into, a.out, a.mix, a.alpha, a.w, a.b, m.final.w,
              m.layers[0].ff.correction, light.norm_w, light.decay,
              light.log_decay, scan.conv_w, scan.A, scan.D, scan.dt_b):
        assert t.dtype == F32


def test_registry(tmp_path, folders):
    folder, cfg, w = folders["varied"]
    assert registry.get_config(folder).vocab_size == 97
    assert registry.get_config("tiny-dibizen") is PRESETS["tiny-dibizen"]
    assert registry.model_class(registry.get_config(folder)) \
        is DibizenForCausalLM
    from safetensors.torch import save_file
    saved = {k: v.to(BF16) for k, v in w.items()}
    for change in ("missing", "shape"):
        d = tmp_path / change
        d.mkdir()
        (d / "config.json").write_text(json.dumps(cfg))
        w2 = dict(saved)
        if change == "missing":
            del w2["l3.mlp.e2.down"]
        else:
            w2["l0.mix.A_log"] = w2["l0.mix.A_log"][:-1].contiguous()
        save_file(w2, str(d / "model.safetensors"))
        with pytest.raises(ValueError):
            registry.build_model(str(d), F32, torch.device("cpu"))


def test_several_extensions_are_built_at_once(monkeypatch):
    asked = []
    monkeypatch.setattr(build, "is_built", lambda n: n == "_C_gated")
    monkeypatch.setattr(build.subprocess, "run", lambda *a, env, **k:
                        asked.append(env["HELIX_BUILD_ONLY"]))
    build.ensure(DibizenForCausalLM.extension)
    build.ensure("_C_gated")
    assert asked == ["_C_routed"]


def test_caches_in_the_cache_manager(folders):
    folder, cfg, w = folders["varied"]
    eng = engine_for(folder, "cpu", "bfloat16", seqs=3)
    layers = eng.model_cfg.kv_layers()
    assert len(layers) == len(eng.kv.caches) == 3
    ring, state = eng.kv.caches[0]
    assert ring.shape == (3, 3, 88) and ring.dtype == BF16
    assert state.shape == (3, 6, 88) and state.dtype == F32
    k, v = eng.kv.caches[1]
    assert k.shape == (64, 2, 16, 24) and v.shape == (64, 2, 40, 16)
    want = sum(t.numel() * t.element_size()
               for l, c in zip(layers, eng.kv.caches)
               if isinstance(l, StateLayer) for t in c)
    assert KVCache.state_bytes(layers, 3, BF16) == want


def test_positions_bound_the_length(folders, tmp_path):
    """No sequence grows past the learned positions."""
    folder, cfg, w = folders["flat"]
    from safetensors.torch import save_file
    (tmp_path / "config.json").write_text(json.dumps(
        {**cfg, "max_positions": 40}))
    save_file({k: (v[:40] if k == "pos" else v).to(BF16).contiguous()
               for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    eng = engine_for(str(tmp_path), "cpu", "float32")
    assert eng.cfg.max_model_len == 40
    ids = prompt(cfg, 41, 3)
    got = run_cut(eng, "a", ids[:40], [38, 1, 1])
    check_rows(got, do.run(cfg, w, ids[:40])[0], "float32")
    with pytest.raises(ValueError):
        eng.extend([("a", ids[40:], [0])])
    out = eng.generate([ids[:36]], SamplingParams(
        temperature=0.0, max_tokens=20, ignore_eos=True))
    assert len(out[0]) == 4


def test_sizes_for_the_planner():
    cfg = registry.get_config("dibizen-3b")
    emb, rest = cfg.num_weights()
    with torch.device("meta"):
        n = sum(p.numel() for p in DibizenForCausalLM(cfg).parameters())
    assert 1.0 <= n / (emb + rest) < 1.01
    assert cfg.activation_bytes(10) > 0


@pytest.mark.parametrize("dev", DEVICES)
def test_random_preset_generates(dev):
    eng = engine_for("tiny-dibizen", dev, "bfloat16")
    out = eng.generate([[1, 2, 3] * 9, [5]], SamplingParams(
        temperature=0.0, max_tokens=5, ignore_eos=True))
    assert [len(o) for o in out] == [5, 5]
    out = eng.generate([[9, 8] * 5], SamplingParams(
        temperature=0.8, top_p=0.9, top_k=20, max_tokens=6, seed=3,
        ignore_eos=True))
    assert len(out[0]) == 6


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
