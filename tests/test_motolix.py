"""Motolix against its plain full-sequence oracle: every mechanism alone,
then the model through the engine (portions, decoding, mixed batches, reused
pages and state slots, greedy generation). Each test runs on the CPU
reference ops and, marked gpu, on the HIP kernels."""
import io
import json
import math

import numpy as np
import pytest
import torch

import motolix_oracle as mo
from helix_amd import ops
from helix_amd.engine import replay
from helix_amd.engine.kv_cache import KVCache
from helix_amd.engine.sampling_params import SamplingParams
from helix_amd.models import registry
from helix_amd.models.gla import GLASpec
from helix_amd.models.meta import MixedMeta, StateLayer
from helix_amd.models.mixer_group import GroupSpec, Member, MixerGroup
from helix_amd.models.motolix import (PRESETS, MotolixConfig,
                                      MotolixForCausalLM, parallel_mixer,
                                      sigmoid_mixer)
from helix_amd.models.rotary_attention import HalvesRotary, RotaryTables
from helix_amd.ops import gated
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


# ------------------------------------------------------------ stream and norms

@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,W", [(3, 64), (5, 250), (2, 1028), (600, 96),
                                 (1, 5120), (3, 77), (2, 1031), (520, 2048),
                                 (2, 12288)])
def test_stream(dev, dtype, T, W):
    g = gen(T + W)

    def put(t, dt=F32):
        return t.to(dt).to(dev)

    # a mean far from zero: the variance is that of the deviations
    x, y = rnd(g, T, W), rnd(g, T, W, dtype=dtype) + 16.0
    y = y.to(dtype).double()
    w1, b1, w2, b2, step = (rnd(g, W) for _ in range(5))
    post, norm = gated.Norm(put(w1), put(b1)), gated.Norm(put(w2), put(b2))
    v = x + mo.layer_norm(y, w1, b1, EPS)
    xd = put(x)
    tap = torch.empty_like(xd)
    h = gated.stream_add(xd, put(y, dtype), post, norm, EPS, tap=tap)
    close(xd, v, F32)
    close(tap, v, F32)
    close(h, mo.layer_norm(v, w2, b2, EPS), dtype)
    # into a pass of the loop: two terms carry what one would lose
    xd = put(x)
    terms = gated.split_terms(xd, dtype)
    assert gated.stream_add(xd, put(y, dtype), post, None, EPS, terms) is None
    if dtype == F32:
        assert terms is None
    else:
        back = terms[0].double() + terms[1].double()
        assert float(((back.cpu() - v).abs() / (1 + v.abs())).max()) < 1e-5
    emb = rnd(g, 11, W, dtype=dtype)
    ids = torch.randint(0, 11, (T,), generator=g)
    if W <= 2048:
        wx, we = (rnd(g, W, W, dtype=dtype, std=W ** -0.5) for _ in range(2))
        e = gated.project32(put(emb, dtype)[ids.to(dev)], put(we, dtype))
        h = gated.stream_enter(xd, terms, put(wx, dtype), e, 3.7, put(step),
                               norm, EPS, dtype)
        v = v @ wx.T + 3.7 * emb[ids] @ we.T + step
        close(xd, v, F32)
        close(h, mo.layer_norm(v, w2, b2, EPS), dtype)
    h = gated.stream_embed(xd, ids.to(dev), put(emb, dtype), 3.7, norm, EPS)
    close(xd, 3.7 * emb[ids], F32)
    close(h, mo.layer_norm(3.7 * emb[ids], w2, b2, EPS), dtype)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,F", [(3, 64), (7, 50), (300, 1032)])
def test_gated_mul(dev, dtype, T, F):
    g = gen(F)
    up = -(-F // 8) * 8
    z = rnd(g, T, up + F, dtype=dtype, std=3.0)
    zd = z.to(dtype).to(dev)
    for act, fn in (("gelu_tanh", mo.gelu), ("silu", mo.silu)):
        close(gated.gated_mul(zd, up, F, act),
              fn(z[:, :F]) * z[:, up:up + F], dtype)
    with pytest.raises(ValueError):
        gated.gated_mul(zd, up, F, "other")


# -------------------------------------------------------------------- rotation

SCALINGS = [None, dict(factor=6.0, original=300, low=1.0, high=4.0),
            dict(factor=2.5, original=40, low=0.5, high=9.0),
            dict(factor=8.0, original=4096, low=2.0, high=2.5)]


@pytest.mark.parametrize("scaling", SCALINGS)
@pytest.mark.parametrize("dims,base", [(12, 1e4), (64, 5e5), (2, 100.0),
                                       (6, 2e6)])
def test_banded_frequencies(dims, base, scaling):
    got = ops.banded_frequencies(dims, base, scaling)
    want = mo.frequencies(dims, base, scaling)
    assert torch.allclose(got, torch.tensor(want, dtype=torch.float64),
                          rtol=1e-12, atol=0)


@pytest.mark.parametrize("dev", DEVICES)
def test_rotary_table(dev):
    f = ops.banded_frequencies(10, 1e3, SCALINGS[2])
    pos = torch.tensor([0, 1, 17, 4095, 1 << 20])
    cs = gated.rotary_table(pos.to(dev), f.to(dev)).double().cpu()
    a = pos.double()[:, None] * f
    assert float((cs[..., 0] - torch.cos(a)).abs().max()) < 1e-6
    assert float((cs[..., 1] - torch.sin(a)).abs().max()) < 1e-6
    tables = RotaryTables(pos.to(dev))
    rot = HalvesRotary(10, 1e3)
    assert tables.get(rot, f.to(dev)) is tables.get(HalvesRotary(10, 1e3), None)
    assert tables.get(None, None) is None


# ------------------------------------------------------------- mixers as a whole

def attn(heads, kv_heads, dim, vdim, dims, scale=None, base=1e4, scaling=None):
    out = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim,
               scale=scale or 4.0 / math.sqrt(dim))
    if dims:
        out["rot"] = dict(dims=dims, base=base)
        if scaling:
            out["rot"]["scaling"] = scaling
    return out


def sizes(m):
    return dict(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
                vdim=m["vdim"], scale=m["scale"],
                rotary=HalvesRotary.from_json(m.get("rot")))


def mixer_weights(layer, W, seed=0, rank=5):
    """bf16-exact weights; the keys' projection repeats that of the group's
    first query head, so a row meets its copies with a score that stands
    out."""
    g, m, out = gen(seed), layer["mixer"], {}

    def add(name, *shape, std=None, mean=0.0):
        std = std if std is not None else shape[-1] ** -0.5
        out[name] = (torch.randn(shape, generator=g) * std
                     + mean).to(BF16).double()

    def qk(p, a):
        H, G, D = a["heads"], a["kv_heads"], a["dim"]
        add(p + "q", H * D, W)
        out[p + "k"] = out[p + "q"].view(G, H // G, D, W)[:, 0].reshape(
            G * D, W).clone()

    if layer["type"] == "attention":
        H, G, D = m["heads"], m["kv_heads"], m["dim"]
        qk("", m)
        add("q.b", H * D, std=0.3)
        add("k.b", G * D, std=0.3)
        add("temp", H, std=0.2, mean=1.0)
        add("pb", H, std=1.0, mean=-4.0)
        add("o", W, H * D)
        add("o.b", W, std=0.5)
        return out
    a, r = m["left"], m["right"]
    qk("left.", a)
    add("left.v", a["kv_heads"] * a["vdim"], W)
    add("left.q.norm", a["heads"] * a["dim"], std=0.2, mean=1.0)
    add("left.k.norm", a["kv_heads"] * a["dim"], std=0.2, mean=1.0)
    add("left.o", W, a["heads"] * a["vdim"])
    K, V = r["heads"] * r["dim"], r["heads"] * r["vdim"]
    for n, rows in (("q", K), ("k", K), ("v", V), ("g", V), ("a1", rank)):
        add("right." + n, rows, W)
    # decays from almost none to several bits a token
    add("right.a2", K, rank, std=1.5)
    add("right.a2.b", K, std=2.0, mean=3.0 * math.log(r["tau"] + 1))
    add("right.norm", r["vdim"], std=0.2, mean=1.0)
    add("right.o", W, V)
    return out


def spec_of(layer, rank=5):
    m = layer["mixer"]
    if layer["type"] == "attention":
        return sigmoid_mixer(**sizes(m))
    return parallel_mixer(sizes(m["left"]), m["left_scale"],
                          GLASpec.from_json(m["right"], rank),
                          m["right_scale"])


def build(layer, w, W, dtype, dev, rank=5):
    mod = MixerGroup(spec_of(layer, rank), W, EPS)
    mod = mod.to(dtype)
    with torch.inference_mode():
        targets = mod.targets("")
        assert set(targets) == set(w)
        for n, t in targets.items():
            assert tuple(t.shape) == tuple(w[n].shape), n
            t.copy_(w[n].to(t.dtype))
    return mod.to(dev)


def rows(n, W, dtype, seed=1):
    """One sequence's inputs, in which some late rows repeat far ones."""
    g = gen(seed)
    h = rnd(g, n, W, dtype=dtype)
    for i, j in ((n // 2, 1), (n - 1, 0), (n - 2, n - 3)):
        if 0 <= j < i:
            h[i] = (h[j] + rnd(g, W, std=0.1)).to(dtype).double()
    return h


def caches_of(mod, blocks, bs, dtype, dev, slots=3):
    kv = KVCache.for_layers(mod.spec.cache_layers(), bs, blocks, dev, dtype,
                            state_slots=slots)
    for pair in kv.caches:
        for t in pair:
            t.uniform_(-3, 3)        # what an earlier sequence left behind
    return kv.caches


def run(mod, h, caches, meta, dtype, dev):
    with torch.inference_mode():
        return mod(torch.cat(h).to(dtype).to(dev), caches, meta,
                   RotaryTables(meta.positions))


def parallel(left, right, ls=0.9, rs=0.6):
    return {"type": "parallel", "mixer": dict(
        left=left, right=right, left_scale=ls, right_scale=rs)}


def gla(heads, dim, vdim, tau):
    return dict(heads=heads, dim=dim, vdim=vdim, tau=tau)


SCALING = dict(factor=3.0, original=64, low=0.5, high=8.0)
LAYERS = {
    "sigmoid": {"type": "attention", "mixer": attn(
        6, 2, 24, 24, 16, scaling=SCALING)},
    "sigmoid one head": {"type": "attention", "mixer": attn(1, 1, 8, 8, 2)},
    "sigmoid odd": {"type": "attention", "mixer": attn(5, 5, 13, 13, 6)},
    "sigmoid many": {"type": "attention", "mixer": attn(
        40, 2, 64, 64, 64, scaling=SCALING)},     # two tiles of heads
    "sigmoid wide": {"type": "attention", "mixer": attn(4, 1, 128, 128, 32)},
    "sigmoid large": {"type": "attention", "mixer": attn(2, 1, 200, 200, 50)},
    "sigmoid plain": {"type": "attention", "mixer": attn(2, 2, 264, 264, 8)},
    "sigmoid unrotated": {"type": "attention", "mixer": attn(3, 1, 16, 16, 0)},
    "parallel": parallel(attn(4, 2, 24, 40, 4, 0.6, 1e8),
                         gla(3, 24, 20, 4.0)),
    "parallel small": parallel(attn(1, 1, 6, 2, 2), gla(1, 1, 1, 1.0), 1., 1.),
    "parallel odd": parallel(attn(3, 1, 10, 14, 10), gla(2, 37, 51, 2.0)),
    "parallel 64": parallel(attn(8, 2, 64, 64, 64, scaling=SCALING),
                            gla(2, 64, 96, 16.0)),
    "parallel 128": parallel(attn(4, 4, 128, 96, 40), gla(2, 128, 128, 16.0)),
    "parallel large": parallel(attn(2, 1, 160, 256, 96), gla(1, 200, 256, 8.)),
    "parallel unrotated": parallel(attn(2, 1, 12, 9, 0), gla(2, 16, 8, 3.0)),
}
WIDTH = 40


def case(name, n, dtype, rank=5):
    layer = LAYERS[name]
    w = mixer_weights(layer, WIDTH, rank=rank)
    h = rows(n, WIDTH, dtype)
    want = mo.mixer(h, w, "", layer, EPS)
    return layer, w, h, want, float(want.pow(2).mean().sqrt())


_CASES = {}


def cached_case(name, n, dtype):
    key = (name, n, dtype)
    if key not in _CASES:
        _CASES[key] = case(*key)
    return _CASES[key]


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", list(LAYERS))
def test_mixer_prompts(dev, dtype, name):
    """Whole prompts, portions down to two tokens, on scattered pages."""
    layer, w, h, want, rms = cached_case(name, 150, dtype)
    mod = build(layer, w, WIDTH, dtype, dev)
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
    mod = build(layer, w, WIDTH, dtype, dev)
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
@pytest.mark.parametrize("name", ["sigmoid", "sigmoid odd", "sigmoid wide",
                                  "parallel odd", "parallel 64"])
def test_long_rows_in_partitions(dev, dtype, name):
    """A single token far into a sequence: its keys are cut into partitions
    on the GPU, and only a far one stands out."""
    n = 700
    layer, w, h, want, rms = cached_case(name, n, dtype)
    mod = build(layer, w, WIDTH, dtype, dev)
    tables = np.random.RandomState(2).permutation(88).reshape(2, 44)
    caches = caches_of(mod, 88, 16, dtype, dev)
    run(mod, [h[:n - 1]], caches, prompt_meta([(0, n - 1)], tables[:1], 16,
                                              dev, [1]), dtype, dev)
    y = run(mod, [h[n - 1:]], caches, decode_meta([n - 1], tables[:1], 16,
                                                  dev, [1]), dtype, dev)
    close_rows(y, want[n - 1:], dtype, rms)


@pytest.mark.parametrize("dev", DEVICES)
def test_rows_without_a_slot_leave_caches_alone(dev):
    layer, w, h, _, _ = cached_case("parallel", 150, BF16)
    mod = build(layer, w, WIDTH, BF16, dev)
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
    for name in ("sigmoid", "parallel"):
        layer, w, h, good, rms = cached_case(name, 150, F32)

        def off(w2=w, layer2=layer, h2=h, at=slice(None)):
            bad = mo.mixer(h2, w2, "", layer2, EPS)
            return float((bad - good)[at].pow(2).mean(-1).sqrt().max()) / rms

        for n in w:              # norms undo the size of some projections
            if n not in ("left.q", "left.k", "right.q", "right.k", "right.v"):
                assert off({**w, n: w[n] * 0.6}) > 0.01, n
        # one far key that is missing, seen from the last row alone
        gone = h.clone()
        gone[0] = 0
        assert off(h2=gone, at=slice(149, 150)) > 0.07
        changes = {"sigmoid": [("scale", 0.3), ("rot", None)],
                   "parallel": [("left_scale", 0.5), ("right_scale", 0.3)]}
        for key, value in changes[name]:
            l2 = json.loads(json.dumps(layer))
            l2["mixer"][key] = value
            assert off(layer2=l2) > 0.01, key
    l2 = json.loads(json.dumps(LAYERS["parallel"]))
    l2["mixer"]["right"]["tau"] = 1.0
    assert off(layer2=l2) > 0.01
    l2["mixer"]["right"]["tau"] = 4.0
    l2["mixer"]["left"]["rot"]["base"] = 50.0
    assert off(layer2=l2) > 0.01


# ------------------------------------------------------ gated linear attention

def gla_alone(heads, dim, vdim, tau, n, bias, dtype, dev, rank=5, std=1.5):
    """A group of one recurrent mixer -> (module, weights, mixer
    configuration, inputs, expected). Queries are keys: where little of the
    state is left, q.k should not vanish by chance."""
    layer = parallel(attn(1, 1, 8, 8, 8), gla(heads, dim, vdim, tau))
    w = mixer_weights(layer, WIDTH, seed=3, rank=rank)
    w = {k[6:]: v for k, v in w.items() if k.startswith("right.")}
    g, w["q"] = gen(4), w["k"]
    w["a2.b"] = (bias + rnd(g, heads * dim, std=std)).to(BF16).double()
    spec = GroupSpec((Member(GLASpec(heads, dim, vdim, tau, rank), "", 1.0),))
    mod = MixerGroup(spec, WIDTH, EPS).to(dtype)
    with torch.inference_mode():
        for k, t in mod.targets("").items():
            t.copy_(w[k].to(t.dtype))
    h = rows(n, WIDTH, dtype, seed=9)
    m = gla(heads, dim, vdim, tau)
    return mod.to(dev), w, m, h, mo.linear_attention(h, w, "", m, EPS)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("heads,dim,vdim,tau,bias,rank", [
    (2, 32, 32, 16.0, 6.0, 16),     # hardly any decay: far tokens count
    (2, 48, 24, 1.0, -7.0, 5),      # ten bits a token: steep within a block
    (1, 64, 40, 1.0, -40.0, 1),     # nothing survives a token
    (3, 20, 72, 2.0, 0.0, 40),
])
def test_decays(dev, dtype, heads, dim, vdim, tau, bias, rank):
    mod, w, m, h, want = gla_alone(heads, dim, vdim, tau, 200, bias, dtype,
                                   dev, rank)
    rms = float(want.pow(2).mean().sqrt())
    tables = np.zeros((1, 30), dtype=np.int64)
    for cuts in ([200], [64, 64, 72], [30, 170], [5, 2, 193]):
        caches, at = caches_of(mod, 1, 8, dtype, dev), 0
        for n in cuts:
            y = run(mod, [h[at:at + n]], caches, prompt_meta(
                [(at, at + n)], tables, 8, dev, [1]), dtype, dev)
            close_rows(y, want[at:at + n], dtype, rms)
            at += n


@pytest.mark.gpu
@pytest.mark.parametrize("bias,tau,std", [(8.0, 16.0, 0.5), (2.0, 4.0, 2.0),
                                          (-3.0, 1.0, 4.0)])
def test_chunk_form_keeps_seventeen_bits(bias, tau, std):
    """The state after a long bf16 prompt beside the recurrence in fp64 from
    the same bf16 inputs: chunking costs no precision."""
    mod, w, m, h, _ = gla_alone(2, 64, 64, tau, 500, bias, BF16, "cuda",
                                std=std)
    p = mod.cores[0].params
    caches = caches_of(mod, 1, 8, BF16, "cuda")
    hd = h.to(BF16).cuda()
    run(mod, [h], caches, prompt_meta([(0, 500)], np.zeros((1, 63), int), 8,
                                      "cuda", [1]), BF16, "cuda")
    with torch.inference_mode():
        z = mod.in_proj(hd).double().cpu()
    x = z[:, p.a_at:p.a_at + 5] @ w["a2"].T + w["a2.b"]
    a = mo.decays(x.view(500, 2, 64), tau)
    S = torch.zeros(2, 64, 64, dtype=torch.float64)
    k, v = (z[:, at:at + 128].reshape(500, 2, 64) for at in (p.k_at, p.v_at))
    for t in range(500):
        S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
    got = caches[0][0][1].double().cpu()
    err = (got - S).abs().amax((0, 2)) / S.pow(2).mean().sqrt()
    assert float(err.max()) < 2e-4, err


def test_state_carries_far():
    """With slow decays a token from the first chunk still shows at the end:
    the cases above see a state that is lost between chunks."""
    _, w, m, h, good = gla_alone(2, 32, 32, 16.0, 200, 6.0, F32, "cpu", 16)
    cut = mo.linear_attention(h[64:], w, "", m, EPS)
    ref = float(good.pow(2).mean().sqrt())
    assert float((cut[60:] - good[124:]).abs().max()) / ref > 0.2


# ----------------------------------------------------------------------- model

def with_ff(layer, ff):
    return {**layer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


CONFIGS = {
    # layers of different shapes, one without a feed-forward, a loop in the
    # middle that begins with a sigmoid layer
    "varied": {"architecture": "Motolix", "vocab": 97, "width": 72,
               "norm": {"eps": 1e-5}, "embedding": {"scale": 5.5},
               "logit_scale": 0.7,
               "loop": {"start": 1, "stop": 3, "times": 2}, "layers": [
                   with_ff(parallel(attn(4, 2, 24, 40, 16),
                                    gla(3, 24, 20, 4.0)), 96),
                   with_ff({"type": "attention", "mixer": attn(
                       6, 2, 20, 20, 12, scaling=SCALING)}, 0),
                   with_ff(parallel(attn(3, 1, 10, 14, 10),
                                    gla(2, 37, 51, 2.0), 0.4, 1.1), 130),
                   with_ff({"type": "attention",
                            "mixer": attn(3, 3, 16, 16, 16, base=50.)}, 52)]},
    # the loop from the first layer to the last
    "wide": {"architecture": "Motolix", "vocab": 300, "width": 128,
             "norm": {"eps": 3e-6}, "embedding": {"scale": 11.0},
             "logit_scale": 1.0,
             "loop": {"start": 0, "stop": 2, "times": 3}, "layers": [
                 with_ff(parallel(attn(8, 2, 64, 64, 64, scaling=SCALING),
                                  gla(2, 64, 64, 16.0)), 264),
                 with_ff({"type": "attention",
                          "mixer": attn(20, 1, 64, 64, 32)}, 264)]},
    # sizes of one, a loop of one pass over one layer
    "single": {"architecture": "Motolix", "vocab": 33, "width": 20,
               "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
               "logit_scale": 0.1,
               "loop": {"start": 1, "stop": 2, "times": 1}, "layers": [
                   with_ff({"type": "attention",
                            "mixer": attn(1, 1, 8, 8, 2)}, 28),
                   with_ff(parallel(attn(1, 1, 6, 2, 2), gla(1, 9, 1, 1.0),
                                    1.0, 1.0), 0)]},
    # attention only, no loop
    "flat": {"architecture": "Motolix", "vocab": 50, "width": 48,
             "norm": {"eps": 1e-5}, "embedding": {"scale": 2.0},
             "logit_scale": 2.0, "loop": None, "layers": [
                 with_ff({"type": "attention",
                          "mixer": attn(4, 2, 16, 16, 8)}, 64),
                 with_ff({"type": "attention",
                          "mixer": attn(2, 1, 32, 32, 32)}, 40)]},
}


def make_weights(cfg, seed=0):
    """bf16 tensors under their checkpoint names."""
    g = gen(seed)
    W, out = cfg["width"], {}

    def add(name, *shape, std=None, mean=0.0):
        std = std if std is not None else 1.0 / math.sqrt(shape[-1])
        out[name] = (torch.randn(shape, generator=g) * std + mean).to(BF16)

    def norm(name):
        add(name, W, std=0.2, mean=1.0)
        add(name + ".b", W, std=0.2)

    add("embed", cfg["vocab"], W, std=0.5)
    add("head", cfg["vocab"], W)
    norm("final.norm")
    if cfg["loop"]:
        add("loop.in", W, 2 * W)
        add("loop.step", cfg["loop"]["times"], W, std=0.5)
    for i, l in enumerate(cfg["layers"]):
        p = f"l{i}."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if l["mlp"]
                                        else ()):
            norm(p + n)
        for k, v in mixer_weights(l, W, seed=seed + i, rank=5 + i).items():
            out[f"{p}mix.{k}"] = v.to(BF16)
        if l["mlp"]:
            F = l["mlp"]["ff"]
            add(p + "mlp.gate", F, W)
            add(p + "mlp.up", F, W)
            add(p + "mlp.down", W, F)
    return out


@pytest.fixture(scope="session")
def folders(tmp_path_factory):
    from safetensors.torch import save_file
    made = {}
    for name, cfg in CONFIGS.items():
        d = tmp_path_factory.mktemp("motolix-" + name)
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
    _WANT[name, tuple(ids)] = mo.run(cfg, w, ids)[0]
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
    _, want = mo.run(cfg, w, ids)
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
        ids.append(int(mo.run(cfg, w, ids)[0][-1].argmax()))
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
        bad, _ = mo.run(c2, w2, ids)
        return float(((bad - good).pow(2).mean(-1).sqrt()
                      / good.std()).max())

    for key, value in (("embedding", {"scale": 4.0}), ("logit_scale", 0.6),
                       ("loop", {"start": 1, "stop": 3, "times": 1})):
        assert off({**cfg, key: value}, w) > 0.08, key
    swapped = {**w, "loop.step": w["loop.step"].flip(0)}
    assert off(cfg, swapped) > 0.08
    turned = {**w, "loop.in": w["loop.in"].roll(72, 1)}
    assert off(cfg, turned) > 0.08
    for n in w:
        if n.split(".")[-1] in ("b", "norm", "norm1", "norm1b", "norm2",
                                "norm2b", "temp", "pb", "a1", "a2"):
            assert off(cfg, {**w, n: w[n] * 0.5}) > \
                10 * MODEL_TOL["float32"], n


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

def shapes_of(w):
    return {k: tuple(v.shape) for k, v in w.items()}


def test_config_reader():
    shapes = shapes_of(make_weights(CONFIGS["varied"]))
    cfg = MotolixConfig.from_json(CONFIGS["varied"], "x", shapes)
    assert [l.ff for l in cfg.layers] == [96, 0, 130, 52]
    assert [r.layer for r in cfg.runs()] == [0, 1, 2, 1, 2, 3]
    assert [r.loop_pass for r in cfg.runs()] == [-1, 0, -1, 1, -1, -1]
    kinds = [isinstance(l, StateLayer) for l in cfg.kv_layers()]
    assert kinds == [False, True, False, False, True, False, False, True,
                     False]
    assert cfg.kv_layers()[0].k_dim == 24 and cfg.kv_layers()[0].v_dim == 40
    assert [m.spec.rank for l in cfg.layers for m in l.mixer.members
            if isinstance(m.spec, GLASpec)] == [5, 7]
    assert cfg.layers[1].mixer.members[0].spec.rotary.scaling == \
        (3.0, 0.5, 8.0, 64.0)
    assert (cfg.embedding_scale, cfg.logit_scale) == (5.5, 0.7)
    assert len(MotolixConfig.from_json(CONFIGS["flat"]).runs()) == 2
    for path, value in ((("layers", 0, "type"), "other"),
                        (("layers", 0, "mlp", "kind"), "other"),
                        (("layers", 1, "mixer", "kv_heads"), 4),
                        (("layers", 1, "mixer", "vdim"), 24),
                        (("layers", 1, "mixer", "rot", "dims"), 7),
                        (("layers", 1, "mixer", "rot", "dims"), 40),
                        (("layers", 0, "mixer", "left", "vdim"), 13),
                        (("loop", "stop"), 9)):
        bad = json.loads(json.dumps(CONFIGS["varied"]))
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ValueError):
            MotolixConfig.from_json(bad, "x", shapes)
    with pytest.raises(ValueError):          # sizes that only tensors have
        MotolixConfig.from_json(CONFIGS["varied"])
    with pytest.raises(ValueError):
        MotolixForCausalLM(cfg, tp_size=2)
    with pytest.raises(ValueError):
        m = sigmoid_mixer(**sizes(attn(1, 1, 8, 8, 2))).members
        GroupSpec(m + m)


def test_small_tensors_keep_their_bits():
    m = MotolixForCausalLM(PRESETS["tiny-motolix"]).to(BF16)
    left, right = m.layers[0].mixer.cores
    sig = m.layers[1].mixer.cores[0]
    assert m.embed_tokens.weight.dtype == m.loop_x.dtype == BF16
    for t in (m.layers[0].norm1_w, m.layers[0].norm2b_b, left.q_norm,
              left.k_norm, right.a2_b, right.norm_w, sig.temp, sig.head_bias,
              m.final_w, m.final_b, m.loop_step):
        assert t.dtype == F32
    assert left.freqs.dtype == left.value_freqs.dtype == torch.float64


def test_registry(tmp_path, folders):
    folder, cfg, w = folders["varied"]
    assert registry.get_config(folder).vocab_size == 97
    assert registry.get_config("tiny-motolix") is PRESETS["tiny-motolix"]
    assert registry.model_class(registry.get_config(folder)) \
        is MotolixForCausalLM
    from safetensors.torch import save_file
    for change in ("missing", "shape"):
        d = tmp_path / change
        d.mkdir()
        (d / "config.json").write_text(json.dumps(cfg))
        w2 = make_weights(cfg)
        if change == "missing":
            del w2["l1.mix.pb"]
        else:
            w2["l0.mix.left.q"] = w2["l0.mix.left.q"][:-1].contiguous()
        save_file(w2, str(d / "model.safetensors"))
        with pytest.raises(ValueError):
            registry.build_model(str(d), F32, torch.device("cpu"))


def test_caches_in_the_cache_manager(folders):
    folder, cfg, w = folders["varied"]
    eng = engine_for(folder, "cpu", "bfloat16", seqs=3)
    layers = eng.model_cfg.kv_layers()
    assert len(layers) == len(eng.kv.caches) == 9
    for l, c in zip(layers, eng.kv.caches):
        if isinstance(l, StateLayer):
            (state,) = c
            assert state.shape[0] == 3 and state.dtype == F32
        else:
            assert c[0].shape[0] == 64 and c[1].shape[2:] == (l.v_dim, 16)
    want = sum(t.numel() * 4 for l, c in zip(layers, eng.kv.caches)
               if isinstance(l, StateLayer) for t in c)
    assert KVCache.state_bytes(layers, 3, BF16) == want


def test_sizes_for_the_planner():
    cfg = registry.get_config("motolix-1b")
    emb, rest = cfg.num_weights()
    with torch.device("meta"):
        n = sum(p.numel() for p in MotolixForCausalLM(cfg).parameters())
    assert 1.0 <= n / (emb + rest) < 1.01
    assert cfg.activation_bytes(10) > 0


@pytest.mark.parametrize("dev", DEVICES)
def test_random_preset_generates(dev):
    eng = engine_for("tiny-motolix", dev, "bfloat16")
    out = eng.generate([[1, 2, 3] * 9, [5]], SamplingParams(
        temperature=0.0, max_tokens=5, ignore_eos=True))
    assert [len(o) for o in out] == [5, 5]


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
