"""Zederax against its plain full-sequence oracle: every mechanism alone,
then the model through the engine (portions, decoding, mixed batches, page
reuse, greedy generation). Each test runs on the CPU reference ops and,
marked gpu, on the HIP kernels."""
import io
import json
import math

import pytest
import torch

import zederax_oracle as zo
from helix_amd import ops
from helix_amd.engine import replay
from helix_amd.engine.engine import EngineConfig, LLMEngine
from helix_amd.engine.kv_cache import KVCache
from helix_amd.engine.sampling_params import SamplingParams
from helix_amd.models import registry
from helix_amd.models.zederax import (PRESETS, ZederaxConfig,
                                      ZederaxForCausalLM)

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F32, BF16 = torch.float32, torch.bfloat16
EPS = 1e-5


def tol(dtype):
    return 2e-5 if dtype == F32 else 2e-2


def close(got, want, dtype, scale=None):
    """Largest deviation, relative to the element plus the rms of all."""
    got, want = got.double().cpu(), want.double().cpu()
    ref = scale or max(float(want.pow(2).mean().sqrt()), 1e-6)
    err = float(((got - want).abs() / (ref + want.abs())).max())
    assert err < tol(dtype), err


def rnd(g, *shape, dtype=F32, std=1.0):
    """Values exactly representable in dtype, as float64."""
    return (torch.randn(*shape, generator=g) * std).to(dtype).double()


# ---------------------------------------------------------------- mechanisms

@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,W,n", [(3, 64, 1), (5, 250, 2), (2, 1028, 4),
                                   (600, 96, 3), (1, 5120, 3), (3, 77, 1),
                                   (520, 2048, 2)])
def test_depth_norm(dev, dtype, T, W, n):
    g = torch.Generator().manual_seed(T + W)
    hist = [rnd(g, T, W) for _ in range(n)]
    x, y = rnd(g, T, W), rnd(g, T, W, dtype=dtype)
    coef, w = rnd(g, n + 1), rnd(g, W)
    want_x = zo.depth_average(hist + [x + y], coef)
    store = torch.zeros(n + 1, T, W, device=dev)
    store[:n] = torch.stack(hist).float()
    xs = x.float().to(dev)
    h = ops.depth_norm(xs, y.to(dtype).to(dev), store, n, coef.float().to(dev),
                       w.float().to(dev), EPS, x_out=xs)
    close(store[n], x + y, F32)
    close(xs, want_x, F32)
    close(h, zo.rms_norm(want_x, w, EPS), dtype)
    # the last layer keeps neither its result nor the averaged stream
    before = store.clone()
    h2 = ops.depth_norm(x.float().to(dev), y.to(dtype).to(dev), store[:n], n,
                        coef.float().to(dev), w.float().to(dev), EPS,
                        store_new=False)
    close(h2, zo.rms_norm(want_x, w, EPS), dtype)
    assert torch.equal(before, store)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_embed_norm(dev, dtype):
    g = torch.Generator().manual_seed(0)
    emb, w = rnd(g, 50, 72, dtype=dtype), rnd(g, 72)
    ids = torch.tensor([0, 49, 7, 7])
    x = torch.empty(4, 72, device=dev)
    h = ops.embed_norm(ids.to(dev), emb.to(dtype).to(dev), w.float().to(dev),
                       EPS, x)
    close(x, emb[ids], F32)
    close(h, zo.rms_norm(emb[ids], w, EPS), dtype)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("F", [64, 333, 4104])
def test_poly_norm(dev, dtype, F):
    g = torch.Generator().manual_seed(F)
    z = rnd(g, 4, F + 16, dtype=dtype)
    coef = torch.tensor([0.7, -0.4, 1.3, 0.25], dtype=torch.float64)
    out = torch.full((4, F + 24), 9.0, dtype=dtype, device=dev)
    ops.poly_norm(z.to(dtype).to(dev)[:, 8:8 + F], coef.float().to(dev), EPS,
                  out[:, 16:16 + F])
    close(out[:, 16:16 + F], zo.poly_norm(z[:, 8:8 + F], coef, EPS), dtype)
    assert bool((out[:, :16] == 9).all()) and bool((out[:, 16 + F:] == 9).all())


def _pages(n_tokens, bs, extra, g):
    """Shuffled page numbers for n_tokens and the pool size."""
    need = -(-n_tokens // bs)
    return torch.randperm(need + extra, generator=g)[:need], need + extra


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("H,G,D,E,T", [
    (6, 2, 40, 24, 21), (3, 3, 20, 17, 21), (8, 1, 64, 80, 7),
    (1, 1, 130, 8, 33), (9, 3, 128, 128, 40), (2, 2, 256, 72, 17)])
def test_unit_qkv_and_value_mixing(dev, dtype, H, G, D, E, T):
    """Unit heads, padding, both roles of value mixing, skipped slots, and
    the fused launch with PolyNorm."""
    g = torch.Generator().manual_seed(H * D)
    bs, F = 8, 56
    Dp = -(-D // 8) * 8
    off, at = [], 8
    for n in (H * D, G * D, G * E, F):
        off.append(at)
        at = -(-(at + n) // 8) * 8
    z = rnd(g, T, at, dtype=dtype)
    pages, pool = _pages(T, bs, 3, g)
    slots = pages[torch.arange(T) // bs] * bs + torch.arange(T) % bs
    slots[5] = -1
    q_w = zo.unit_rms(z[:, off[0]:off[0] + H * D].view(T, H, D), EPS)
    k_w = zo.unit_rms(z[:, off[1]:off[1] + G * D].view(T, G, D), EPS)
    v_w = z[:, off[2]:off[2] + G * E].view(T, G, E)
    lam = torch.tensor(0.375)
    carry = rnd(g, T, G * E, dtype=dtype)
    coef = torch.tensor([0.7, -0.4, 1.3, 0.25])
    for mode in ("none", "first", "later"):
        kc = torch.zeros(pool, G, bs, Dp, dtype=dtype, device=dev)
        vc = torch.zeros(pool, G, E, bs, dtype=dtype, device=dev)
        vf = carry.to(dtype).to(dev)
        fo = torch.zeros(T, F, dtype=dtype, device=dev)
        zd = z.to(dtype).to(dev)
        q = ops.unit_qkv_cache(
            zd, off[:3], H, D, (kc, vc), slots.to(dev), EPS,
            v_first=None if mode == "none" else vf,
            lam=None if mode == "none" else lam.to(dev),
            first=mode == "first",
            ff=None if mode == "none" else
            (zd[:, off[3]:off[3] + F], fo, coef.to(dev)))
        close(q[..., :D], q_w, dtype)
        assert not bool(q[..., D:].any())
        want_v = v_w
        if mode == "first":
            close(vf, v_w.reshape(T, -1), dtype)
        if mode == "later":
            want_v = zo.mix_values(v_w, carry.view(T, G, E), lam.double())
        if mode != "none":
            close(fo, zo.poly_norm(z[:, off[3]:off[3] + F], coef.double(),
                                   EPS), dtype)
        live = slots >= 0
        blk, o = slots[live] // bs, slots[live] % bs
        close(kc.cpu()[blk, :, o][..., :D], k_w[live], dtype)
        close(vc.cpu()[blk, :, :, o], want_v[live], dtype)
        # nothing else was written: the skipped token's page slot is empty
        assert not bool(kc.cpu()[pages[0], :, 5].any())


ATTN = [
    # H, G, D, E, window, cap, talk, bias
    (6, 2, 40, 24, 19, 6.0, True, True),
    (4, 4, 16, 64, 0, 0.0, True, True),
    (5, 1, 64, 16, 33, 9.0, True, False),
    (12, 4, 72, 48, 50, 7.0, False, True),
    (16, 2, 128, 128, 64, 10.0, True, True),
    (32, 8, 128, 96, 40, 50.0, True, True),
    (32, 8, 128, 128, 45, 12.0, True, True),
    (8, 2, 64, 64, 31, 9.0, True, True),
    (32, 4, 64, 64, 0, 9.0, True, True),
    (12, 6, 64, 64, 31, 9.0, True, True),
    (6, 6, 128, 128, 0, 9.0, True, True),
    (24, 24, 24, 40, 1, 30.0, True, True),
    (40, 8, 32, 32, 37, 8.0, True, True),      # beyond the MFMA kernel
    (3, 1, 144, 136, 45, 50.0, True, True),     # beyond the MFMA kernel
    (1, 1, 8, 8, 300, 50.0, True, True),
]


def _attention_case(H, G, D, E, window, cap, talk, bias, n, dtype, seed=0):
    """One sequence of n tokens with some keys that stand out for a late
    query: a far one, and those at the window's edge."""
    g = torch.Generator().manual_seed(seed + H * D + n)
    q, k, v = (rnd(g, n, H, D), rnd(g, n, G, D), rnd(g, n, G, E))
    rows = [n - 1, n // 2]
    for i in rows:
        for j in {0, i - window, i - window + 1, i - 1} if window else {0, 3}:
            if 0 <= j < n:
                k[j] = q[i].view(G, H // G, D)[:, 0] * 1.5
    q, k = zo.unit_rms(q, EPS), zo.unit_rms(k, EPS)
    q, k, v = (t.to(dtype).double() for t in (q, k, v))
    mix = torch.eye(H, dtype=torch.float64) * 0.7 + rnd(g, H, H, std=0.3) \
        if talk else None
    scale = 12.0 / D
    s = torch.stack([q[:, h] @ k[:, h // (H // G)].T for h in range(H)])
    s = zo.soft_cap(s * scale, cap)
    if bias:
        s = zo.distance_bias(s)
    w = torch.softmax(s.masked_fill(~zo.visible(n, window), -math.inf), -1)
    w = zo.talk(w, mix) if talk else w
    gate = rnd(g, n, H, dtype=dtype)
    o = zo.output_gate(zo.apply_values(w, v), gate).reshape(n, H * E)
    p = dict(scale=scale, softcap=cap, window=window,
             slopes=zo.head_slopes(H).float() if bias else None,
             talk=mix.float() if talk else None)
    return q, k, v, gate, p, o


def _fill_pool(seqs, bs, dtype, dev, g):
    """Caches holding the sequences' k, v on shuffled pages; free slots hold
    large values that must not show."""
    G, D = seqs[0][0].shape[1:]
    E = seqs[0][1].shape[2]
    Dp = -(-D // 8) * 8
    need = [-(-k.shape[0] // bs) for k, _ in seqs]
    pool = sum(need) + 4
    perm = torch.randperm(pool, generator=g)
    kc = torch.full((pool, G, bs, Dp), 50.0)
    kc[..., D:] = 0
    vc = torch.full((pool, G, E, bs), 1e4)
    bt = torch.zeros(len(seqs), max(need), dtype=torch.int32)
    at = 0
    for i, (k, v) in enumerate(seqs):
        pages = perm[at:at + need[i]]
        at += need[i]
        bt[i, :need[i]] = pages
        t = torch.arange(k.shape[0])
        kc[pages[t // bs], :, t % bs, :D] = k.float()
        vc[pages[t // bs], :, :, t % bs] = v.float()
    return kc.to(dtype).to(dev), vc.to(dtype).to(dev), bt.to(dev)


def _prompt_meta(spans, dev):
    """spans: (start, end) of each sequence's rows."""
    lens = [e - s for s, e in spans]
    cu = torch.tensor([0] + lens).cumsum(0).int()
    which = torch.repeat_interleave(torch.arange(len(spans)),
                                    torch.tensor(lens)).int()
    rl = torch.cat([torch.arange(s, e) + 1 for s, e in spans]).int()
    ends = torch.tensor([e for _, e in spans]).int()
    return [t.to(dev) for t in (cu, ends, which, rl)] + [max(lens),
                                                         int(ends.max())]


def _talk_params(p, dev):
    return ops.TalkParams(**{k: v.to(dev) if torch.is_tensor(v) else v
                             for k, v in p.items()})


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("case", ATTN, ids=str)
def test_attention_prompt_and_rows(dev, dtype, case):
    """Two sequences: whole prompt and a late portion, then every row alone
    through the decode path; pages shuffled, stale slots poisoned."""
    H, G, D, E = case[:4]
    bs = 8 if D == 40 else 16
    g = torch.Generator().manual_seed(1)
    n0, n1 = 150, 71
    q0, k0, v0, g0, p, o0 = _attention_case(*case, n0, dtype)
    q1, k1, v1, g1, _, o1 = _attention_case(*case, n1, dtype, seed=9)
    if p["talk"] is not None:       # one layer: one mixing matrix
        o1 = _redo(q1, k1, v1, g1, p, case)
    kc, vc, bt = _fill_pool([(k0, v0), (k1, v1)], bs, dtype, dev, g)
    pad = kc.shape[3] - D
    tp = _talk_params(p, dev)
    for spans in (((0, n0), (n1 - 2, n1)), ((n0 - 37, n0), (0, n1))):
        cu, ends, which, rl, mq, ml = _prompt_meta(spans, dev)
        pick = lambda a, b: torch.cat([a[slice(*spans[0])],  # noqa: E731
                                       b[slice(*spans[1])]])
        q = torch.nn.functional.pad(pick(q0, q1), (0, pad)).to(dtype).to(dev)
        gate = pick(g0, g1).to(dtype).to(dev)
        out = torch.zeros(q.shape[0], H * E + 8, dtype=dtype, device=dev)
        ops.talk_attn_prefill(out[:, :H * E], q, (kc, vc), bt, cu, ends, mq,
                              ml, which, rl, tp, gate)
        close(out[:, :H * E], pick(o0, o1), dtype)
        assert not bool(out[:, H * E:].any())
    # decode rows: unequal lengths side by side, more rows than one
    for lens in ([n0, n1], [1, 2], [16, 17], [33, 64], [n0 - 5, 50]):
        q = torch.stack([q0[lens[0] - 1], q1[lens[1] - 1]])
        gate = torch.stack([g0[lens[0] - 1], g1[lens[1] - 1]])
        q = torch.nn.functional.pad(q, (0, pad)).to(dtype).to(dev)
        out = torch.zeros(2, H * E, dtype=dtype, device=dev)
        ops.talk_attn_rows(
            out, q, (kc, vc), bt,
            torch.tensor(lens, dtype=torch.int32, device=dev), max(lens), tp,
            gate.to(dtype).to(dev))
        close(out, torch.stack([o0[lens[0] - 1], o1[lens[1] - 1]]), dtype,
              scale=float(o0.pow(2).mean().sqrt()))


def _redo(q, k, v, gate, p, case):
    H, G, window, cap, bias = case[0], case[1], case[4], case[5], case[7]
    s = torch.stack([q[:, h] @ k[:, h // (H // G)].T for h in range(H)])
    s = zo.soft_cap(s * p["scale"], cap)
    if bias:
        s = zo.distance_bias(s)
    w = torch.softmax(s.masked_fill(~zo.visible(len(q), window), -math.inf),
                      -1)
    w = zo.talk(w, p["talk"].double())
    return zo.output_gate(zo.apply_values(w, v), gate).reshape(len(q), -1)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("window", [0, 700, 1000])
def test_long_context_partitions(dev, dtype, window):
    """Rows whose window spans several partitions, the last one partial."""
    n = 1203
    case = (4, 2, 64, 32, window, 30.0, True, True)
    g = torch.Generator().manual_seed(2)
    q, k, v, gate, p, o = _attention_case(*case, n, dtype)
    kc, vc, bt = _fill_pool([(k, v)], 16, dtype, dev, g)
    for ln in (n, 1024, 1025, 900, 130):
        out = torch.zeros(1, 128, dtype=dtype, device=dev)
        ops.talk_attn_rows(
            out, q[ln - 1:ln].to(dtype).to(dev), (kc, vc), bt,
            torch.tensor([ln], dtype=torch.int32, device=dev), 1500,
            _talk_params(p, dev), gate[ln - 1:ln].to(dtype).to(dev))
        close(out, o[ln - 1:ln], dtype, scale=float(o.pow(2).mean().sqrt()))


def test_oracle_notices_mistakes():
    """The attention cases above tell a window that is one token off, a
    missing mix, cap or bias from the right result."""
    case = list(ATTN[0])
    good = _attention_case(*case, 150, F32)[5]
    ref = float(good.pow(2).mean().sqrt())
    for pos, bad in ((4, 20), (4, 18), (5, 0.0), (7, False)):
        wrong = list(case)
        wrong[pos] = bad
        q, k, v, gate, p, _ = _attention_case(*case, 150, F32)
        s = _redo(q, k, v, gate, p, wrong)
        assert float((s - good).abs().max()) / ref > 0.3, (pos, bad)
    q, k, v, gate, p, _ = _attention_case(*case, 150, F32)
    s = _redo(q, k, v, gate, {**p, "talk": torch.eye(6)}, case)
    assert float((s - good).abs().max()) / ref > 0.3


# --------------------------------------------------------------------- model

def layer(heads, kv, dim, vdim, size, ff, scale=None, cap=25.0, v_mix=True):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim,
                      "vdim": vdim, "mask": {"size": size},
                      "scale": scale or 6.0 / dim, "softcap": cap,
                      "v_mix": v_mix},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


CONFIGS = {
    # layers of different shapes, a layer without feed-forward, value mixing
    # that starts at the second layer and skips one
    "varied": {"architecture": "Zederax", "vocab": 97, "width": 72,
               "norm": {"eps": 1e-5}, "layers": [
                   layer(3, 3, 24, 40, 21, 96, v_mix=False),
                   layer(6, 2, 40, 24, 50, 0, cap=18.0),
                   layer(2, 1, 16, 8, 9, 52, v_mix=False),
                   layer(4, 2, 20, 24, 37, 130, scale=0.4)]},
    "wide": {"architecture": "Zederax", "vocab": 300, "width": 128,
             "norm": {"eps": 3e-6}, "layers": [
                 layer(16, 4, 64, 64, 70, 264) for _ in range(3)]},
    # every size of one, the window of one token, one head
    "single": {"architecture": "Zederax", "vocab": 33, "width": 20,
               "norm": {"eps": 1e-6}, "layers": [
                   layer(1, 1, 12, 20, 1, 28),
                   layer(1, 1, 8, 20, 300, 0, cap=50.0)]},
}


def make_weights(cfg, seed=0):
    """bf16 tensors under their checkpoint names; queries and keys are
    large enough for single keys to stand out."""
    g = torch.Generator().manual_seed(seed)
    W, out = cfg["width"], {}

    def add(name, *shape, std=None, mean=0.0):
        std = std if std is not None else 1.0 / math.sqrt(shape[-1])
        out[name] = (torch.randn(shape, generator=g) * std + mean).to(BF16)

    add("embed", cfg["vocab"], W, std=1.0)
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        H, G = m["heads"], m["kv_heads"]
        add(p + "norm1", W, std=0.2, mean=1.0)
        for n, rows in (("q", H * m["dim"]), ("k", G * m["dim"]),
                        ("v", G * m["vdim"])):
            add(p + "mix." + n, rows, W)
            add(p + f"mix.{n}.b", rows, std=0.5)
        if m["v_mix"]:
            add(p + "mix.vmix", std=0.0, mean=0.4)
        add(p + "mix.talk", H, H, std=0.3)
        out[p + "mix.talk"] += torch.eye(H).to(BF16)
        add(p + "mix.g", H, W)
        add(p + "mix.o", W, H * m["vdim"])
        if l["mlp"]:
            F = l["mlp"]["ff"]
            add(p + "mlp.up", F, W)
            add(p + "mlp.down", W, F)
            add(p + "mlp.act", 4, std=0.2, mean=0.5)
        add(p + "dwa", i + 2, std=0.2)
        out[p + "dwa"][-1] += 0.8
    add("final.norm", W, std=0.2, mean=1.0)
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
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


_WANT = {}


def want_logits(name, cfg, w, ids):
    key = (name, tuple(ids))
    if key not in _WANT:
        _WANT[key] = zo.forward(cfg, w, ids)
    return _WANT[key]


def engine_for(folder, dev, dtype, blocks=64, seqs=4, **kw):
    kw.setdefault("enable_prefix_caching", False)
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
def test_layers_one_by_one(folders, dev):
    folder, cfg, w = folders["varied"]
    eng = engine_for(folder, dev, "float32", enforce_eager=True)
    ids = prompt(cfg, 60, 7)
    want, tap = [], []
    zo.forward(cfg, w, ids, layers_out=want)
    eng.model.layer_tap = tap
    eng.extend([("a", ids, [])])
    assert len(tap) == len(want)
    for a, b in zip(tap, want):
        close(a, b, F32)


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_and_reused_pages(folders, dev, dtype):
    """Portions beside single tokens, requests left out of steps, and a pool
    so small that pages and rows are used again."""
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


@pytest.mark.parametrize("dev", DEVICES)
def test_wanted_places_in_order(folders, dev):
    folder, cfg, w = folders["wide"]
    eng = engine_for(folder, dev, "float32")
    a, b = prompt(cfg, 30, 1), prompt(cfg, 21, 2)
    eng.extend([("b", b[:20], [])])
    out = eng.extend([("a", a, [29, 0]), ("b", b[20:], [0])])
    wa, wb = (want_logits("wide", cfg, w, t) for t in (a, b))
    check_rows(out, torch.stack([wa[29], wa[0], wb[20]]), "float32")
    assert eng.extend([("c", a[:3], [])]) is None
    for bad in ([("d", [], [])], [("d", [cfg["vocab"]], [])],
                [("d", [1], [1])], [("d", [1], []), ("d", [1], [])]):
        with pytest.raises(ValueError):
            eng.extend(bad)


def oracle_greedy(cfg, w, ids, n):
    ids = list(ids)
    for _ in range(n):
        ids.append(int(zo.forward(cfg, w, ids)[-1].argmax()))
    return ids[-n:]


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("mixed", [False, True])
def test_greedy_generation(folders, dev, mixed):
    """Through generate(): chunked prompts, shared prefixes, preemption."""
    folder, cfg, w = folders["varied"]
    prompts = [prompt(cfg, n, 40 + n) for n in (50, 3, 61)]
    prompts.append(prompts[0][:32] + prompt(cfg, 9, 3))     # shared prefix
    want = [oracle_greedy(cfg, w, p, 14) for p in prompts]
    sp = SamplingParams(temperature=0.0, max_tokens=14, ignore_eos=True)
    for kw in (dict(max_prefill_tokens=4096, enable_prefix_caching=True),
               dict(max_prefill_tokens=24, enable_prefix_caching=True),
               dict(max_prefill_tokens=24, blocks=10)):
        eng = engine_for(folder, dev, "float32", mixed_steps=mixed, **kw)
        outs = eng.generate(prompts, sp)
        full = [eng.seqs[f"gen-1-{i}"] for i in range(4)]
        outs = [(s.prompt_ids + s.output_ids)[len(p):]
                for s, p in zip(full, prompts)]
        assert outs == want, kw


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
        bad = zo.forward(c2, w2, ids)
        return float(((bad - good).pow(2).mean(-1).sqrt()
                      / good.std()).max())

    for i in range(4):
        c2 = json.loads(json.dumps(cfg))
        c2["layers"][i]["mixer"]["mask"]["size"] += 1
        assert off(c2, w) > 10 * MODEL_TOL["float32"], i
    c2 = json.loads(json.dumps(cfg))
    c2["layers"][3]["mixer"]["v_mix"] = False
    assert off(c2, w) > 0.08
    for n in ("l1.mix.talk", "l2.dwa", "l3.mlp.act", "l3.mix.vmix",
              "l0.mix.g", "l1.mix.q.b"):
        assert off(cfg, {**w, n: w[n] * 0.5}) > 10 * MODEL_TOL["float32"], n


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_graph_replays_match_eager(folders, dtype):
    """Captured decode, replayed many times with eager prompts between."""
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


# ----------------------------------------------------------------- framework

def test_config_reader():
    cfg = ZederaxConfig.from_json(CONFIGS["varied"], "x")
    assert [l.ff for l in cfg.layers] == [96, 0, 52, 130]
    assert cfg.layers[3].mixer.scale == 0.4
    assert [k.k_dim for k in cfg.kv_layers()] == [24, 40, 16, 24]
    m = ZederaxForCausalLM(cfg)
    assert m.first_v_mix == 1
    bad = json.loads(json.dumps(CONFIGS["wide"]))
    bad["layers"][0]["type"] = "other"
    with pytest.raises(ValueError):
        ZederaxConfig.from_json(bad)
    bad = json.loads(json.dumps(CONFIGS["wide"]))
    bad["layers"][0]["mlp"]["kind"] = "other"
    with pytest.raises(ValueError):
        ZederaxConfig.from_json(bad)
    bad = json.loads(json.dumps(CONFIGS["wide"]))
    bad["layers"][1]["mixer"]["vdim"] = 32     # values no longer blend
    with pytest.raises(ValueError):
        ZederaxForCausalLM(ZederaxConfig.from_json(bad))
    with pytest.raises(ValueError):
        ZederaxForCausalLM(cfg, tp_size=2)


def test_small_tensors_stay_fp32():
    m = ZederaxForCausalLM(PRESETS["tiny-zederax"]).to(BF16)
    l = m.layers[0]
    assert m.embed_tokens.weight.dtype == l.in_proj.weight.dtype == BF16
    for t in (l.norm_w, l.talk, l.vmix, l.act, l.dwa, l.slopes,
              m.final_norm_w):
        assert t.dtype == F32
    assert torch.equal(l.slopes, zo.head_slopes(6).float())


def test_registry(tmp_path, folders):
    folder, cfg, w = folders["varied"]
    assert registry.get_config(folder).vocab_size == 97
    assert registry.get_config("llama3-8b").num_layers == 32
    with pytest.raises(KeyError):
        registry.get_config("no-such-model")
    (tmp_path / "config.json").write_text('{"architecture": "Other"}')
    with pytest.raises(ValueError):
        registry.get_config(str(tmp_path))
    m = registry.build_model(folder, F32, torch.device("cpu"))
    for n, dst in m.checkpoint_targets().items():
        assert torch.equal(dst, w[n].float()), n


def test_registry_loads_llama_folders(tmp_path):
    from helix_amd.engine.weights import save_sharded
    from helix_amd.models.llama import PRESETS as LLAMA, LlamaForCausalLM
    c = LLAMA["tiny-qwen"]
    (tmp_path / "config.json").write_text(json.dumps({
        "architectures": ["Qwen2ForCausalLM"], "vocab_size": c.vocab_size,
        "hidden_size": c.hidden_size, "num_hidden_layers": c.num_layers,
        "intermediate_size": c.intermediate_size, "num_attention_heads": 4,
        "num_key_value_heads": 2, "rope_theta": 10000.0, "rms_norm_eps": 1e-5,
        "max_position_embeddings": 512}))
    src = LlamaForCausalLM(c).init_random(5)
    save_sharded(src, str(tmp_path))
    m = registry.build_model(str(tmp_path), F32, torch.device("cpu"))
    assert m.cfg.attention_bias and m.cfg.sliding_window == 0
    for (n, a), (_, b) in zip(src.named_parameters(), m.named_parameters()):
        assert torch.equal(a, b), n


def test_checkpoint_errors(tmp_path, folders):
    from safetensors.torch import save_file
    folder, cfg, w = folders["varied"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    cpu = torch.device("cpu")
    part = {n: t for n, t in w.items() if n != "l1.mix.vmix"}
    save_file(part, str(tmp_path / "model.safetensors"))
    registry.build_model(str(tmp_path), F32, cpu)  # unused coefficient
    part = {n: t for n, t in w.items() if n != "l2.mix.talk"}
    save_file(part, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="l2.mix.talk"):
        registry.build_model(str(tmp_path), F32, cpu)
    save_file({**w, "l0.dwa": torch.ones(3)},
              str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="l0.dwa"):
        registry.build_model(str(tmp_path), F32, cpu)


def test_cache_geometry():
    cfg = ZederaxConfig.from_json(CONFIGS["varied"])
    kv = KVCache.for_layers(cfg.kv_layers(), 16, 3, "cpu", dtype=F32)
    assert kv.caches[0][0].shape == (3, 3, 16, 24)
    assert kv.caches[0][1].shape == (3, 3, 40, 16)
    total = sum(t.numel() * 4 for c in kv.caches for t in c)
    assert total == 3 * KVCache.block_bytes(0, 0, 0, 16, F32,
                                            cfg.kv_layers())


def test_engine_refuses_what_it_cannot_serve(folders):
    folder = folders["wide"][0]
    for kw in (dict(quantization="fp8"), dict(kv_cache_dtype="fp8"),
               dict(block_size=12)):
        with pytest.raises(ValueError):
            engine_for(folder, "cpu", "float32", **kw)
    with pytest.raises(ValueError):
        LLMEngine(EngineConfig(model="tiny", dtype="float32",
                               kv_cache_blocks=8), device="cpu")


@pytest.mark.parametrize("dev", DEVICES)
def test_replay_program(folders, dev, tmp_path, monkeypatch, capsys):
    import numpy as np
    folder, cfg, w = folders["varied"]
    a, b = prompt(cfg, 70, 1), prompt(cfg, 20, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:64], "want": []}],
         "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[64:], "want": [5]},
                                {"id": "b", "tokens": b, "want": [0, 19]}],
         "end": ["a", "b"]},
        {"step": 2, "entries": [{"id": "a", "tokens": b[:1], "want": [0]}],
         "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO(
        "".join(json.dumps(s) + "\n" for s in steps)))
    rc = replay.main(["--model", folder, "--dtype", "float32", "--out",
                      str(tmp_path / "o"), "--max-tokens", "192",
                      "--device", dev])
    assert rc == 0
    assert capsys.readouterr().out.split("\n")[:3] == [
        "done 0", "done 1", "done 2"]
    assert not (tmp_path / "o" / "0.f32").exists()

    def read(n):
        return torch.from_numpy(np.fromfile(tmp_path / "o" / f"{n}.f32",
                                            "<f4")).view(-1, cfg["vocab"])

    wa, wb = (want_logits("varied", cfg, w, t) for t in (a, b))
    check_rows(read(1), torch.stack([wa[69], wb[0], wb[19]]), "float32")
    check_rows(read(2), wb[:1], "float32")


def test_command_line_generate(folders):
    from typer.testing import CliRunner
    from helix_amd.cli import app
    folder, cfg, w = folders["varied"]
    ids = prompt(cfg, 12, 9)
    r = CliRunner().invoke(app, [
        "generate", " ".join(map(str, ids)), "--ids", "-m", folder,
        "--max-tokens", "6", "--dtype", "float32", "--device", "cpu"])
    assert r.exit_code == 0, r.output
    assert [int(t) for t in r.output.split()] == oracle_greedy(cfg, w, ids, 6)


def test_runner_serves_it():
    from helix_amd.runner.service import (DEFAULT_SPECS, LLMInstance,
                                          estimate_model_bytes)
    import threading
    spec = DEFAULT_SPECS["tiny-zederax"]
    assert estimate_model_bytes(spec) > 1 << 30
    inst = LLMInstance(spec, "cpu")
    try:
        done, toks = threading.Event(), []

        def on_token(seq, tok, fin):
            toks.append(tok)
            if fin:
                done.set()
        inst.submit("r", [5, 6, 7], SamplingParams(max_tokens=4,
                                                   ignore_eos=True), on_token)
        assert done.wait(60) and len(toks) == 4
    finally:
        inst.shutdown()


@pytest.mark.parametrize("dev", DEVICES)
def test_mixed_steps_of_the_llama_path(dev):
    """The other models take mixed batches through the same step."""
    outs = []
    for mixed in (False, True):
        eng = LLMEngine(EngineConfig(
            model="tiny", max_num_seqs=4, max_model_len=128,
            kv_cache_blocks=64, eos_token_id=-1, max_prefill_tokens=20,
            mixed_steps=mixed, enforce_eager=True), device=dev)
        g = torch.Generator().manual_seed(3)
        ids = torch.randint(0, 512, (3, 44), generator=g).tolist()
        alone = [eng.extend([(f"x{i}", t, [43])]).float().cpu()
                 for i, t in enumerate(ids)]
        for i in range(3):
            eng.release(f"x{i}")
        eng.extend([("a", ids[0][:43], []), ("b", ids[1][:30], [])])
        both = eng.extend([("a", ids[0][43:], [0]), ("b", ids[1][30:], [13]),
                           ("c", ids[2], [43])]).float().cpu()
        for got, want in zip(both, alone):
            assert float((got - want[0]).abs().max()) < 0.05 * float(
                want.abs().max()) + 1e-3
        for sid in "abc":
            eng.release(sid)
        outs.append([len(o) for o in eng.generate(
            ids, SamplingParams(max_tokens=5, ignore_eos=True))])
    assert outs[0] == outs[1] == [5, 5, 5]
