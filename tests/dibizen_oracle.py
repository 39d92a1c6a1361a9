"""Plain, slow Dibizen: one function per mechanism, full sequences only.

Every function works on one whole sequence with no cache, no batch and no
chunking, in whatever dtype it is handed (tests use float64). It shares no
code with helix_amd; the framework is compared against it.

Notation: T tokens, W width, H query heads, G key/value heads, D query/key
size, E value size, C channels, N state size per channel, S streams.
"""
import math

import torch


def sigmoid(x):
    return 1 / (1 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0) + torch.log(1 + torch.exp(-x.abs()))


def softmax(s):
    e = torch.exp(s - s.max())
    return e / e.sum()


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


# ------------------------------------------------------------ stream and norms

def dyn_tanh(x, w, name):
    return torch.tanh(w[name + ".alpha"] * x) * w[name] + w[name + ".b"]


def embedding(w, tokens):
    at = torch.as_tensor(tokens)
    return w["embed"][at] + w["pos"][torch.arange(len(tokens))]


def read_streams(xs, into):
    """xs: list of S streams [T, W] -> what a sublayer reads."""
    u = torch.zeros_like(xs[0])
    for s, x in enumerate(xs):
        u = u + into[s] * x
    return u


def write_streams(xs, y, mix, out):
    """mix[from, to]: every new stream from all the old ones."""
    new = []
    for t in range(len(xs)):
        v = out[t] * y
        for s, x in enumerate(xs):
            v = v + mix[s, t] * x
        new.append(v)
    return new


# ------------------------------------------------------------------- attention

def query_temperature(pos, coef, every):
    return 1 + coef * math.log(math.floor((pos + 1) / every) + 1)


def keys_values(h, w, p, m):
    T, G = h.shape[0], m["kv_heads"]
    return ((h @ w[p + "k"].T).view(T, G, m["dim"]),
            (h @ w[p + "v"].T).view(T, G, m["vdim"]))


def attend(q, k, v, scale):
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E]; causal softmax."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // per
        for i in range(T):
            s = (k[:i + 1, g] @ q[i, h]) * scale
            out[i, h] = softmax(s) @ v[:i + 1, g]
    return out


def attention(h, w, p, m, kv):
    """kv: keys and values, of this layer or of the one it shares with."""
    T, H, D = h.shape[0], m["heads"], m["dim"]
    q = (h @ w[p + "q"].T).view(T, H, D)
    if m.get("q_temp"):
        t = [query_temperature(i, m["q_temp"]["coef"], m["q_temp"]["every"])
             for i in range(T)]
        q = q * torch.tensor(t, dtype=q.dtype)[:, None, None]
    o = attend(q, *kv, m["scale"]).reshape(T, -1)
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---------------------------------------------------------- lightning attention

def decayed_recurrence(q, k, v, decay):
    """q, k [T, H, D], v [T, H, E], decay per head -> [T, H, E]."""
    T, H, D = q.shape
    a = torch.tensor(decay, dtype=q.dtype)[:, None, None]
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        S = a * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def lightning(h, w, p, m, eps):
    T, H, D, E = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w[p + "q"].T).view(T, H, D)
    k = silu(h @ w[p + "k"].T).view(T, H, D)
    v = silu(h @ w[p + "v"].T).view(T, H, E)
    o = decayed_recurrence(q, k, v, m["decay"]).reshape(T, -1)
    o = rms_norm(o, w[p + "norm"], eps) * sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


# -------------------------------------------------------------- selective scan

def short_conv(x, taps, bias):
    """x [T, C], taps [C, K]: the last tap meets the current token."""
    T, K = x.shape[0], taps.shape[1]
    out = bias.expand_as(x).clone()
    for k in range(K):
        back = K - 1 - k
        if back < T:
            out[back:] = out[back:] + taps[:, k] * x[:T - back]
    return out


def scan(x, dt, A, B, C, D):
    """x, dt [T, C], A [C, N], B, C [T, N], D [C] -> [T, C]."""
    S = torch.zeros_like(A)
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S \
            + (dt[t] * x[t])[:, None] * B[t][None]
        out[t] = (S * C[t][None]).sum(1) + D * x[t]
    return out


def mamba1(h, w, p, m):
    I, R, N = m["inner"], m["dt_rank"], m["state"]
    xz = h @ w[p + "in"].T
    x = silu(short_conv(xz[:, :I], w[p + "conv"], w[p + "conv.b"]))
    dbc = x @ w[p + "x"].T
    dt = softplus(dbc[:, :R] @ w[p + "dt"].T + w[p + "dt.b"])
    y = scan(x, dt, -torch.exp(w[p + "A_log"]), dbc[:, R:R + N],
             dbc[:, R + N:], w[p + "D"])
    return (y * silu(xz[:, I:])) @ w[p + "o"].T


# --------------------------------------------------------------- feed-forward

def expert(h, up, down):
    u = torch.clamp(h @ up.T, min=0)
    return (u * u) @ down.T


def choose(scores, correction, r):
    """Of one token: scores over all experts -> the chosen ones, best
    first."""
    choice = (scores + correction).tolist()
    n, groups = len(choice), r["groups"]["count"]
    size = n // groups
    best = sorted(range(groups), key=lambda g: (
        -max(choice[g * size:(g + 1) * size]), g))[:r["groups"]["keep"]]
    open_ = [e for e in range(n) if e // size in best]
    return sorted(open_, key=lambda e: (-choice[e], e))[:r["top"]]


def mixture(h, w, p, m):
    r = m["router"]
    out = torch.zeros_like(h)
    z = h @ w[p + "router"].T
    for t in range(h.shape[0]):
        s = softmax(z[t])
        picked = choose(s, w[p + "correction"], r)
        total = sum(s[e] for e in picked) + 1e-20
        for e in picked:
            y = h[t] if e >= r["experts"] else expert(
                h[t], w[f"{p}e{e}.up"], w[f"{p}e{e}.down"])
            out[t] = out[t] + s[e] / total * y
    return out


# ----------------------------------------------------------------------- model

def run(cfg, w, tokens):
    """-> (logits [T, V], sum of the streams after every layer)."""
    eps, S = cfg["norm"]["eps"], cfg["streams"]
    xs = [embedding(w, tokens)] * S
    kv, taps = {}, []
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = dyn_tanh(read_streams(xs, w[p + "hc1.in"]), w, p + "norm1")
        if layer["type"] == "attention":
            src = m.get("kv_from")
            if src is None:
                src = i
                kv[i] = keys_values(h, w, p + "mix.", m)
            y = attention(h, w, p + "mix.", m, kv[src])
        elif layer["type"] == "lightning":
            y = lightning(h, w, p + "mix.", m, eps)
        else:
            y = mamba1(h, w, p + "mix.", m)
        xs = write_streams(xs, y, w[p + "hc1.mix"], w[p + "hc1.out"])
        if layer.get("mlp"):
            h = dyn_tanh(read_streams(xs, w[p + "hc2.in"]), w, p + "norm2")
            y = mixture(h, w, p + "mlp.", layer["mlp"])
            xs = write_streams(xs, y, w[p + "hc2.mix"], w[p + "hc2.out"])
        taps.append(sum(xs))
    x = dyn_tanh(sum(xs), w, "final.norm")
    cap = cfg["logit_softcap"]
    return cap * torch.tanh(x @ w["head"].T / cap), torch.stack(taps)
