"""Plain, slow Motolix: one function per mechanism, full sequences only.

Every function works on one whole sequence with no cache, no batch and no
chunking, in whatever dtype it is handed (tests use float64). It shares no
code with helix_amd; the framework is compared against it.

Notation: T tokens, W width, H query heads, G key/value heads, D query/key
size, E value size.
"""
import math

import torch


def layer_norm(x, w, b, eps):
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * w + b


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def sigmoid(x):
    return 1 / (1 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def gelu(x):
    """The form with a hyperbolic tangent."""
    return 0.5 * x * (1 + torch.tanh(math.sqrt(2 / math.pi)
                                     * (x + 0.044715 * x ** 3)))


# -------------------------------------------------------------------- rotation

def frequencies(dims, base, scaling=None):
    """One per pair; scaling slows down pairs of long wavelength."""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling:
            turns = scaling["original"] * f / (2 * math.pi)
            if turns < scaling["low"]:
                f = f / scaling["factor"]
            elif turns <= scaling["high"]:
                s = (turns - scaling["low"]) / (scaling["high"]
                                                - scaling["low"])
                f = (1 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return out


def turn(x, freqs, sign=1):
    """x [T, heads, n]: dimension i and i + len(freqs) of the first
    2 len(freqs) turn by sign * position * freqs[i]."""
    half = len(freqs)
    out = x.clone()
    pos = torch.arange(x.shape[0], dtype=x.dtype)[:, None]
    for i, f in enumerate(freqs):
        c, s = torch.cos(pos * f), sign * torch.sin(pos * f)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def rotate(x, rot):
    if not rot:
        return x
    return turn(x, frequencies(rot["dims"], rot["base"], rot.get("scaling")))


# ------------------------------------------------------------------- attention

def attend(q, k, v, weigh):
    """q [T, H, D], k [T, G, D], v [T, G, E]; weigh(head, raw scores of the
    keys a query sees) -> their weights. -> [T, H, E]."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // per
        for i in range(T):
            s = k[:i + 1, g] @ q[i, h]
            out[i, h] = weigh(h, s) @ v[:i + 1, g]
    return out


def softmax(s):
    e = torch.exp(s - s.max())
    return e / e.sum()


def sigmoid_attention(h, w, p, m):
    """Keys are also the values (before rotation); weights are sigmoids."""
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, D)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, D)
    temp, bias = w[p + "temp"], w[p + "pb"]
    o = attend(rotate(q, m.get("rot")), rotate(k, m.get("rot")), k,
               lambda j, s: sigmoid(s * m["scale"] * temp[j] + bias[j]))
    return o.reshape(T, -1) @ w[p + "o"].T + w[p + "o.b"]


def softmax_attention(h, w, p, m, eps):
    """Whole-projection norms of q and k; values travel rotated."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    D, E, rot = m["dim"], m["vdim"], m.get("rot")
    q = rms_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps).view(T, H, D)
    k = rms_norm(h @ w[p + "k"].T, w[p + "k.norm"], eps).view(T, G, D)
    v = (h @ w[p + "v"].T).view(T, G, E)
    vf = frequencies(E, rot["base"]) if rot else []
    o = attend(rotate(q, rot), rotate(k, rot), turn(v, vf),
               lambda j, s: softmax(s * m["scale"]))
    return turn(o, vf, -1).reshape(T, -1) @ w[p + "o"].T


# ------------------------------------------------------------ linear attention

def decays(z, tau):
    """Per key channel, in (0, 1)."""
    return sigmoid(z) ** (1.0 / tau)


def recurrence(q, k, v, a):
    """q, k, a [T, H, D], v [T, H, E] -> [T, H, E]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def linear_attention(h, w, p, m, eps):
    T, H, D, E = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, D)
    v = (h @ w[p + "v"].T).view(T, H, E)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    o = recurrence(q, k, v, decays(z.view(T, H, D), m["tau"]))
    o = rms_norm(o, w[p + "norm"], eps).reshape(T, -1)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


# ----------------------------------------------------------------------- model

def mixer(h, w, p, layer, eps):
    m = layer["mixer"]
    if layer["type"] == "attention":
        return sigmoid_attention(h, w, p, m)
    left = softmax_attention(h, w, p + "left.", m["left"], eps)
    right = linear_attention(h, w, p + "right.", m["right"], eps)
    return m["left_scale"] * left + m["right_scale"] * right


def feed_forward(h, w, p):
    return (gelu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def run_layer(x, w, i, layer, eps):
    p = f"l{i}."

    def norm(name, t):
        return layer_norm(t, w[p + name], w[p + name + ".b"], eps)

    x = x + norm("norm1b", mixer(norm("norm1", x), w, p + "mix.", layer, eps))
    if layer.get("mlp"):
        x = x + norm("norm2b", feed_forward(norm("norm2", x), w, p + "mlp."))
    return x


def order(cfg):
    """(layer, number of the pass that begins with it or None)."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


def run(cfg, w, tokens):
    """-> (logits [T, V], stream after every layer run [runs, T, W])."""
    eps = cfg["norm"]["eps"]
    x0 = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    x, taps = x0, []
    for i, t in order(cfg):
        if t is not None:
            x = torch.cat([x, x0], -1) @ w["loop.in"].T + w["loop.step"][t]
        x = run_layer(x, w, i, cfg["layers"][i], eps)
        taps.append(x)
    x = layer_norm(x, w["final.norm"], w["final.norm.b"], eps)
    return x @ w["head"].T * cfg["logit_scale"], torch.stack(taps)
