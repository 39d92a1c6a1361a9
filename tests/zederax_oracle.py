"""Plain, slow Zederax: one function per mechanism, full sequences only.

Every function works on one whole sequence with no cache, no batch and no
tiling, in whatever dtype it is handed (tests use float64). It shares no
code with helix_amd; the framework is compared against it.

Notation: T tokens, W width, H query heads, G key/value heads, D key size,
E value size, F feed-forward size.
"""
import math

import torch


def unit_rms(x, eps):
    """x over its root mean square along the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def head_slopes(H, dtype=torch.float64):
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)],
                        dtype=dtype)


def soft_cap(s, cap):
    return s if not cap else cap * torch.tanh(s / cap)


def distance_bias(s):
    """s [H, T, T]: take slope_h * (i - j) off."""
    H, T, _ = s.shape
    i = torch.arange(T, dtype=s.dtype)
    return s - head_slopes(H, s.dtype)[:, None, None] * (i[:, None] - i[None])


def visible(T, window):
    i = torch.arange(T)
    dist = i[:, None] - i[None, :]
    ok = dist >= 0
    return ok & (dist < window) if window else ok


def attention_weights(q, k, scale, cap, window):
    """q [T, H, D], k [T, G, D] -> softmax weights [H, T, T]."""
    T, H, _ = q.shape
    G = k.shape[1]
    s = torch.stack([q[:, h] @ k[:, h // (H // G)].T for h in range(H)])
    s = distance_bias(soft_cap(s * scale, cap))
    s = s.masked_fill(~visible(T, window), -math.inf)
    return torch.softmax(s, -1)


def talk(weights, mix):
    """New head h's weights: sum over g of mix[h, g] * weights[g]."""
    return torch.stack([sum(mix[h, g] * weights[g]
                            for g in range(weights.shape[0]))
                        for h in range(weights.shape[0])])


def apply_values(weights, v):
    """weights [H, T, T], v [T, G, E] -> [T, H, E]."""
    H, G = weights.shape[0], v.shape[1]
    return torch.stack([weights[h] @ v[:, h // (H // G)] for h in range(H)],
                       dim=1)


def mix_values(v, v_first, lam):
    return (1 - lam) * v + lam * v_first


def output_gate(o, gate_logits):
    """o [T, H, E], gate_logits [T, H]."""
    return o * torch.sigmoid(gate_logits)[..., None]


def attention(h, t, m, eps, v_first):
    """t(name) gives a tensor of this mixer. Returns (out, v_first)."""
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ t("q").T + t("q.b")).view(T, H, D)
    k = (h @ t("k").T + t("k.b")).view(T, G, D)
    v = (h @ t("v").T + t("v.b")).view(T, G, E)
    q, k = unit_rms(q, eps), unit_rms(k, eps)
    if m.get("v_mix"):
        if v_first is None:
            v_first = v
        else:
            v = mix_values(v, v_first, t("vmix"))
    w = attention_weights(q, k, m["scale"], m.get("softcap"),
                          m["mask"]["size"])
    o = apply_values(talk(w, t("talk")), v)
    o = output_gate(o, h @ t("g").T)
    return o.reshape(T, H * E) @ t("o").T, v_first


def poly_norm(z, coef, eps):
    a, b, c, e = coef
    return (a * unit_rms(z, eps) + b * unit_rms(z ** 2, eps)
            + c * unit_rms(z ** 3, eps) + e)


def feed_forward(h, t, eps):
    return poly_norm(h @ t("up").T, t("act"), eps) @ t("down").T


def depth_average(history, coef):
    """history: [X_0 .. X_{i+1}], coef [i + 2]."""
    return sum(c * x for c, x in zip(coef, history))


def forward(cfg, weights, tokens, dtype=torch.float64, layers_out=None):
    """cfg as config.json holds it. Returns logits [T, vocab]; layers_out
    (a list) receives the stream after every layer's averaging."""
    W = {n: w.to(dtype) for n, w in weights.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens)]
    history, v_first = [x], None
    for i, lay in enumerate(cfg["layers"]):
        h = rms_norm(x, W[f"l{i}.norm1"], eps)
        y, v_first = attention(h, lambda n, i=i: W[f"l{i}.mix.{n}"],
                               lay["mixer"], eps, v_first)
        if lay.get("mlp"):
            y = y + feed_forward(h, lambda n, i=i: W[f"l{i}.mlp.{n}"], eps)
        history.append(x + y)
        x = depth_average(history, W[f"l{i}.dwa"])
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, W["final.norm"], eps) @ W["embed"].T
