"""Plain whole-sequence float64 evaluation of a Sepitar model: one function per mechanism, numpy only, no code shared
with the package.  ``w`` maps checkpoint tensor names to float64 arrays, ``cfg`` is the config.json dict; a sequence is
evaluated from position 0 in one go (no cache, keys and values of latent attention materialised head by head)."""
import math

import numpy as np

ALPHA = 1.702          # of the gated unit's sigmoid


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def plus_one_norm(x, w, eps):
    """RMS norm whose stored weight is the difference from one."""
    return rms(x, eps) * (1.0 + w)


# -- positions -----------------------------------------------------------------------------------------
def base_freqs(rot):
    return np.array([float(rot["base"]) ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)])


def wavelength_freqs(rot):
    """Frequencies scaled by their wavelength: short ones kept, long ones divided, a blend between."""
    sc = rot.get("scaling")
    out = base_freqs(rot)
    if not sc:
        return out
    for i, f in enumerate(base_freqs(rot)):
        wave = 2.0 * math.pi / f
        if wave < sc["original"] / sc["high"]:
            continue
        if wave > sc["original"] / sc["low"]:
            out[i] = f / sc["factor"]
        else:
            s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
            out[i] = (1.0 - s) * f / sc["factor"] + s * f
    return out


def ramp_freqs(rot):
    """(frequencies, factor on cos and sin) of the ramp between kept and divided pairs."""
    sc = rot.get("scaling")
    f = base_freqs(rot)
    if not sc:
        return f, 1.0
    at = lambda turns: rot["dims"] * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(rot["base"]))  # noqa: E731
    lo, hi = max(math.floor(at(sc["fast"])), 0), min(math.ceil(at(sc["slow"])), rot["dims"] - 1)
    ramp = np.array([min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(len(f))])
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_half(x, freqs):
    """x [T, heads, D]: entry i turns with entry i + n, n = len(freqs); entries from 2n on pass."""
    n = len(freqs)
    y = x.copy()
    a = np.arange(x.shape[0])[:, None, None] * freqs
    u, v = x[..., :n], x[..., n:2 * n]
    y[..., :n], y[..., n:2 * n] = u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)
    return y


def rotate_pairs(x, freqs, m):
    """x [T, heads, D]: entry 2i turns with entry 2i + 1; cos and sin times m."""
    n = 2 * len(freqs)
    y = x.copy()
    a = np.arange(x.shape[0])[:, None, None] * freqs
    c, s = m * np.cos(a), m * np.sin(a)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y[..., 0:n:2], y[..., 1:n:2] = u * c - v * s, v * c + u * s
    return y


def bucket(n, B, far):
    """Row of a B-row distance table: one row per distance in the first half, logarithmic steps up to ``far`` beyond."""
    half = B // 2
    if n < half:
        return n
    r = math.log(n / half) / math.log(far / half) * (B - half)
    if abs(r - round(r)) < 1e-9:          # a whole number: not left to rounding
        r = round(r)
    return min(B - 1, half + math.floor(r))


def distance_bias(T, rel, far):
    """[heads, T, T]: rel[bucket(i - j), head], zero above the diagonal."""
    out = np.zeros((rel.shape[1], T, T))
    rows = [rel[bucket(n, rel.shape[0], far)] for n in range(T)]
    for i in range(T):
        for j in range(i + 1):
            out[:, i, j] = rows[i - j]
    return out


# -- attention -------------------------------------------------------------------------------------------
def visible(T, mask=None):
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    v = j <= i
    if mask and mask.get("size"):
        v &= i - j < mask["size"]
    return v


def weights(s, vis, sink=None):
    """exp(s_j) / (sum over the visible keys [+ exp(sink)]), row by row."""
    s = np.where(vis, s, -np.inf)
    top = s.max(-1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, sink)
    e = np.exp(s - top)
    return e / (e.sum(-1, keepdims=True) + (np.exp(sink - top) if sink is not None else 0.0))


def soft_cap(s, cap):
    return cap * np.tanh(s / cap) if cap else s


def attend(q, k, v, scale, vis, bias=None, cap=None, sink=None):
    """q [T, H, D] over k [T, G, D], v [T, G, P] -> [T, H, P]."""
    T, H, _ = q.shape
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // k.shape[1])
        s = soft_cap(q[:, h] @ k[:, g].T * scale, cap)
        if bias is not None:
            s = s + bias[h]
        out[:, h] = weights(s, vis, None if sink is None else sink[h]) @ v[:, g]
    return out


def biased_attention(h, w, p, m, eps):
    """Biased projections, distance bias, sliding window, a gate per output element."""
    T, H, G = h.shape[0], m["heads"], m.get("kv_heads", m["heads"])
    lin = lambda n: h @ w[p + n].T + w[p + n + ".b"]  # noqa: E731
    q, k, v = (lin(n).reshape(T, c, -1) for n, c in (("q", H), ("k", G), ("v", G)))
    o = attend(q, k, v, m["scale"], visible(T, m.get("mask")), bias=distance_bias(T, w[p + "rel"], m["bias_max"]))
    return (o.reshape(T, -1) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T + w[p + "o.b"]


def capped_attention(h, w, p, m, eps):
    """Norms over whole projections, half-split rotation, capped scores, a sink, a gate per head."""
    T, H, G = h.shape[0], m["heads"], m.get("kv_heads", m["heads"])
    q = (rms(h @ w[p + "q"].T, eps) * w[p + "q.norm"]).reshape(T, H, -1)
    k = (rms(h @ w[p + "k"].T, eps) * w[p + "k.norm"]).reshape(T, G, -1)
    v = (h @ w[p + "v"].T).reshape(T, G, -1)
    if m.get("rot"):
        f = wavelength_freqs(m["rot"])
        q, k = rotate_half(q, f), rotate_half(k, f)
    o = attend(q, k, v, m["scale"], visible(T, m.get("mask")), cap=m.get("softcap"), sink=w[p + "sink"])
    return (o * sigmoid(h @ w[p + "g"].T)[:, :, None]).reshape(T, -1) @ w[p + "o"].T


def latent_attention(h, w, p, m, eps):
    """Keys and values from one normed latent per token, a rotated key part shared by the heads, a sink."""
    T, H, dn, dr, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    q = ((rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]) @ w[p + "uq"].T).reshape(T, H, dn + dr)
    down = h @ w[p + "dkv"].T
    c, kr = rms(down[:, :R], eps) * w[p + "dkv.norm"], down[:, R:]
    f, mult = ramp_freqs(m["rot"])
    qr, kr = rotate_pairs(q[..., dn:], f, mult), rotate_pairs(kr[:, None], f, mult)
    k = np.concatenate([(c @ w[p + "uk"].T).reshape(T, H, dn), np.repeat(kr, H, 1)], -1)
    v = (c @ w[p + "uv"].T).reshape(T, H, -1)
    o = attend(np.concatenate([q[..., :dn], qr], -1), k, v, m["scale"], visible(T, m.get("mask")), sink=w[p + "sink"])
    return o.reshape(T, -1) @ w[p + "o"].T


MIXERS = {"attention": biased_attention, "attention_2": capped_attention, "latent_attention": latent_attention}


# -- feed-forward ------------------------------------------------------------------------------------------
def clamped_unit(h, w, p, limit):
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(ALPHA * g) * (u + 1.0)) @ w[p + "down"].T


def route(z, top):
    """(chosen experts, their softmax) of one token's biased router logits."""
    chosen = np.argsort(-z, kind="stable")[:top]
    e = np.exp(z[chosen] - z[chosen].max())
    return chosen, e / e.sum()


def experts_ff(h, w, p, mlp):
    z = h @ w[p + "router"].T + w[p + "router.b"]
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(*route(z[t], mlp["router"]["top"])):
            out[t] += a * clamped_unit(h[t:t + 1], w, f"{p}e{e}.", mlp["expert"]["limit"])[0]
    if mlp.get("shared"):
        out += clamped_unit(h, w, p + "shared.", mlp["shared"]["limit"])
    return out


# -- the model ---------------------------------------------------------------------------------------------
def layer_order(cfg):
    """(layer, starts a repeated pass) in the order in which layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    out = [(i, False) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t > 0 and i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return out + [(i, False) for i in range(loop["stop"], n)]


def as_arrays(w):
    """Checkpoint tensors (torch, any dtype) -> float64 arrays."""
    return {k: (v if isinstance(v, np.ndarray) else v.double().cpu().numpy()) for k, v in w.items()}


def forward(cfg, w, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; ``layers_out`` (a list) receives the residual stream after every layer run."""
    w = as_arrays(w)
    eps = cfg["norm"]["eps"]
    first = w["embed"][np.asarray(tokens)]
    x = first
    for i, again in layer_order(cfg):
        spec, p = cfg["layers"][i], f"l{i}."
        if again:
            x = x + first
        h = plus_one_norm(x, w[p + "norm1"], eps)
        y = MIXERS[spec["type"]](h, w, p + "mix.", spec["mixer"], eps)
        if spec.get("mlp"):
            y = y + experts_ff(h, w, p + "mlp.", spec["mlp"])
        x = x + y
        if layers_out is not None:
            layers_out.append(x.copy())
    return plus_one_norm(x, w["final.norm"], eps) @ w["head"].T


def greedy(cfg, w, prompt, n):
    """``n`` greedy tokens after ``prompt``, each from a whole-sequence evaluation."""
    w = as_arrays(w)
    toks, out = list(prompt), []
    for _ in range(n):
        nxt = int(forward(cfg, w, toks)[-1].argmax())
        out.append(nxt)
        toks.append(nxt)
    return out
