"""Plain whole-sequence float64 evaluation of a Fanotar model: one function per mechanism, numpy only, no
code shared with the package.  ``w`` maps checkpoint tensor names to float64 arrays, ``cfg`` is the
config.json dict; a sequence is evaluated from position 0 in one go (no cache, no state hand-over)."""
import math

import numpy as np

ALPHA = 1.702          # of the gated unit's sigmoid


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def dyn_tanh(x, w, name):
    """Elementwise norm: tanh(alpha x) * weight + bias."""
    return np.tanh(float(w[name + ".alpha"]) * x) * w[name] + w[name + ".b"]


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def short_conv(u, taps):
    """y_t[c] = sum_j taps[c, j] u_(t - K + 1 + j)[c], zeros before the start."""
    K = taps.shape[1]
    y = np.zeros_like(u)
    for t in range(u.shape[0]):
        for j in range(K):
            s = t - K + 1 + j
            if s >= 0:
                y[t] += taps[:, j] * u[s]
    return y


def query_temperature(T, q_temp):
    """One factor per position: 1 + coef ln(floor((p + 1) / every) + 1)."""
    return np.array([1.0 + q_temp["coef"] * math.log((p + 1) // q_temp["every"] + 1) for p in range(T)])


def slopes(H):
    return np.array([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)])


def sink_softmax(s, visible, sink):
    """Rows of exp(s_j) / (sum_j exp(s_j) + exp(sink)) over the visible j."""
    s = np.where(visible, s, -np.inf)
    top = np.maximum(s.max(-1, keepdims=True), sink)
    e = np.exp(s - top)
    return e / (e.sum(-1, keepdims=True) + np.exp(sink - top))


def keys_values(h, w, pre, m, eps):
    """Finished keys [T, G, D] (convolved, normed) and values [T, G, P] (convolved)."""
    T = h.shape[0]
    G, D, P = m["kv_heads"], m["dim"], m["vdim"]
    k = short_conv(h @ w[pre + "k"].T, w[pre + "k.conv"]).reshape(T, G, D)
    v = short_conv(h @ w[pre + "v"].T, w[pre + "v.conv"]).reshape(T, G, P)
    return rms(k, eps) * w[pre + "k.norm"], v


def attend(q, k, v, m, sink):
    """Finished queries [T, H, D] over keys and values: distance bias, sliding window, sink."""
    T, H, _ = q.shape
    G = k.shape[1]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    vis = j <= i
    size = (m.get("mask") or {}).get("size")
    if size:
        vis &= i - j < size
    sl = slopes(H)
    out = np.zeros((T, H, v.shape[2]))
    for hd in range(H):
        g = hd // (H // G)
        s = q[:, hd] @ k[:, g].T * m["scale"] - sl[hd] * (i - j)
        out[:, hd] = sink_softmax(s, vis, sink[hd]) @ v[:, g]
    return out


def attention(h, w, pre, m, eps, kv=None):
    """The mixer; ``kv``: the finished (keys, values) of an earlier layer instead of its own.  Returns
    (output, the keys and values it used)."""
    T = h.shape[0]
    H, D, P = m["heads"], m["dim"], m["vdim"]
    q = short_conv(h @ w[pre + "q"].T, w[pre + "q.conv"]).reshape(T, H, D)
    q = rms(q, eps) * w[pre + "q.norm"]
    if m.get("q_temp"):
        q = q * query_temperature(T, m["q_temp"])[:, None, None]
    if kv is None:
        kv = keys_values(h, w, pre, m, eps)
    o = attend(q, kv[0], kv[1], m, w[pre + "sink"]).reshape(T, H * P)
    return (o * sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T, kv


def clamped_unit(h, w, pre, limit):
    g = np.minimum(h @ w[pre + "gate"].T, limit)
    u = np.clip(h @ w[pre + "up"].T, -limit, limit)
    return (g * sigmoid(ALPHA * g) * (u + 1.0)) @ w[pre + "down"].T


def route(z, correction, top, scale):
    """(chosen experts, weights) of one token's router logits."""
    s = sigmoid(z)
    chosen = np.argsort(-(s + correction), kind="stable")[:top]
    return chosen, s[chosen] / (s[chosen].sum() + 1e-20) * scale


def experts_ff(h, w, pre, mlp):
    r = mlp["router"]
    z = h @ w[pre + "router"].T
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        chosen, wt = route(z[t], w[pre + "correction"], r["top"], r["scale"])
        for e, a in zip(chosen, wt):
            out[t] += a * clamped_unit(h[t:t + 1], w, f"{pre}e{e}.", mlp["expert"]["limit"])[0]
    if mlp.get("shared"):
        out += clamped_unit(h, w, pre + "shared.", mlp["shared"]["limit"])
    return out


def feed_forward(h, w, pre, mlp):
    if mlp["kind"] == "dense":
        return clamped_unit(h, w, pre, mlp["limit"])
    return experts_ff(h, w, pre, mlp)


def as_arrays(w):
    """Checkpoint tensors (torch, any dtype) -> float64 arrays."""
    return {k: (v if isinstance(v, np.ndarray) else v.double().cpu().numpy()) for k, v in w.items()}


def forward(cfg, w, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; ``layers_out`` (a list) receives the residual stream after every layer."""
    w = as_arrays(w)
    eps = cfg["norm"]["eps"]
    x = dyn_tanh(w["embed"][np.asarray(tokens)] * (cfg.get("embedding") or {}).get("scale", 1.0), w, "embed.norm")
    kvs = []
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        src = m.get("kv_from")
        y, kv = attention(dyn_tanh(x, w, p + "norm1"), w, p + "mix.", m, eps, kvs[src] if src is not None else None)
        kvs.append(kv)
        x = x + dyn_tanh(y, w, p + "norm1b")
        if spec.get("mlp"):
            x = x + dyn_tanh(feed_forward(dyn_tanh(x, w, p + "norm2"), w, p + "mlp.", spec["mlp"]), w, p + "norm2b")
        if layers_out is not None:
            layers_out.append(x.copy())
    return dyn_tanh(x, w, "final.norm") @ w["head"].T


def greedy(cfg, w, prompt, n):
    """``n`` greedy tokens after ``prompt``, each from a whole-sequence evaluation."""
    w = as_arrays(w)
    toks, out = list(prompt), []
    for _ in range(n):
        nxt = int(forward(cfg, w, toks)[-1].argmax())
        out.append(nxt)
        toks.append(nxt)
    return out
