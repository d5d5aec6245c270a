"""A plain, slow implementation of the Vugotar decoder in NumPy float64, one function per mechanism, written
from the design's equations and sharing no code with the package.  Tests compare the engine with it; it reads a
configuration as the dictionary config.json holds and tensors by their checkpoint names.

Notation: T tokens of one sequence at positions 0 .. T-1; a stored matrix W is [out, in] and "W x" is
``x @ W.T``.  A layer is parallel: with h = rms(x) * (1 + w), x <- x + (mixer(h) + ff(h)).
"""
import json
import struct

import numpy as np


# ----------------------------------------------------------------------------------- files
def read_tensors(path):
    """name -> float64 (or int64) array of a safetensors file; bfloat16 is widened exactly."""
    with open(path, "rb") as f:
        (n,) = struct.unpack("<Q", f.read(8))
        header = json.loads(f.read(n))
        blob = f.read()
    out = {}
    for name, info in header.items():
        if name == "__metadata__":
            continue
        lo, hi = info["data_offsets"]
        kind = info["dtype"]
        if kind == "BF16":
            a = (np.frombuffer(blob[lo:hi], dtype="<u2").astype(np.uint32) << 16).view(np.float32).astype(np.float64)
        elif kind == "F32":
            a = np.frombuffer(blob[lo:hi], dtype="<f4").astype(np.float64)
        else:
            raise ValueError(f"{name}: dtype {kind}")
        out[name] = a.reshape(info["shape"])
    return out


# ------------------------------------------------------------------------------ elementwise
def logistic(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * logistic(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def offset_norm(x, weight, eps):
    """An RMS norm whose weight is stored around zero."""
    return rms(x, eps) * (1.0 + weight)


# ---------------------------------------------------------------------------------- rotation
def rotate_pairs(x, positions, dims, base):
    """x [T, heads, n]: entries (2i, 2i+1) of the first ``dims`` are turned by position * base^(-2i/dims)."""
    out = np.array(x, dtype=np.float64, copy=True)
    f = float(base) ** (-2.0 * np.arange(dims // 2) / dims)
    a = (np.asarray(positions, dtype=np.float64)[:, None] * f[None, :])[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * np.cos(a) - v * np.sin(a)
    out[..., 1:dims:2] = v * np.cos(a) + u * np.sin(a)
    return out


# --------------------------------------------------------------------------------- attention
def sink_softmax(s):
    """exp(s_j) / (1 + sum exp(s_j)) along the last axis, -inf for what is not seen."""
    m = np.maximum(np.max(s, axis=-1, keepdims=True), 0.0)
    e = np.exp(s - m)
    return e / (np.exp(-m) + np.sum(e, axis=-1, keepdims=True))


def chunk_attention(q, k, v, scale, qpos, kpos, chunk=0):
    """q [Tq, H, d], k [Tk, G, d], v [Tk, G, dv]; head h reads key/value head h // (H / G).  A query at position i sees
    the keys at j <= i of its own chunk of ``chunk`` positions (0: all); a sink of score 0 joins the denominator."""
    Tq, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((Tq, H, v.shape[2]))
    qpos, kpos = np.asarray(qpos), np.asarray(kpos)
    seen = kpos[None, :] <= qpos[:, None]
    if chunk:
        seen &= (qpos[:, None] // chunk) == (kpos[None, :] // chunk)
    for h in range(H):
        g = h // (H // G)
        s = np.where(seen, (q[:, h, :] @ k[:, g, :].T) * scale, -np.inf)
        out[:, h, :] = sink_softmax(s) @ v[:, g, :]
    return out


def attention(h, w, pre, m, eps):
    T = h.shape[0]
    pos = np.arange(T)
    H, d = m["heads"], m["dim"]
    G, dv = m.get("kv_heads", H), m.get("vdim", d)
    q = (h @ w[pre + "q"].T).reshape(T, H, d)
    k = (h @ w[pre + "k"].T).reshape(T, G, d)
    v = (h @ w[pre + "v"].T).reshape(T, G, dv)
    rot = m.get("rot") or {}
    if rot.get("dims"):
        q, k = (rotate_pairs(t, pos, rot["dims"], rot["base"]) for t in (q, k))
    q, k = rms(q, eps), rms(k, eps)
    o = chunk_attention(q, k, v, m["scale"], pos, pos, (m.get("mask") or {}).get("size", 0))
    return o.reshape(T, -1) @ w[pre + "o"].T


# -------------------------------------------------------------------------------- recurrences
def causal_conv(x, taps, bias=None):
    """x [T, C], taps [C, K], the last column for the current token; zeros before the start."""
    T, K = x.shape[0], taps.shape[1]
    y = np.zeros_like(x)
    for j in range(K):
        back = K - 1 - j
        if back < T:
            y[back:] += x[:T - back] * taps[:, j]
    return y if bias is None else y + bias


def gated_delta(q, k, v, g, beta):
    """q, k [T, G, d] (unit keys, scaled unit queries), v [T, H, dv], g, beta [T, H]:
    S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q."""
    T, H, dv = v.shape
    G, d = q.shape[1:]
    S = np.zeros((H, d, dv))
    out = np.zeros((T, H, dv))
    for t in range(T):
        for h in range(H):
            kk, qq = k[t, h // (H // G)], q[t, h // (H // G)]
            S[h] *= g[t, h]
            u = beta[t, h] * (v[t, h] - S[h].T @ kk)
            S[h] += np.outer(kk, u)
            out[t, h] = S[h].T @ qq
    return out


def delta_mixer(h, w, pre, m, eps):
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    G, dv = m.get("kv_heads", H), m.get("vdim", d)
    q, k, v = (silu(causal_conv(h @ w[pre + n].T, w[pre + n + ".conv"])) for n in ("q", "k", "v"))
    q = unit(q.reshape(T, G, d)) * d ** -0.5
    k = unit(k.reshape(T, G, d))
    beta = logistic(h @ w[pre + "b"].T)
    g = np.exp(-np.exp(w[pre + "A_log"]) * softplus(h @ w[pre + "a"].T + w[pre + "dt_bias"]))
    o = gated_delta(q, k, v.reshape(T, H, dv), g, beta)
    o = rms(o, eps) * w[pre + "norm"]
    return (o.reshape(T, -1) * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def state_space(x, B, C, dt, a_log, D):
    """x [T, H, P], B, C [T, G, N], dt [T, H]: S_t = exp(-exp(a_log) dt) S_(t-1) + dt B x^T, y = S_t^T C + D x."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    S = np.zeros((H, N, P))
    y = np.zeros((T, H, P))
    keep = np.exp(-np.exp(a_log) * dt)
    for t in range(T):
        for h in range(H):
            g = h // (H // G)
            S[h] = keep[t, h] * S[h] + dt[t, h] * np.outer(B[t, g], x[t, h])
            y[t, h] = S[h].T @ C[t, g] + D[h] * x[t, h]
    return y


def mamba2_mixer(h, w, pre, m, eps):
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, xbc, dt = np.split(h @ w[pre + "in"].T, [inner, 2 * inner + 2 * G * N], axis=1)
    xbc = silu(causal_conv(xbc, w[pre + "conv"], w[pre + "conv.b"]))
    x, B, C = np.split(xbc, [inner, inner + G * N], axis=1)
    dt = softplus(dt + w[pre + "dt_bias"])
    y = state_space(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N), dt, w[pre + "A_log"], w[pre + "D"])
    y = y.reshape(T, inner) * silu(z)
    y = rms(y.reshape(T, m["norm_groups"], -1), eps).reshape(T, inner) * w[pre + "norm"]
    return y @ w[pre + "o"].T


def parallel_mixer(h, w, pre, m, eps):
    return (m["left_scale"] * attention(h, w, pre + "left.", m["left"], eps)
            + m["right_scale"] * delta_mixer(h, w, pre + "right.", m["right"], eps))


# ------------------------------------------------------------------------------ feed-forward
def dense_ff(h, w, pre):
    gate, up = (h @ w[pre + n].T + w[pre + n + ".b"] for n in ("gate", "up"))
    return (silu(gate) * up) @ w[pre + "down"].T + w[pre + "down.b"]


def gated_expert(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def choose_experts(logits, top, scale):
    """-> (indices [T, top] of the largest softmax scores, those scores over their sum (+ 1e-20), times scale)."""
    e = np.exp(logits - np.max(logits, axis=-1, keepdims=True))
    s = e / np.sum(e, axis=-1, keepdims=True)
    order = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    c = np.take_along_axis(s, order, axis=-1)
    return order, c / (np.sum(c, axis=-1, keepdims=True) + 1e-20) * scale


def mixture(h, w, pre, mlp):
    r = mlp["router"]
    chosen, weight = choose_experts(h @ w[pre + "router"].T, r["top"], r["scale"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(chosen[t], weight[t]):
            out[t] += a * gated_expert(h[t:t + 1], w, f"{pre}e{e}.")[0]
    if mlp.get("shared"):
        out = out + gated_expert(h, w, pre + "shared.") * logistic(h @ w[pre + "shared.sg"].T)
    return out


def feed_forward(h, w, pre, mlp):
    return dense_ff(h, w, pre) if mlp["kind"] == "dense" else mixture(h, w, pre, mlp)


# ------------------------------------------------------------------------------------ model
def layer_runs(raw):
    """[(layer, starts a pass that is not the first?)] in running order."""
    n, loop = len(raw["layers"]), raw.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    runs = [(i, False) for i in range(a)]
    for t in range(loop["times"]):
        runs += [(i, t > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


MIXERS = {"parallel": parallel_mixer, "mamba2": mamba2_mixer}


def forward(raw, w, tokens, trace=None):
    """Logits [T, vocab] of one sequence.  ``trace``: a list that receives the stream after every layer run."""
    eps = raw["norm"]["eps"]
    x0 = w["embed"][np.asarray(tokens)]
    x = x0
    for i, again in layer_runs(raw):
        layer, p = raw["layers"][i], f"l{i}."
        if again:
            x = x + x0
        h = offset_norm(x, w[p + "norm1"], eps)
        y = MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp"):
            y = y + feed_forward(h, w, p + "mlp.", layer["mlp"])
        x = x + y
        if trace is not None:
            trace.append(x.copy())
    return offset_norm(x, w["final.norm"], eps) @ w["head"].T
