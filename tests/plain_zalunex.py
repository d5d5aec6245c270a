"""A plain, slow implementation of the Zalunex decoder in NumPy float64, one function per mechanism, written
from the design's equations and sharing no code with the package.  Tests compare the engine with it; it reads a
configuration as the dictionary config.json holds and tensors by their checkpoint names.

Notation: T tokens of one sequence at positions 0 .. T-1; a stored matrix W is [out, in] and "W x" is
``x @ W.T``.  x starts as embed[token] + pos[position]; a sublayer s is added as x <- x + m * n_b(s(n(x))), n and n_b
root-mean-square norms whose weights are stored around zero.
"""
import json
import math
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
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * logistic(z)


def gelu(z):
    """The exact form, z times the normal distribution's function of z."""
    return 0.5 * z * (1.0 + np.vectorize(math.erf)(z / math.sqrt(2.0)))


def clamped_gate(gate, up, limit):
    """g = min(gate, limit), u = up held within +-limit: g * logistic(1.702 g) * (u + 1)."""
    g, u = np.minimum(gate, limit), np.clip(up, -limit, limit)
    return g * logistic(1.702 * g) * (u + 1.0)


def softcap(z, cap):
    return cap * np.tanh(z / cap) if cap else z


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def offset_norm(x, weight, eps):
    """An RMS norm whose weight is stored around zero."""
    return rms(x, eps) * (1.0 + weight)


def embedding(w, tokens, first=0):
    tokens = np.asarray(tokens)
    return w["embed"][tokens] + w["pos"][first + np.arange(len(tokens))]


# --------------------------------------------------------------------------------- attention
def sink_softmax(s, sink):
    """exp(s_j) / (exp(sink) + sum exp(s_j)) along the last axis, -inf for what is not seen."""
    m = np.maximum(np.max(s, axis=-1, keepdims=True), sink)
    e = np.exp(s - m)
    return e / (np.exp(sink - m) + np.sum(e, axis=-1, keepdims=True))


def window_attention(q, k, v, scale, sink, qpos, kpos, window=0):
    """q [Tq, H, d], k [Tk, G, d], v [Tk, G, dv]; head h reads key/value head h // (H / G).  A query at position i sees
    the keys at j with 0 <= i - j < window (0: every j <= i); exp(sink[h]) joins head h's denominator."""
    Tq, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((Tq, H, v.shape[2]))
    back = np.asarray(qpos)[:, None] - np.asarray(kpos)[None, :]
    seen = (back >= 0) & ((back < window) if window else True)
    for h in range(H):
        g = h // (H // G)
        s = np.where(seen, (q[:, h, :] @ k[:, g, :].T) * scale, -np.inf)
        out[:, h, :] = sink_softmax(s, sink[h]) @ v[:, g, :]
    return out


def attention(h, w, pre, m, eps):
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    G, dv = m.get("kv_heads", H), m.get("vdim", d)
    q = rms((h @ w[pre + "q"].T).reshape(T, H, d), eps) * w[pre + "q.norm"]
    k = rms((h @ w[pre + "k"].T).reshape(T, G, d), eps) * w[pre + "k.norm"]
    v = (h @ w[pre + "v"].T).reshape(T, G, dv)
    o = window_attention(q, k, v, m["scale"], w[pre + "sink"], np.arange(T), np.arange(T), (m.get("mask") or {}).get("size", 0))
    o = o * logistic(h @ w[pre + "g"].T)[:, :, None]
    return o.reshape(T, -1) @ w[pre + "o"].T


# -------------------------------------------------------------------------------- recurrence
def decayed_state(q, k, v, decay):
    """q, k [T, H, d], v [T, H, dv], decay [H]: S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]))
    out = np.zeros(v.shape)
    decay = np.asarray(decay, dtype=np.float64)[:, None, None]
    for t in range(T):
        S = decay * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hij,hi->hj", S, q[t])
    return out


def lightning(h, w, pre, m, eps):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    dv = m.get("vdim", d)
    q, k, v = (silu(h @ w[pre + n].T).reshape(T, H, -1) for n in ("q", "k", "v"))
    assert v.shape[2] == dv
    o = decayed_state(q, k, v, m["decay"]).reshape(T, -1)
    return (rms(o, eps) * w[pre + "norm"] * logistic(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def parallel_mixer(h, w, pre, m, eps):
    return (m.get("left_scale", 1.0) * attention(h, w, pre + "left.", m["left"], eps)
            + m.get("right_scale", 1.0) * lightning(h, w, pre + "right.", m["right"], eps))


# ------------------------------------------------------------------------------ feed-forward
def dense_ff(h, w, pre, limit):
    return clamped_gate(h @ w[pre + "gate"].T, h @ w[pre + "up"].T, limit) @ w[pre + "down"].T


def expert(h, w, pre):
    return gelu(h @ w[pre + "up"].T) @ w[pre + "down"].T


def choose_experts(logits, top):
    """-> (indices [T, top] of the largest scores logistic(z), those scores as they are)."""
    s = logistic(logits)
    order = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    return order, np.take_along_axis(s, order, axis=-1)


def mixture(h, w, pre, mlp):
    """An expert's weight multiplies what goes into it."""
    chosen, weight = choose_experts(h @ w[pre + "router"].T, mlp["router"]["top"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(chosen[t], weight[t]):
            out[t] += expert(a * h[t:t + 1], w, f"{pre}e{e}.")[0]
    return out


def feed_forward(h, w, pre, mlp):
    return dense_ff(h, w, pre, mlp["limit"]) if mlp["kind"] == "dense" else mixture(h, w, pre, mlp)


# ------------------------------------------------------------------------------------ model
def layer_runs(raw):
    """Layer numbers in running order."""
    n, loop = len(raw["layers"]), raw.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def forward(raw, w, tokens, trace=None):
    """Logits [T, vocab] of one sequence.  ``trace``: a list that receives the stream after every layer run."""
    eps, mult = raw["norm"]["eps"], raw.get("residual_mult", 1.0)
    x = embedding(w, tokens)
    for i in layer_runs(raw):
        layer, p = raw["layers"][i], f"l{i}."
        y = parallel_mixer(offset_norm(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps)
        x = x + mult * offset_norm(y, w[p + "norm1b"], eps)
        if layer.get("mlp"):
            y = feed_forward(offset_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"])
            x = x + mult * offset_norm(y, w[p + "norm2b"], eps)
        if trace is not None:
            trace.append(x.copy())
    return softcap(offset_norm(x, w["final.norm"], eps) @ w["head"].T, raw.get("logit_softcap"))
