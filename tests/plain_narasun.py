"""The Narasun decoder written out plainly, in float64 on the CPU: one function per mechanism, no cache, no batching, nothing
shared with the engine.  What the engine's kernels are compared with.

A model is (config, tensors): ``config`` the parsed config.json (a dict), ``tensors`` a dict of float64 arrays by the
names the model file uses.  Everything works on one whole sequence [T, ...].
"""
from __future__ import annotations

import math

import numpy as np


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    """An RMS norm whose stored weight is the difference from one."""
    return unit_rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


# ---- softmax attention with a query temperature and a sink -------------------------------------------------------------
def query_temperature(T, t):
    """[T] the factor on the query at position p: 1 + coef ln(floor((p + 1) / every) + 1) (all ones without ``t``)."""
    if not t:
        return np.ones(T)
    p = np.arange(T)
    return 1.0 + t["coef"] * np.log((p + 1) // t["every"] + 1.0)


def causal_softmax(s, sink):
    """Softmax of each row i of s [T, T] over the keys j <= i, with one more term exp(sink) in the denominator."""
    T = s.shape[0]
    s = np.where(np.tril(np.ones((T, T), bool)), s, -np.inf)
    m = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - m)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - m))


def attention(h, W, p, m):
    T = h.shape[0]
    H, G, d = m["heads"], m.get("kv_heads", m["heads"]), m["dim"]
    dv = m.get("vdim", d)
    q = (h @ W[p + ".q"].T).reshape(T, H, d) * query_temperature(T, m.get("q_temp"))[:, None, None]
    k = (h @ W[p + ".k"].T).reshape(T, G, d)
    v = (h @ W[p + ".v"].T).reshape(T, G, dv)
    out = np.zeros((T, H, dv))
    for hd in range(H):
        g = hd // (H // G)
        out[:, hd] = causal_softmax((q[:, hd] @ k[:, g].T) * m["scale"], float(W[p + ".sink"][hd])) @ v[:, g]
    return out.reshape(T, H * dv) @ W[p + ".o"].T


# ---- time mixing with a bonus for the current token ---------------------------------------------------------------------
def shifted_mix(h, mu):
    """h + (h' - h) mu with h' the row before (zeros before the first)."""
    before = np.concatenate([np.zeros((1, h.shape[1])), h[:-1]])
    return h + (before - h) * mu


def time_mix_recurrence(r, k, v, w, u):
    """One head: r, k, w [T, d], v [T, dv], u [d].  o_t = (S + diag(u) k v^T)^T r; then S <- diag(w) S + k v^T."""
    S, out = np.zeros((r.shape[1], v.shape[1])), np.zeros_like(v)
    for t in range(r.shape[0]):
        kv = np.outer(k[t], v[t])
        out[t] = (S + u[:, None] * kv).T @ r[t]
        S = w[t][:, None] * S + kv
    return out


def time_mix(h, W, p, m, eps):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    mix = {s: shifted_mix(h, W[f"{p}.mu.{s}"]) for s in "rkvgw"}
    r, k, v = ((mix[s] @ W[f"{p}.{s}"].T).reshape(T, H, d) for s in "rkv")
    gate = silu(mix["g"] @ W[p + ".g"].T)
    w = np.exp(-np.exp(np.tanh(mix["w"] @ W[p + ".w1"].T) @ W[p + ".w2"].T + W[p + ".w0"])).reshape(T, H, d)
    out = np.zeros((T, H, d))
    for hd in range(H):
        out[:, hd] = time_mix_recurrence(r[:, hd], k[:, hd], v[:, hd], w[:, hd], W[p + ".u"][hd])
    return (unit_rms(out, eps).reshape(T, H * d) * W[p + ".norm"] * gate) @ W[p + ".o"].T


def parallel_mixers(h, W, p, m, eps):
    return m["left_scale"] * attention(h, W, p + ".left", m["left"]) + m["right_scale"] * time_mix(h, W, p + ".right", m["right"], eps)


# ---- matrix memory with exponential gates -------------------------------------------------------------------------------
def soft_cap(z, cap):
    return cap * np.tanh(z / cap)


def matrix_memory_recurrence(q, k, v, log_i, log_f):
    """One head: q (already scaled), k [T, d], v [T, dv], log_i, log_f [T]: the memory S and the normaliser n, both kept
    relative to exp(m) with the running maximum m, which starts at 0."""
    T, d = q.shape
    S, n, m, out = np.zeros((d, v.shape[1])), np.zeros(d), 0.0, np.zeros_like(v)
    for t in range(T):
        m_new = max(log_f[t] + m, log_i[t])
        keep, write = math.exp(log_f[t] + m - m_new), math.exp(log_i[t] - m_new)
        S = keep * S + write * np.outer(k[t], v[t])
        n = keep * n + write * k[t]
        m = m_new
        out[t] = (S.T @ q[t]) / (max(abs(float(n @ q[t])), math.exp(-m)) + 1e-6)
    return out


def matrix_memory(h, W, p, m, eps):
    T, H, d, cap = h.shape[0], m["heads"], m["dim"], m["gate_cap"]
    dv = m.get("vdim", d)
    q = (h @ W[p + ".q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ W[p + ".k"].T).reshape(T, H, d)
    v = (h @ W[p + ".v"].T).reshape(T, H, dv)
    log_i = soft_cap(h @ W[p + ".i"].T + W[p + ".i.b"], cap)
    log_f = log_sigmoid(soft_cap(h @ W[p + ".f"].T + W[p + ".f.b"], cap))
    out = np.stack([matrix_memory_recurrence(q[:, a], k[:, a], v[:, a], log_i[:, a], log_f[:, a]) for a in range(H)], axis=1)
    return (unit_rms(out, eps).reshape(T, H * dv) * W[p + ".norm"] * sigmoid(h @ W[p + ".g"].T)) @ W[p + ".o"].T


# ---- feed-forward ---------------------------------------------------------------------------------------------------------
def expert(h, W, p):
    return (silu(h @ W[p + ".gate"].T) * (h @ W[p + ".up"].T)) @ W[p + ".down"].T


def route(h, W, p, r):
    """(ids [T, top], weights [T, top]): the highest scores sigmoid(W_r h) and the scores themselves."""
    s = sigmoid(h @ W[p + ".router"].T)
    ids = np.argsort(-s, axis=-1, kind="stable")[:, :r["top"]]
    return ids, np.take_along_axis(s, ids, axis=-1)


def moe(h, W, p, m):
    """The chosen experts read the row times their weight; their outputs are added as they are."""
    ids, weights = route(h, W, p, m["router"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(ids[t], weights[t]):
            out[t] += expert(w * h[t:t + 1], W, f"{p}.e{e}")[0]
    return out


def feed_forward(h, W, p, m):
    return expert(h, W, p) if m.get("kind", "dense") == "dense" else moe(h, W, p, m)


# ---- the model ------------------------------------------------------------------------------------------------------------
def run_order(config):
    """[(layer, pass or None)]: the looped span ``times`` times in a row; pass is set on a pass's first layer."""
    n, lp = len(config["layers"]), config.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        out += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return out + [(i, None) for i in range(lp["stop"], n)]


def pass_input(x, x0, W, t):
    """The stream with the embedding's output through one matrix, plus the pass's vector."""
    return np.concatenate([x, x0], axis=-1) @ W["loop.in"].T + W["loop.step"][t]


def layer(x, W, i, L, eps):
    """Both sub-blocks read the same normed row."""
    h = rms_norm(x, W[f"l{i}.norm1"], eps)
    if L["type"] == "parallel":
        y = parallel_mixers(h, W, f"l{i}.mix", L["mixer"], eps)
    else:
        y = matrix_memory(h, W, f"l{i}.mix", L["mixer"], eps)
    if L.get("mlp"):
        y = y + feed_forward(h, W, f"l{i}.mlp", L["mlp"])
    return x + y


def forward(config, W, tokens, return_layers=False):
    """float64 logits [T, vocab] of one sequence (and the stream after every layer run)."""
    tokens = np.asarray(tokens)
    eps = config["norm"]["eps"]
    x0 = W["embed"][tokens]
    x, after = x0.copy(), []
    for i, t in run_order(config):
        if t is not None:
            x = pass_input(x, x0, W, t)
        x = layer(x, W, i, config["layers"][i], eps)
        after.append(x.copy())
    logits = rms_norm(x, W["final.norm"], eps) @ W["head"].T
    return (logits, np.stack(after)) if return_layers else logits


def greedy_generate(config, W, prompt, n):
    """The n tokens that follow ``prompt`` when the most likely token is taken every time (the lowest id among equals)."""
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(np.argmax(forward(config, W, ids)[-1])))
    return ids[len(prompt):]
