"""Plain oracle of the Mogisun design, written from its equations only: one
function per mechanism, float64 numpy throughout, whole sequences from
position 0, no cache, no batching, nothing shared with the serving path.

A model is (cfg, W): ``cfg`` the dictionary of config.json and ``W`` a
dictionary tensor name -> numpy array.
"""

import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def sigmoid(z):
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def softmax_rows(scores):
    e = np.exp(scores - scores.max())
    return e / e.sum()


# ------------------------------------------------ gated linear attention
def channel_decay(h, P, tau):
    """One decay per key channel and token, sigmoid(z)^(1/tau) with z a
    low-rank projection plus a bias."""
    z = (h @ P["a1"].T) @ P["a2"].T + P["a2.b"]
    return np.exp(-np.logaddexp(0.0, -z) / tau)


def decayed_memory(q, k, v, alpha):
    """S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t, one head:
    q, k, alpha [T, D], v [T, V]."""
    S = np.zeros((q.shape[1], v.shape[1]))
    o = np.zeros_like(v)
    for t in range(q.shape[0]):
        S = alpha[t][:, None] * S + np.outer(k[t], v[t])
        o[t] = S.T @ q[t]
    return o


def gla(h, P, mc, eps):
    H, D, V = mc["heads"], mc["dim"], mc["vdim"]
    T = h.shape[0]
    q = (h @ P["q"].T).reshape(T, H, D) / math.sqrt(D)
    k = (h @ P["k"].T).reshape(T, H, D)
    v = (h @ P["v"].T).reshape(T, H, V)
    alpha = channel_decay(h, P, mc["tau"]).reshape(T, H, D)
    o = np.stack([decayed_memory(q[:, i], k[:, i], v[:, i], alpha[:, i])
                  for i in range(H)], 1)
    o = rms(o, eps) * P["norm"]
    return (o.reshape(T, H * V) * silu(h @ P["g"].T)) @ P["o"].T


# ------------------------------------------------------------- attention
def query_temperature(pos, qt):
    return 1.0 + qt["coef"] * math.log(math.floor((pos + 1) / qt["every"])
                                       + 1)


def attention(h, P, mc, eps):
    """Position-free grouped-query attention: unit-RMS queries and keys, a
    temperature that grows with the query's position, one output gate per
    head, biased projections."""
    H, G, D, V = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    T = h.shape[0]
    q = rms((h @ P["q"].T + P["q.b"]).reshape(T, H, D), eps)
    k = rms((h @ P["k"].T + P["k.b"]).reshape(T, G, D), eps)
    v = (h @ P["v"].T + P["v.b"]).reshape(T, G, V)
    gate = sigmoid(h @ P["g"].T)
    o = np.zeros((T, H, V))
    for i in range(T):
        t = query_temperature(i, mc["q_temp"])
        for hd in range(H):
            g = hd // (H // G)
            p = softmax_rows((k[:i + 1, g] @ (q[i, hd] * t)) * mc["scale"])
            o[i, hd] = (p @ v[:i + 1, g]) * gate[i, hd]
    return o.reshape(T, H * V) @ P["o"].T + P["o.b"]


# ---------------------------------------------------------- feed-forward
def gated_ff(h, P):
    return (silu(h @ P["gate"].T) * (h @ P["up"].T)) @ P["down"].T


def under(P, prefix):
    return {k[len(prefix):]: v for k, v in P.items() if k.startswith(prefix)}


def moe(h, P, spec):
    """Top-k experts weighted by the softmax over the chosen logits, plus
    a shared expert behind one sigmoid gate per token."""
    E, top = spec["router"]["experts"], spec["router"]["top"]
    z = h @ P["router"].T
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        chosen = np.argsort(-z[t], kind="stable")[:top]
        for w, e in zip(softmax_rows(z[t, chosen]), chosen):
            assert e < E
            out[t] += w * gated_ff(h[t:t + 1], under(P, f"e{e}."))[0]
    if spec.get("shared"):
        out += gated_ff(h, under(P, "shared.")) \
            * sigmoid(h @ P["shared.sg"].T)
    return out


# ----------------------------------------------------------------- model
def run_order(cfg):
    """(layer, first of a pass?) in execution order."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, False) for i in range(a)]
    for _ in range(loop["times"]):
        out += [(i, i == a) for i in range(a, b)]
    return out + [(i, False) for i in range(b, n)]


def forward(cfg, W, tokens, layer_out=None):
    """Logits [T, vocab] of one sequence from position 0; ``layer_out`` (a
    list) receives the residual after every layer run."""
    W = {k: np.asarray(v, dtype=np.float64) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    x0 = W["embed"][np.asarray(tokens, dtype=np.int64)]
    x = x0
    for i, first in run_order(cfg):
        lc = cfg["layers"][i]
        if first:
            x = np.concatenate([x, x0], 1) @ W["loop.in"].T
        L = under(W, f"l{i}.")
        h = rms(x, eps) * L["norm1"]
        mixer = {"gla": gla, "attention": attention}[lc["type"]]
        y = mixer(h, under(L, "mix."), lc["mixer"], eps)
        x = x + y * sigmoid(h @ L["rg1"].T + L["rg1.b"])
        if lc.get("mlp") is not None:
            h = rms(x, eps) * L["norm2"]
            P = under(L, "mlp.")
            y = moe(h, P, lc["mlp"]) if lc["mlp"]["kind"] == "moe" \
                else gated_ff(h, P)
            x = x + y * sigmoid(h @ L["rg2"].T + L["rg2.b"])
        if layer_out is not None:
            layer_out.append(x.copy())
    z = (rms(x, eps) * W["final.norm"]) @ W["head"].T
    z = z * cfg.get("logit_scale", 1.0)
    cap = cfg.get("logit_softcap")
    return cap * np.tanh(z / cap) if cap else z
