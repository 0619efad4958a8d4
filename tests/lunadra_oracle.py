"""Plain oracle of the Lunadra design, written from its equations only: one
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


def softplus(z):
    return np.logaddexp(0.0, z)


def under(P, prefix):
    return {k[len(prefix):]: v for k, v in P.items() if k.startswith(prefix)}


# ------------------------------------------------------------- embedding
def bigram_rows(tokens, spec):
    """Row of the bigram table for every token: the last one for the first
    token, a hash of (previous, current) elsewhere."""
    n = spec["buckets"]
    rows = [n]
    for a, b in zip(tokens, tokens[1:]):
        rows.append((int(a) * spec["mul_prev"] + int(b) * spec["mul_cur"])
                    % n)
    return rows[:len(tokens)]


# ----------------------------------------------------------- matrix memory
def matrix_memory(q, k, v, li, lf):
    """One head, stabilised: q, k [T, D], v [T, V], log gates [T]."""
    S = np.zeros((q.shape[1], v.shape[1]))
    n = np.zeros(q.shape[1])
    m = 0.0
    out = np.zeros_like(v)
    for t in range(q.shape[0]):
        top = max(lf[t] + m, li[t])
        keep, write = math.exp(lf[t] + m - top), math.exp(li[t] - top)
        S = keep * S + write * np.outer(k[t], v[t])
        n = keep * n + write * k[t]
        m = top
        out[t] = (S.T @ q[t]) / (max(abs(n @ q[t]), math.exp(-m)) + 1e-6)
    return out


def mlstm(h, P, mc, eps):
    H, D, V, cap = mc["heads"], mc["dim"], mc["vdim"], mc["gate_cap"]
    T = h.shape[0]
    q = (h @ P["q"].T).reshape(T, H, D) / math.sqrt(D)
    k = (h @ P["k"].T).reshape(T, H, D)
    v = (h @ P["v"].T).reshape(T, H, V)
    li = cap * np.tanh((h @ P["i"].T + P["i.b"]) / cap)
    lf = -softplus(-cap * np.tanh((h @ P["f"].T + P["f.b"]) / cap))
    o = np.stack([matrix_memory(q[:, a], k[:, a], v[:, a], li[:, a],
                                lf[:, a]) for a in range(H)], 1)
    o = rms(o, eps).reshape(T, H * V) * P["norm"]
    return (o * sigmoid(h @ P["g"].T)) @ P["o"].T


# --------------------------------------------------------------- attention
def rotate_half(x, dims, base):
    """x [T, heads, D]; the first ``dims`` dimensions, pairs (i, i+dims/2)."""
    y = x.copy()
    half = dims // 2
    for i in range(half):
        a = np.arange(x.shape[0])[:, None] * float(base) ** (-2.0 * i / dims)
        u, v = x[:, :, i], x[:, :, i + half]
        y[:, :, i] = u * np.cos(a) - v * np.sin(a)
        y[:, :, i + half] = v * np.cos(a) + u * np.sin(a)
    return y


def window_attention(h, P, mc):
    H, G, D, V = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    T, rot = h.shape[0], mc["rot"]
    q = rotate_half((h @ P["q"].T).reshape(T, H, D), rot["dims"], rot["base"])
    k = rotate_half((h @ P["k"].T).reshape(T, G, D), rot["dims"], rot["base"])
    v = (h @ P["v"].T).reshape(T, G, V)
    out = np.zeros((T, H, V))
    for i in range(T):
        lo = max(0, i - mc["mask"]["size"] + 1)
        for a in range(H):
            g = a // (H // G)
            s = (k[lo:i + 1, g] @ q[i, a]) * mc["scale"]
            e = np.exp(s - s.max())
            out[i, a] = (e / e.sum()) @ v[lo:i + 1, g]
    return out.reshape(T, H * V) @ P["o"].T


# -------------------------------------------------------- gated delta rule
def short_conv_silu(u, taps):
    """u [T, N], taps [N, K], the last column is the current token's."""
    K = taps.shape[1]
    pad = np.concatenate([np.zeros((K - 1, u.shape[1])), u], 0)
    y = sum(pad[j:j + u.shape[0]] * taps[:, j] for j in range(K))
    return y * sigmoid(y)


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def delta_memory(q, k, v, beta, g):
    """One head: decay the rows, correct what the key reads, write, read."""
    S = np.zeros((q.shape[1], v.shape[1]))
    out = np.zeros_like(v)
    for t in range(q.shape[0]):
        S = g[t][:, None] * S
        S = S + np.outer(k[t], beta[t] * (v[t] - S.T @ k[t]))
        out[t] = S.T @ q[t]
    return out


def delta_decay(h, P, H):
    """One decay per head and key channel [T, H, D]."""
    z = softplus((h @ P["a1"].T) @ P["a2"].T + P["dt_bias"])
    z = z.reshape(h.shape[0], H, -1)
    return np.exp(-np.exp(P["A_log"])[:, None] * z)


def gated_delta(h, P, mc, eps):
    H, G, D, V = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    T = h.shape[0]
    q = short_conv_silu(h @ P["q"].T, P["q.conv"]).reshape(T, G, D)
    k = short_conv_silu(h @ P["k"].T, P["k.conv"]).reshape(T, G, D)
    v = short_conv_silu(h @ P["v"].T, P["v.conv"]).reshape(T, H, V)
    q, k = unit(q) / math.sqrt(D), unit(k)
    beta = sigmoid(h @ P["b"].T)
    g = delta_decay(h, P, H)
    o = np.stack([delta_memory(q[:, a // (H // G)], k[:, a // (H // G)],
                               v[:, a], beta[:, a], g[:, a])
                  for a in range(H)], 1)
    o = (rms(o, eps) * P["norm"]).reshape(T, H * V)
    return (o * sigmoid((h @ P["g1"].T) @ P["g2"].T)) @ P["o"].T


def parallel(h, P, mc, eps):
    return (mc["left_scale"] * window_attention(h, under(P, "left."),
                                                mc["left"])
            + mc["right_scale"] * gated_delta(h, under(P, "right."),
                                              mc["right"], eps))


# ------------------------------------------------------------ feed-forward
def dense_ff(h, P):
    return (np.maximum(h @ P["gate"].T, 0.0) * (h @ P["up"].T)) @ P["down"].T


def clamped_ff(h, P, limit):
    g = np.minimum(h @ P["gate"].T, limit)
    u = np.clip(h @ P["up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ P["down"].T


def route(z, correction, top):
    """Chosen experts of one token and their weights."""
    s = np.exp(z - z.max())
    s = s / s.sum()
    chosen = np.argsort(-(s + correction), kind="stable")[:top]
    return chosen, s[chosen]


def moe(h, P, spec):
    r = spec["router"]
    out = np.zeros_like(h)
    z = h @ P["router"].T
    for t in range(h.shape[0]):
        for e, w in zip(*route(z[t], P["correction"], r["top"])):
            x = h[t:t + 1]
            y = x if e >= r["experts"] else clamped_ff(
                x, under(P, f"e{e}."), spec["expert"]["limit"])
            out[t] += w * y[0]
    if spec.get("shared"):
        out += clamped_ff(h, under(P, "shared."), spec["shared"]["limit"])
    return out


# ------------------------------------------------------------------- model
def forward(cfg, W, tokens, layer_out=None):
    """Logits [T, vocab] of one sequence from position 0; ``layer_out`` (a
    list) receives the residual after every layer."""
    W = {k: np.asarray(v, dtype=np.float64) for k, v in W.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    tokens = [int(t) for t in tokens]
    x = W["embed"][tokens] + W["bigram"][
        bigram_rows(tokens, cfg["embedding"]["bigram"])]
    for i, lc in enumerate(cfg["layers"]):
        L = under(W, f"l{i}.")
        h = rms(x, eps) * L["norm1"]
        P = under(L, "mix.")
        mixer = parallel if lc["type"] == "parallel" else mlstm
        y = mixer(h, P, lc["mixer"], eps)
        mlp = lc.get("mlp")
        if mlp is not None:
            P = under(L, "mlp.")
            y = y + (dense_ff(h, P) if mlp["kind"] == "dense"
                     else moe(h, P, mlp))
        x = x + m * y
        if layer_out is not None:
            layer_out.append(x.copy())
    return (rms(x, eps) * W["final.norm"]) @ W["head"].T
