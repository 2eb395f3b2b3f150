"""Plain, slow implementation of the Dupenex decoder for the tests: one function per mechanism, written from the model's equations in
float64 (or whatever dtype the weights come in), token by token where the model is sequential.  It shares no code with the package.

Model.  The residual is carried by S parallel streams X_1 .. X_S, all equal to the embedding row at the start.  A sublayer f with its norm N
reads one weighted sum of them and writes back to all:  y = f(N(sum_s a[s] X_s)),  X_t <- sum_s M[s, t] X_s + b[t] y,  with a, b, M learned
per layer and sublayer (a mixer, then a feed-forward).  Mixers: a delta-rule recurrence with a decay per key channel behind short
convolutions; windowed attention with an elementwise output gate side by side with a matrix memory under exponential gates.  A span of
layers may run several times in a row with the same weights.  Logits: head @ N(sum_s X_s)."""
import math

import torch


# ------------------------------------------------------------------------------------------------ norms and activations
def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def unit(x, eps=1e-6):
    """x / sqrt(sum(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def log_sigmoid(z):
    return -softplus(-z)


# ------------------------------------------------------------------------------------------------ residual streams
def stream_read(X, a):
    """X [S, T, W], a [S] -> [T, W]."""
    out = torch.zeros_like(X[0])
    for s in range(X.shape[0]):
        out = out + a[s] * X[s]
    return out


def stream_write(X, M, b, y):
    """X_t <- sum_s M[s, t] X_s + b[t] y, every new stream from the old ones."""
    S = X.shape[0]
    new = []
    for t in range(S):
        acc = b[t] * y
        for s in range(S):
            acc = acc + M[s, t] * X[s]
        new.append(acc)
    return torch.stack(new)


# ------------------------------------------------------------------------------------------------ short convolution
def short_conv(x, w, history=None):
    """x [T, C], w [C, taps]: out[t, c] = silu(sum_j w[c, j] x[t - (taps - 1) + j, c]), zeros (or `history` [taps - 1, C]) before the first row."""
    T, C = x.shape
    taps = w.shape[1]
    pad = torch.zeros(taps - 1, C, dtype=x.dtype) if history is None else history
    full = torch.cat([pad, x], 0)
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            out[t] = out[t] + w[:, j] * full[t + j]
    return silu(out)


# ------------------------------------------------------------------------------------------------ delta rule with a decay per key channel
def delta_step(S, q, k, v, g, beta):
    """One token of one head: S [d, dv] -> (new S, o).  The rows of S decay by g, the value that k reads out is moved by beta towards v, q
    reads the new S."""
    S = g[:, None] * S
    u = beta * (v - S.T @ k)
    S = S + torch.outer(k, u)
    return S, S.T @ q


def channel_delta(h, w, p, mx, eps):
    """h [T, W] -> [T, W]."""
    H, G, d, dv = int(mx["heads"]), int(mx["kv_heads"]), int(mx["dim"]), int(mx["vdim"])
    T = h.shape[0]
    q = unit(short_conv(h @ w[p + "q"].T, w[p + "q.conv"]).view(T, G, d)) * d ** -0.5
    k = unit(short_conv(h @ w[p + "k"].T, w[p + "k.conv"]).view(T, G, d))
    v = short_conv(h @ w[p + "v"].T, w[p + "v.conv"]).view(T, H, dv)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    pre = ((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"].reshape(-1)).view(T, H, d)
    gate = torch.sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).view(T, H, dv)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(H):
        j = i // (H // G)
        S = torch.zeros(d, dv, dtype=h.dtype)
        rate = torch.exp(w[p + "A_log"].reshape(-1)[i])
        for t in range(T):
            g = torch.exp(-rate * softplus(pre[t, i]))
            S, o = delta_step(S, q[t, j], k[t, j], v[t, i], g, beta[t, i])
            out[t, i] = rms_norm(o, w[p + "norm"], eps) * gate[t, i]
    return out.reshape(T, H * dv) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------------ windowed attention
def rotate(vec, position, dims, base):
    """Turn the first `dims` channels of one head's vector: channel 2i is paired with 2i + 1 and turned by position * base^(-2i / dims)."""
    out = vec.clone()
    for i in range(dims // 2):
        a = position * base ** (-2.0 * i / dims)
        c, s = math.cos(a), math.sin(a)
        u, v = vec[2 * i], vec[2 * i + 1]
        out[2 * i] = u * c - v * s
        out[2 * i + 1] = v * c + u * s
    return out


def window_attention(h, w, p, mx):
    H, G, d, dv = int(mx["heads"]), int(mx["kv_heads"]), int(mx["dim"]), int(mx["vdim"])
    T = h.shape[0]
    q, k, v = (h @ w[p + "q"].T).view(T, H, d), (h @ w[p + "k"].T).view(T, G, d), (h @ w[p + "v"].T).view(T, G, dv)
    rot = mx.get("rot") or {}
    dims = int(rot.get("dims") or 0)
    if dims:
        base = float(rot["base"])
        q = torch.stack([torch.stack([rotate(q[t, i], t, dims, base) for i in range(H)]) for t in range(T)])
        k = torch.stack([torch.stack([rotate(k[t, i], t, dims, base) for i in range(G)]) for t in range(T)])
    window = int((mx.get("mask") or {}).get("size") or 0)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(H):
        j = i // (H // G)
        for t in range(T):
            lo = max(0, t - window + 1) if window > 0 else 0
            s = (k[lo:t + 1, j] @ q[t, i]) * float(mx["scale"])
            e = torch.exp(s - s.max())
            out[t, i] = (e[:, None] * v[lo:t + 1, j]).sum(0) / e.sum()
    return (out.reshape(T, H * dv) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------------ matrix memory under exponential gates
def memory_step(S, n, m, q, k, v, i, f):
    """One token of one head with log gates i and f, kept in range by the running maximum m -> (S, n, m, o)."""
    mn = max(f + m, i)
    keep, take = math.exp(f + m - mn), math.exp(i - mn)
    S = keep * S + take * torch.outer(k, v)
    n = keep * n + take * k
    return S, n, mn, (S.T @ q) / (max(abs(float(n @ q)), math.exp(-mn)) + 1e-6)


def matrix_memory(h, w, p, mx, eps):
    H, d, dv, cap = int(mx["heads"]), int(mx["dim"]), int(mx["vdim"]), float(mx["gate_cap"])
    T = h.shape[0]
    q, k, v = (h @ w[p + "q"].T).view(T, H, d) * d ** -0.5, (h @ w[p + "k"].T).view(T, H, d), (h @ w[p + "v"].T).view(T, H, dv)
    li = cap * torch.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    lf = log_sigmoid(cap * torch.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for a in range(H):
        S, n, m = torch.zeros(d, dv, dtype=h.dtype), torch.zeros(d, dtype=h.dtype), 0.0
        for t in range(T):
            S, n, m, o = memory_step(S, n, m, q[t, a], k[t, a], v[t, a], float(li[t, a]), float(lf[t, a]))
            out[t, a] = o / torch.sqrt((o * o).mean() + eps)
    return (out.reshape(T, H * dv) * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(h, w, p, mx, eps):
    a = window_attention(h, w, p + "left.", mx["left"])
    b = matrix_memory(h, w, p + "right.", mx["right"], eps)
    return 0.5 * (rms_norm(a, w[p + "left.out"], eps) + rms_norm(b, w[p + "right.out"], eps))


# ------------------------------------------------------------------------------------------------ feed-forwards
def dense(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def expert(h, up, down):
    z = torch.clamp(h @ up.T, min=0.0)
    return (z * z) @ down.T


def route(z, top):
    """Router logits [E] of one token -> (chosen experts, their weights): the `top` largest logits, softmax over those alone."""
    ids = sorted(range(z.numel()), key=lambda e: (-float(z[e]), e))[:top]
    e = torch.exp(z[ids] - z[ids].max())
    return ids, [float(x) for x in e / e.sum()]


def mixture(h, w, p, mlp):
    z = h @ w[p + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        ids, wts = route(z[t], int(mlp["router"]["top"]))
        for e, a in zip(ids, wts):
            out[t] += a * expert(h[t:t + 1], w[p + f"e{e}.up"], w[p + f"e{e}.down"])[0]
    return out


# ------------------------------------------------------------------------------------------------ the model
def layer_runs(cfg):
    """The layers in the order they run: the span of `loop` as often as it says."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    return list(range(a)) + list(range(a, b)) * times + list(range(b, n))


def forward(cfg, w, tokens, collect=None):
    """Logits [T, vocab] of one sequence run from its start.  collect: receives the sum of the streams after every layer run."""
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    X = torch.stack([x.clone() for _ in range(int(cfg["streams"]))])
    for i in layer_runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        h = rms_norm(stream_read(X, w[p + "hc1.in"]), w[p + "norm1"], eps)
        y = {"channel_delta": channel_delta, "parallel": parallel}[L["type"]](h, w, p + "mix.", L["mixer"], eps)
        X = stream_write(X, w[p + "hc1.mix"], w[p + "hc1.out"], y)
        mlp = L.get("mlp")
        if mlp is not None:
            h = rms_norm(stream_read(X, w[p + "hc2.in"]), w[p + "norm2"], eps)
            y = dense(h, w, p + "mlp.") if mlp["kind"] == "dense" else mixture(h, w, p + "mlp.", mlp)
            X = stream_write(X, w[p + "hc2.mix"], w[p + "hc2.out"], y)
        if collect is not None:
            collect.append(X.sum(0))
    return rms_norm(X.sum(0), w["final.norm"], eps) @ w["head"].T
