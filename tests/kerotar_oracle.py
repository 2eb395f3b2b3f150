"""Plain, slow implementation of the Kerotar decoder for the tests: one function per mechanism, written from the model's equations in float64 (or
whatever dtype the weights come in).  It shares no code with the package.

Model.  x = scale * E[token], x0 = x.  A layer with norm N:  h = N(x),  x <- x + M(h) + F(h)  (mixer and feed-forward read the same h).  A span of layers
may run several times in a row with the same weights; before its pass t the stream is replaced by  x <- A [x; x0] + s_t  with A [width, 2 width] and one
vector s_t per pass.  Mixers: windowed attention that always keeps the first tokens, with a learned sink; latent attention whose queries pass a latent as
well.  Feed-forwards: a clamped gated MLP, a mixture of silu-gated experts.  Logits: head N(x)."""
import math

import torch


def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotate(t, dims, base):
    """t [T, heads, d], row p at position p: channels i and i + dims / 2 are turned by p * base^(-2 i / dims), channels from dims on stay."""
    out = t.clone()
    half = dims // 2
    for i in range(half):
        step = base ** (-2.0 * i / dims)
        a = torch.arange(t.shape[0], dtype=torch.float64) * step
        c, s = torch.cos(a).to(t.dtype)[:, None], torch.sin(a).to(t.dtype)[:, None]
        u, v = t[:, :, i], t[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def visible(T, window, keep):
    """[T, T] bool: row i sees column j when j <= i and (i - j < window or j < keep); window 0: every j <= i."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    near = (i - j < window) if window > 0 else torch.ones(T, T, dtype=torch.bool)
    return (j <= i) & (near | (j < keep))


def softmax_sink(s, sink=None):
    """Rows of s (-inf where nothing is seen) -> weights; exp(sink) joins the denominator."""
    m = s.max(-1, keepdim=True).values
    if sink is not None:
        m = torch.maximum(m, sink)
    e = torch.exp(s - m)
    den = e.sum(-1, keepdim=True)
    return e / (den if sink is None else den + torch.exp(sink - m))


def attention(h, w, p, mx, eps):
    H, G, d, dv = int(mx["heads"]), int(mx["kv_heads"]), int(mx["dim"]), int(mx["vdim"])
    T = h.shape[0]
    q, k = rms_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps).view(T, H, d), rms_norm(h @ w[p + "k"].T, w[p + "k.norm"], eps).view(T, G, d)
    v = (h @ w[p + "v"].T).view(T, G, dv)
    rot = mx.get("rot") or {}
    if rot.get("dims"):
        q, k = rotate(q, int(rot["dims"]), float(rot["base"])), rotate(k, int(rot["dims"]), float(rot["base"]))
    mask = mx.get("mask") or {}
    see = visible(T, int(mask.get("size") or 0), int(mask.get("keep_first") or 0))
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(H):
        g = i // (H // G)
        s = (q[:, i] @ k[:, g].T) * float(mx["scale"])
        out[:, i] = softmax_sink(s.masked_fill(~see, -math.inf), w[p + "sink"][i]) @ v[:, g]
    return out.reshape(T, H * dv) @ w[p + "o"].T


def latent_attention(h, w, p, mx, eps):
    """Keys and values are written out per head (no absorption)."""
    H, d, dr, dv, R = int(mx["heads"]), int(mx["dim"]), int(mx["rot_dim"]), int(mx["vdim"]), int(mx["kv_rank"])
    T = h.shape[0]
    dims, base = int(mx["rot"]["dims"]), float(mx["rot"]["base"])
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).view(T, H, d + dr)
    qp, qr = q[:, :, :d], rotate(q[:, :, d:], dims, base)
    down = h @ w[p + "dkv"].T
    c = rms_norm(down[:, :R], w[p + "dkv.norm"], eps)
    kr = rotate(down[:, None, R:], dims, base)[:, 0]
    kp, v = (c @ w[p + "uk"].T).view(T, H, d), (c @ w[p + "uv"].T).view(T, H, dv)
    see = visible(T, 0, 0)
    gate = torch.sigmoid(h @ w[p + "g"].T)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(H):
        s = (qp[:, i] @ kp[:, i].T + qr[:, i] @ kr.T) * float(mx["scale"])
        out[:, i] = (softmax_sink(s.masked_fill(~see, -math.inf)) @ v[:, i]) * gate[:, i:i + 1]
    return out.reshape(T, H * dv) @ w[p + "o"].T


def clamped_mlp(h, w, p, limit):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def expert(h, w, p):
    g = h @ w[p + "gate"].T
    return (g * torch.sigmoid(g) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(z, top):
    """Router logits [E] of one token -> (chosen experts, weights): softmax over all experts, the `top` largest, divided by their sum."""
    e = torch.exp(z - z.max())
    s = e / e.sum()
    ids = sorted(range(z.numel()), key=lambda j: (-float(s[j]), j))[:top]
    total = sum(float(s[j]) for j in ids) + 1e-20
    return ids, [float(s[j]) / total for j in ids]


def mixture(h, w, p, mlp):
    z = h @ w[p + "router"].T
    picks = [route(z[t], int(mlp["router"]["top"])) for t in range(h.shape[0])]
    out = torch.zeros_like(h)
    for e in range(int(mlp["router"]["experts"])):
        rows = [t for t, (ids, _) in enumerate(picks) if e in ids]
        if rows:
            wt = torch.tensor([picks[t][1][picks[t][0].index(e)] for t in rows], dtype=h.dtype)
            out[rows] += wt[:, None] * expert(h[rows], w, p + f"e{e}.")
    return out


def inject(x, x0, a, step):
    """A [x; x0] + s."""
    return torch.cat([x, x0], -1) @ a.T + step


def schedule(cfg):
    """[(layer, number of the pass that starts right before it or None)] in the order of the runs."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    span = [(i, t if i == a else None) for t in range(times) for i in range(a, b)]
    return [(i, None) for i in range(a)] + span + [(i, None) for i in range(b, n)]


def forward(cfg, w, tokens, collect=None):
    """Logits [T, vocab] of one sequence run from its start.  collect: receives the stream after every layer run."""
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    x0 = x
    for i, t in schedule(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        if t is not None:
            x = inject(x, x0, w["loop.in"], w["loop.step"][t])
        h = rms_norm(x, w[p + "norm1"], eps)
        y = {"attention": attention, "latent_attention": latent_attention}[L["type"]](h, w, p + "mix.", L["mixer"], eps)
        mlp = L.get("mlp")
        if mlp is not None:
            y = y + (clamped_mlp(h, w, p + "mlp.", float(mlp["limit"])) if mlp["kind"] == "dense" else mixture(h, w, p + "mlp.", mlp))
        x = x + y
        if collect is not None:
            collect.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T
