"""Small random configurations and checkpoints of the Kerotar decoder for the tests (config.json dicts + name -> tensor)."""
import torch


def window_layer(heads=4, kv_heads=2, dim=16, vdim=24, scale=None, window=24, keep=5, rot_dims=8, base=1000.0, mlp=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale,
                                           "mask": {"size": window, "keep_first": keep}, "rot": {"base": base, "dims": rot_dims}}, "mlp": mlp}


def latent_layer(heads=3, dim=16, rot_dim=8, vdim=12, kv_rank=20, q_rank=28, scale=None, base=500.0, mlp=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                                                  "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"base": base, "dims": rot_dim}}, "mlp": mlp}


def dense(ff=40, limit=0.8):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts=6, top=2, ff=40):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def make_config(layers, vocab=96, width=64, eps=1e-5, scale=1.7, loop=None):
    cfg = {"architecture": "Kerotar", "layers": layers, "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale}}
    if loop is not None:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def make_weights(cfg, seed=0):
    """Random float32 tensors under the checkpoint names (values exactly representable in bfloat16)."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    rn = lambda *s, k=1.0, off=0.0: (torch.randn(*s, generator=g) * k + off).bfloat16().float()
    lin = lambda o, i: rn(o, i, k=i ** -0.5)
    gain = lambda n: rn(n, k=0.2, off=1.0)
    w = {"embed": rn(cfg["vocab"], W, k=0.5), "head": lin(cfg["vocab"], W), "final.norm": gain(W)}
    if cfg.get("loop"):
        w["loop.in"], w["loop.step"] = rn(W, 2 * W, k=(2 * W) ** -0.5), rn(cfg["loop"]["times"], W, k=0.5)
    for i, L in enumerate(cfg["layers"]):
        p, mx, mlp = f"l{i}.", L["mixer"], L.get("mlp")
        q = p + "mix."
        w[p + "norm1"] = gain(W)
        H, d, dv = mx["heads"], mx["dim"], mx["vdim"]
        if L["type"] == "attention":
            G = mx["kv_heads"]
            w[q + "q"], w[q + "k"], w[q + "v"], w[q + "o"] = lin(H * d, W), lin(G * d, W), lin(G * dv, W), lin(W, H * dv)
            w[q + "q.norm"], w[q + "k.norm"], w[q + "sink"] = gain(H * d), gain(G * d), rn(H, k=0.7, off=0.5)
        else:
            R, dr, Rq = mx["kv_rank"], mx["rot_dim"], mx["q_rank"]
            w[q + "dq"], w[q + "dq.norm"], w[q + "uq"] = lin(Rq, W), gain(Rq), lin(H * (d + dr), Rq)
            w[q + "dkv"], w[q + "dkv.norm"], w[q + "uk"], w[q + "uv"] = lin(R + dr, W), gain(R), lin(H * d, R), lin(H * dv, R)
            w[q + "g"], w[q + "o"] = lin(H, W), lin(W, H * dv)
        if mlp is not None and mlp["kind"] == "dense":
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = lin(mlp["ff"], W), lin(mlp["ff"], W), lin(W, mlp["ff"])
        elif mlp is not None:
            w[p + "mlp.router"] = rn(mlp["router"]["experts"], W, k=0.3)
            for j in range(mlp["router"]["experts"]):
                ff = mlp["expert"]["ff"]
                w[p + f"mlp.e{j}.gate"], w[p + f"mlp.e{j}.up"], w[p + f"mlp.e{j}.down"] = lin(ff, W), lin(ff, W), lin(W, ff)
    return w


def oracle_logits(cfg, w, tokens, collect=None):
    """float64 logits [T, vocab] of the plain implementation."""
    import kerotar_oracle
    return kerotar_oracle.forward(cfg, {k: v.double() for k, v in w.items()}, tokens, collect)
