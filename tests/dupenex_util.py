"""Small random configurations and checkpoints of the Dupenex decoder for the tests (config.json dicts + name -> tensor)."""
import torch


def delta_layer(heads=4, kv_heads=2, dim=16, vdim=24, conv=4, mlp=None):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": mlp}


def window_side(heads=4, kv_heads=2, dim=16, vdim=24, scale=None, window=24, rot_dims=8, base=1000.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale, "mask": {"size": window},
            "rot": {"base": base, "dims": rot_dims}}


def memory_side(heads=3, dim=16, vdim=20, cap=9.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def parallel_layer(left=None, right=None, mlp=None):
    return {"type": "parallel", "mixer": {"left": left or window_side(), "right": right or memory_side()}, "mlp": mlp}


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=40):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def make_config(layers, vocab=96, width=64, eps=1e-5, streams=3, loop=None):
    cfg = {"architecture": "Dupenex", "layers": layers, "vocab": vocab, "width": width, "norm": {"eps": eps}, "streams": streams}
    if loop is not None:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def make_weights(cfg, seed=0, rank_a=12, rank_g=20):
    """Random float32 tensors under the checkpoint names (values exactly representable in bfloat16)."""
    g = torch.Generator().manual_seed(seed)
    W, S = cfg["width"], cfg["streams"]
    rn = lambda *s, k=1.0, off=0.0: (torch.randn(*s, generator=g) * k + off).bfloat16().float()
    lin = lambda o, i: rn(o, i, k=i ** -0.5)
    gain = lambda n: rn(n, k=0.2, off=1.0)
    w = {"embed": rn(cfg["vocab"], W, k=0.5), "head": lin(cfg["vocab"], W), "final.norm": gain(W)}
    for i, L in enumerate(cfg["layers"]):
        p, mx, mlp = f"l{i}.", L["mixer"], L.get("mlp")
        for q in (1, 2) if mlp is not None else (1,):
            w[p + f"norm{q}"] = gain(W)
            w[p + f"hc{q}.in"], w[p + f"hc{q}.out"] = rn(S, k=0.4, off=1.0 / S), rn(S, k=0.4, off=0.7)
            w[p + f"hc{q}.mix"] = (0.8 * torch.eye(S) + 0.3 * S ** -0.5 * torch.randn(S, S, generator=g)).bfloat16().float()
        if L["type"] == "channel_delta":
            H, G, d, dv, q = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"], p + "mix."
            for n, rows in (("q", G * d), ("k", G * d), ("v", H * dv)):
                w[q + n], w[q + n + ".conv"] = lin(rows, W), rn(rows, mx["conv"], k=mx["conv"] ** -0.5)
            w[q + "b"], w[q + "A_log"], w[q + "dt_bias"] = lin(H, W), rn(H, k=0.7), rn(H * d, k=1.0, off=-1.5)
            w[q + "a1"], w[q + "a2"], w[q + "g1"], w[q + "g2"] = lin(rank_a, W), lin(H * d, rank_a), lin(rank_g, W), lin(H * dv, rank_g)
            w[q + "norm"], w[q + "o"] = gain(dv), lin(W, H * dv)
        else:
            a, q = mx["left"], p + "mix.left."
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            w[q + "q"], w[q + "k"], w[q + "v"], w[q + "g"], w[q + "o"] = lin(H * d, W), lin(G * d, W), lin(G * dv, W), lin(H * dv, W), lin(W, H * dv)
            w[q + "out"] = gain(W)
            b, q = mx["right"], p + "mix.right."
            H, d, dv = b["heads"], b["dim"], b["vdim"]
            w[q + "q"], w[q + "k"], w[q + "v"], w[q + "g"], w[q + "o"] = lin(H * d, W), lin(H * d, W), lin(H * dv, W), lin(H * dv, W), lin(W, H * dv)
            w[q + "i"], w[q + "f"], w[q + "i.b"], w[q + "f.b"] = lin(H, W), lin(H, W), rn(H), rn(H, k=1.0, off=2.0)
            w[q + "norm"], w[q + "out"] = gain(H * dv), gain(W)
        if mlp is not None and mlp["kind"] == "dense":
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = lin(mlp["ff"], W), lin(mlp["ff"], W), lin(W, mlp["ff"])
        elif mlp is not None:
            w[p + "mlp.router"] = rn(mlp["router"]["experts"], W, k=0.3)
            for j in range(mlp["router"]["experts"]):
                w[p + f"mlp.e{j}.up"], w[p + f"mlp.e{j}.down"] = lin(mlp["expert"]["ff"], W), lin(W, mlp["expert"]["ff"])
    return w


def oracle_logits(cfg, w, tokens, collect=None):
    """float64 logits [T, vocab] of the plain implementation."""
    import dupenex_oracle
    return dupenex_oracle.forward(cfg, {k: v.double() for k, v in w.items()}, tokens, collect)
