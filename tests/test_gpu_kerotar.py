"""The Kerotar member of the hybrid family on the GPU against the plain implementation in kerotar_oracle (float64, CPU): single operations, every
mechanism alone in many shapes, layer loops, whole prompts against token-by-token decoding, portions down to two tokens, unequal batches, reused pages
and slots, keys just inside / just outside the window, the last kept and the first dropped of the first tokens and keys at page borders with weights built
so that they dominate, a sink that takes most of the weight, long decoding, split decode rows, graph replay, and greedy generation through the scheduler
and the command line."""
import json
import math
import os
import subprocess
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import kerotar_oracle as O  # noqa: E402
import kerotar_util as U  # noqa: E402

pytestmark = pytest.mark.gpu
DEV = "cuda:0"


def engine(cfg, w, dtype=torch.float32, max_tokens=1024, max_seqs=4, **kw):
    from rtp_llm_amd.hybrid import HybridConfig, HybridModel
    from rtp_llm_amd.scheduler import ServingEngine
    return ServingEngine(HybridModel(HybridConfig.from_json(cfg), w, dtype, DEV), max_tokens=max_tokens, max_seqs=max_seqs, **kw)


def toks(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def close(got, ref, tol):
    err = float((got.double().cpu() - ref).abs().max())
    assert err <= tol, f"max |error| {err} > {tol}"


def bf16_close(got, ref, median=0.04, tail=0.08):
    """Row by row: rounding to 16 bits moves a row's logits by a few per cent of their size."""
    d = got.double().cpu() - ref
    rel = d.pow(2).mean(-1).sqrt() / ref.pow(2).mean(-1).sqrt()
    assert float(rel.median()) < median and float(rel.quantile(0.9)) < tail, f"bf16 step is off by more than rounding: median {float(rel.median())}, 90% {float(rel.quantile(0.9))}"


def whole(eng, t, sid="s"):
    out = eng.run_step([(sid, t, range(len(t)))])
    eng.release(sid)
    return out


def I(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


# head sizes of 32 and value sizes of 16 (latent rows are padded to 32): prompts take the matrix-core attention in bf16; the others the row kernel
FULL = [U.window_layer(mlp=U.dense()), U.latent_layer(mlp=U.moe()), U.window_layer(heads=2, kv_heads=1, dim=32, vdim=16, window=40, keep=3, rot_dims=32, mlp=U.moe(experts=5, top=3)),
        U.latent_layer(heads=2, dim=8, rot_dim=4, vdim=16, kv_rank=16, q_rank=12, mlp=U.dense(33, limit=2.0))]
LOOP = (1, 3, 3)
NO_ROUTER = [U.window_layer(heads=4, kv_heads=2, dim=32, vdim=48, window=20, keep=9, mlp=U.dense()), U.latent_layer(kv_rank=32, mlp=U.dense(24)),
             U.window_layer(heads=3, kv_heads=3, mlp=None)]


# ------------------------------------------------------------------------------------------------ single operations
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W", [64, 50])
def test_stream_rounded_beside_the_embedding_output(dtype, W):
    """The operand of the linear in front of a pass: [stream with its last branches | embedding rows], both rounded from fp32."""
    from rtp_llm_amd import hybrid_ops as hops
    g = torch.Generator().manual_seed(W)
    T, top = 13, 3
    table = torch.randn(20, W, generator=g).to(dtype).to(DEV)
    ids = I([i % 20 for i in range(T)])
    pair = torch.full((T, 2 * W), 7.0, dtype=dtype, device=DEV)
    x, cp = hops.embed_scaled(ids, table, 1.25, copy=pair[:, W:])
    emb = table.double().cpu()[ids.cpu().long()] * 1.25
    close(x, emb, 1e-6)
    assert torch.equal(pair[:, W:], x.to(dtype)) and torch.equal(pair[:, :W], torch.full_like(pair[:, :W], 7.0)) and cp.data_ptr() == pair[:, W:].data_ptr()
    x0 = x.to(dtype).clone()
    a, y = torch.randn(T, W, generator=g).to(DEV), torch.randn(T * top, W, generator=g).to(DEV)
    wts, place = torch.rand(T, top, generator=g).to(DEV), torch.randperm(T * top, generator=g).int().to(DEV)
    extra = torch.randn(T, W, generator=g).to(DEV)
    ref = emb + a.double().cpu() + extra.double().cpu() + (wts.double().cpu()[..., None] * y.double().cpu()[place.cpu().long()].view(T, top, W)).sum(1)
    hops.residual_round(x, a, hops.MoeSum(y, place, wts, extra), 1.0, pair[:, :W])
    close(x, ref, 1e-5)
    assert torch.equal(pair[:, :W], x.to(dtype)) and torch.equal(pair[:, W:], x0)
    before = x.clone()
    hops.residual_round(x, None, None, 1.0, pair[:, :W])                 # nothing to add: the stream stays
    assert torch.equal(x, before)


def test_norm_over_columns_of_a_wider_buffer():
    from rtp_llm_amd import hybrid_ops as hops
    for n, ld in ((7, 20), (64, 100), (300, 301)):
        x = torch.randn(9, ld, generator=torch.Generator().manual_seed(n)).to(DEV)
        w = torch.randn(n, generator=torch.Generator().manual_seed(n + 1)).to(DEV)
        close(hops.head_norm(x[:, 2:2 + n] if ld >= n + 2 else x[:, 1:1 + n], 1, n, w, 1e-3),
              O.rms_norm((x[:, 2:2 + n] if ld >= n + 2 else x[:, 1:1 + n]).double().cpu(), w.double().cpu(), 1e-3), 1e-5)


@pytest.mark.parametrize("layout", ["interleaved", "halves"])
def test_latent_rows_with_queries_from_a_buffer_of_their_own(layout):
    """Both pair layouts, a span shorter than the rotated part, queries beside the down projection and in a tensor of their own."""
    from rtp_llm_amd import hybrid_ops as hops
    g = torch.Generator().manual_seed(3)
    T, H, d, dr, R, span, page = 11, 3, 10, 8, 21, 6, 4
    dpad = 32
    q, down = torch.randn(T, H * (d + dr), generator=g), torch.randn(T, R + dr, generator=g)
    cw = torch.rand(R, generator=g) + 0.5
    freq = torch.tensor([50.0 ** (-2.0 * i / span) for i in range(span // 2)])
    pos = list(range(T))
    geom = hops.latent_geometry(H, d, dr, R, dpad, span, page, 8, 5)
    bt = I([3, 0, 4, 0, 0, 0, 0, 0]).view(1, 8)

    def turn(t):                                                          # [T, heads, dr]
        if layout == "halves":
            return O.rotate(t, span, 50.0)
        perm = list(range(0, span, 2)) + list(range(1, span, 2)) + list(range(span, dr))
        out = torch.empty_like(t)
        out[:, :, perm] = O.rotate(t[:, :, perm], span, 50.0)
        return out
    qr = turn(q.double().view(T, H, d + dr)[:, :, d:])
    row = torch.cat([O.rms_norm(down.double()[:, :R], cw.double(), 1e-5), turn(down.double()[:, None, R:])[:, 0], torch.zeros(T, dpad - R - dr, dtype=torch.float64)], 1)
    for own in (True, False):
        qn, qabs = torch.zeros(T, H * d, device=DEV), torch.zeros(T, H * dpad, device=DEV)
        cache = torch.zeros(5, page, dpad, device=DEV)
        wide = torch.cat([q, torch.zeros(T, 3), down, torch.zeros(T, 2)], 1).to(DEV)
        proj, off = (torch.cat([torch.zeros(T, 5), down], 1).to(DEV), 5) if own else (wide, q.shape[1] + 3)
        hops.latent_prep(proj, off, geom, freq.to(DEV), 1.0, cw.to(DEV), 1e-5, I(pos), I([0] * T), bt, qn, qabs, cache, q=q.to(DEV) if own else None, layout=hops.LAYOUTS[layout])
        assert torch.equal(qn.cpu().view(T, H, d), q.view(T, H, d + dr)[:, :, :d])
        close(qabs.view(T, H, dpad)[:, :, R:R + dr], qr, 1e-5)
        close(cache[[3, 0, 4]].view(-1, dpad)[:T], row, 1e-5)
        assert float(cache[[1, 2]].abs().max()) == 0.0


@pytest.mark.parametrize("H,G,d,dv", [(4, 2, 32, 16), (2, 2, 128, 48), (4, 1, 64, 64), (3, 1, 20, 12), (1, 1, 256, 160), (4, 1, 160, 32), (4, 2, 64, 192)])
@pytest.mark.parametrize("window,keep", [(40, 20), (70, 0), (0, 9), (1, 1), (5, 64), (33, 65), (64, 31), (32, 32), (3, 33), (100, 400)])
def test_window_with_kept_first_tokens(H, G, d, dv, window, keep):
    """Both attention kernels over scattered pages: a whole prompt, a portion in the middle, and rows far behind the kept tokens; with a sink and head gates."""
    from rtp_llm_amd import hybrid_ops as hops
    g = torch.Generator().manual_seed(window + keep)
    T, pages = 170, [4, 0, 2]
    q = torch.randn(T, H * d, generator=g)
    K, V = torch.randn(T, G, d, generator=g).bfloat16(), torch.randn(T, G, dv, generator=g).bfloat16()
    sink, gate = torch.randn(H, generator=g), torch.randn(T, H + 2, generator=g)
    see = O.visible(T, window, keep)
    ref = torch.zeros(T, H, dv, dtype=torch.float64)
    for h in range(H):
        s = (q.double().view(T, H, d)[:, h] @ K.double()[:, h // (H // G)].T) * d ** -0.5
        ref[:, h] = (O.softmax_sink(s.masked_fill(~see, -math.inf), sink[h].double()) @ V.double()[:, h // (H // G)]) * torch.sigmoid(gate[:, 1 + h:2 + h].double())
    geom = hops.attn_geometry(H, G, d, dv, 0, 0, 0, 64, 8, 5)
    bt = I(pages + [0] * 5).view(1, 8)
    for dtype in (torch.float32, torch.bfloat16):
        kc, vc = torch.zeros(5, G, 64, d, dtype=dtype), torch.zeros(5, G, 64, dv, dtype=dtype)
        for t in range(T):
            kc[pages[t // 64], :, t % 64], vc[pages[t // 64], :, t % 64] = K[t].to(dtype), V[t].to(dtype)
        for a, b in ((0, T), (37, 91), (128, 129), (150, 170)):
            n = b - a
            args = (I(list(range(a, b))), I([0] * n), bt)
            kw = dict(window=window, keep=keep, out_gate=gate[a:b, 1:1 + H].to(DEV))
            tol = 2e-5 if dtype == torch.float32 else 0.02
            qd = q[a:b].to(DEV)
            close(hops.attn_rows(qd, d ** -0.5, geom, 0, sink.to(DEV), None, *args, kc.to(DEV), vc.to(DEV), H, dv, **kw).view(n, H, dv), ref[a:b], tol)
            if hops.attn_tiles_supported(dtype, d, dv, False, 0):
                t0 = list(range(0, n, 16))
                close(hops.attn_tiles(qd, d ** -0.5, geom, 0, sink.to(DEV), None, *args, I(t0), I([min(16, n - x) for x in t0]), kc.to(DEV), vc.to(DEV), H, dv, **kw).view(n, H, dv),
                      ref[a:b], tol)


@pytest.mark.parametrize("E,top", [(8, 4), (6, 6), (5, 1), (70, 9)])
def test_router_weights_are_scores_over_their_sum(E, top):
    from rtp_llm_amd import hybrid_ops as hops
    z = torch.randn(21, E, generator=torch.Generator().manual_seed(E)) * 2.0
    ids, wts = hops.moe_route_sorted(z.to(DEV), E, 1, 1, top, chosen=True)[:2]
    for t in range(21):
        ri, rw = O.route(z[t].double(), top)
        assert ids[t].cpu().tolist() == ri
        close(wts[t], torch.tensor(rw, dtype=torch.float64), 1e-6)


# ------------------------------------------------------------------------------------------------ mechanisms alone
ALONE = {
    "window": (U.window_layer(), {}),
    "window of one": (U.window_layer(window=1, keep=2), {}),
    "nothing kept": (U.window_layer(window=9, keep=0), {}),
    "one kept": (U.window_layer(window=7, keep=1), {}),
    "more kept than the window": (U.window_layer(window=5, keep=17), {}),
    "everything kept": (U.window_layer(window=5, keep=400), {}),
    "window past the sequence": (U.window_layer(window=400, keep=3), {}),
    "no mask": (U.window_layer(window=0, keep=0), {}),
    "one head": (U.window_layer(heads=1, kv_heads=1), {}),
    "heads of their own": (U.window_layer(heads=3, kv_heads=3), {}),
    "one key head": (U.window_layer(heads=5, kv_heads=1, dim=12, vdim=7), {}),
    "whole head turned": (U.window_layer(dim=20, rot_dims=20), {}),
    "nothing turned": (U.window_layer(rot_dims=0), {}),
    "wide head": (U.window_layer(heads=2, kv_heads=1, dim=160, vdim=136), {}),
    "latent": (U.latent_layer(), {}),
    "latent one head": (U.latent_layer(heads=1), {}),
    "latent odd sizes": (U.latent_layer(heads=3, dim=13, rot_dim=6, vdim=9, kv_rank=19, q_rank=11), {}),
    "latent wide": (U.latent_layer(heads=2, dim=40, rot_dim=32, vdim=56, kv_rank=224, q_rank=200), {}),
    "latent wider than the matrix cores take": (U.latent_layer(heads=2, dim=24, rot_dim=16, vdim=20, kv_rank=300), {}),
    "latent rank of one": (U.latent_layer(kv_rank=1, q_rank=1), {}),
    "latent scale": (U.latent_layer(scale=0.9), {}),
    "dense": (U.window_layer(mlp=U.dense(56, limit=0.3)), {}),
    "dense wide limit": (U.latent_layer(mlp=U.dense(31, limit=50.0)), {}),
    "mixture": (U.latent_layer(mlp=U.moe()), {}),
    "mixture in a window layer": (U.window_layer(mlp=U.moe(experts=7, top=4, ff=33)), {}),
    "one expert": (U.latent_layer(mlp=U.moe(experts=1, top=1)), {}),
    "all experts": (U.latent_layer(mlp=U.moe(experts=4, top=4)), {}),
    "embedding scale": (U.window_layer(mlp=U.dense()), {"scale": 11.0}),
    "embedding scale of one": (U.latent_layer(mlp=U.dense()), {"scale": 1.0}),
    "large eps": (U.latent_layer(mlp=U.dense()), {"eps": 0.3}),
    "large eps window": (U.window_layer(mlp=U.dense()), {"eps": 0.3}),
    "loop of one pass": (U.window_layer(mlp=U.dense()), {"loop": (0, 1, 1)}),
}


@pytest.mark.parametrize("name", sorted(ALONE))
def test_one_layer_models(name):
    layer, kw = ALONE[name]
    cfg = U.make_config([layer], vocab=80, width=48, **kw)
    w = U.make_weights(cfg, seed=3)
    t = toks(70, 80, 4)
    col, ocol = [], []
    ref = U.oracle_logits(cfg, w, t, ocol)
    eng = engine(cfg, w)
    got = eng.run_step([("x", t, range(len(t)))], collect=col)
    close(col[0], ocol[0], 3e-4)
    close(got, ref, 3e-4)
    eng.release("x")
    one = torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[:30]])       # and token by token from the first token on
    close(one, ref[:30], 3e-4)


def test_other_widths_and_constants():
    """Widths that are no multiple of four or eight, another eps."""
    for width in (50, 36, 130):
        cfg = U.make_config([U.window_layer(window=11, mlp=U.moe(ff=33)), U.latent_layer(mlp=U.dense(30))], vocab=61, width=width, eps=1e-3, loop=(0, 2, 2))
        w = U.make_weights(cfg, seed=width)
        t = toks(40, 61, width)
        ref = U.oracle_logits(cfg, w, t)
        eng = engine(cfg, w)
        close(whole(eng, t), ref, 3e-4)
        eng.run_step([("d", t[:25], [])])
        close(torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[25:]]), ref[25:], 3e-4)
        eng = engine(cfg, w, torch.bfloat16)                                # odd row lengths in 16 bits run (routers may turn close calls over)
        assert torch.isfinite(whole(eng, t)).all()


@pytest.mark.parametrize("loop", [None, (0, 1, 1), (0, 4, 2), (1, 2, 3), (3, 4, 2), (1, 3, 1), (2, 4, 3)])
def test_layer_loops(loop):
    """A span at the start, in the middle, at the end, the whole stack, once; every run keeps keys of its own and every pass takes in the embedding."""
    cfg = U.make_config(FULL, width=48, loop=loop)
    w = U.make_weights(cfg, seed=4)
    t = toks(60, cfg["vocab"], 5)
    col, ocol = [], []
    ref = U.oracle_logits(cfg, w, t, ocol)
    eng = engine(cfg, w)
    got = eng.run_step([("x", t, range(len(t)))], collect=col)
    assert len(col) == len(ocol) == len(O.schedule(cfg))
    for a, b in zip(col, ocol):
        close(a / b.abs().max().to(DEV), b / b.abs().max(), 2e-4)
    close(got, ref, 5e-4)
    eng.run_step([("d", t[:37], [])])
    close(torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[37:]]), ref[37:], 5e-4)


def test_all_mechanisms_together_and_bf16():
    cfg = U.make_config(FULL, loop=LOOP)
    w = U.make_weights(cfg, seed=5)
    t = toks(90, cfg["vocab"], 6)
    ref = U.oracle_logits(cfg, w, t)
    close(whole(engine(cfg, w), t), ref, 5e-4)
    cfg = U.make_config(NO_ROUTER, loop=LOOP)
    w = U.make_weights(cfg, seed=5)
    ref = U.oracle_logits(cfg, w, t)
    for tiles in (True, False):                                    # prompt attention on the matrix cores and on the row kernel
        eng = engine(cfg, w, torch.bfloat16)
        for L, mixer, *_ in eng.model.layers:
            mixer.use_tiles = tiles
        bf16_close(whole(eng, t), ref)
        eng.run_step([("d", t[:60], [])])
        bf16_close(torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[60:]]), ref[60:])


def test_every_part_of_the_model_matters():
    """The oracle itself: changing a constant, or a tensor of the kind that is easily left out, moves the logits, so a part the engine lost would show in
    the comparisons above."""
    cfg = U.make_config(FULL[:2], loop=(0, 2, 2))
    w = U.make_weights(cfg, seed=7)
    t = toks(40, cfg["vocab"], 8)
    ref = U.oracle_logits(cfg, w, t)
    moved = lambda c, ww: float((U.oracle_logits(c, ww, t) - ref).abs().max())
    for name in ("loop.in", "l0.norm1", "l0.mix.q.norm", "l0.mix.k.norm", "l0.mix.sink", "l1.mix.dq.norm", "l1.mix.dkv.norm", "l1.mix.uq", "l1.mix.uk", "l1.mix.g", "l1.mlp.router",
                 "final.norm"):
        w2 = dict(w); w2[name] = w[name] * 0.5 + 0.1
        assert moved(cfg, w2) > 0.01, name
    w2 = dict(w); w2["loop.step"] = w["loop.step"].flip(0)               # which vector belongs to which pass
    assert moved(cfg, w2) > 0.01
    w2 = dict(w); W = cfg["width"]; w2["loop.in"] = torch.cat([w["loop.in"][:, W:], w["loop.in"][:, :W]], 1)
    assert moved(cfg, w2) > 0.01
    for path, val in ((("layers", 0, "mixer", "mask", "size"), 5), (("layers", 0, "mixer", "mask", "keep_first"), 4), (("layers", 0, "mixer", "scale"), 0.6),
                      (("layers", 0, "mixer", "rot", "base"), 10.0), (("layers", 0, "mixer", "rot", "dims"), 4), (("layers", 1, "mixer", "rot", "base"), 10.0),
                      (("layers", 0, "mlp", "limit"), 0.4), (("layers", 1, "mlp", "router", "top"), 3), (("embedding", "scale"), 1.0), (("loop", "start"), 1), (("loop", "stop"), 1)):
        c2 = json.loads(json.dumps(cfg))
        node = c2
        for key in path[:-1]:
            node = node[key]
        node[path[-1]] = val
        assert moved(c2, w) > 0.01, path


# ------------------------------------------------------------------------------------------------ schedules
def test_prefill_against_token_by_token_and_first_tokens():
    cfg = U.make_config(FULL, loop=LOOP)
    w = U.make_weights(cfg, seed=9)
    t = toks(100, cfg["vocab"], 10)
    ref = U.oracle_logits(cfg, w, t)
    eng = engine(cfg, w)
    close(whole(eng, t), ref, 5e-4)
    one = torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t])
    eng.release("d")
    close(one, ref, 5e-4)
    for n in (1, 2, 3):                                            # the shortest sequences
        close(whole(eng, t[:n]), ref[:n], 5e-4)


@pytest.mark.parametrize("sizes", [[2] * 40, [33, 2, 31, 5, 64, 1, 1, 2, 60], [63, 1, 64, 65, 6], [1, 198], [23, 1, 24, 25, 47, 70], [3, 2, 2, 130, 2, 1, 62], [5, 19, 1, 40, 3]])
def test_portions(sizes):
    n = sum(sizes)
    for layers, dtype in ((FULL, torch.float32), (NO_ROUTER, torch.bfloat16)):
        cfg = U.make_config(layers, loop=LOOP)
        w = U.make_weights(cfg, seed=11)
        t = toks(n, cfg["vocab"], 12)
        ref = U.oracle_logits(cfg, w, t)
        eng = engine(cfg, w, dtype)
        at, outs = 0, []
        for s in sizes:
            outs.append(eng.run_step([("p", t[at:at + s], range(s))]))
            at += s
        if dtype == torch.float32:
            close(torch.cat(outs), ref, 5e-4)
        else:
            bf16_close(torch.cat(outs), ref)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 5e-4), (torch.bfloat16, None)])
def test_unequal_batches_reused_pages_and_slots(dtype, tol):
    cfg = U.make_config(FULL if tol is not None else NO_ROUTER, loop=LOOP)
    w = U.make_weights(cfg, seed=13)
    lens = {"a": 150, "b": 9, "c": 70, "d": 131, "e": 64, "f": 40}
    seqs = {k: toks(n, cfg["vocab"], 20 + i) for i, (k, n) in enumerate(lens.items())}
    ref = {k: U.oracle_logits(cfg, w, v) for k, v in seqs.items()}
    # pool: 7 pages of 64 and 3 slots -- less than the requests need together, so pages and slots come back and go out again
    eng = engine(cfg, w, dtype, max_tokens=7 * 64, max_seqs=3)
    plan = [
        [("a", 100), ("b", 4)],
        [("a", 1), ("b", 1), ("c", 30)],
        [("b", 4), ("c", 40), ("a", 49)],            # a, b, c complete -> released
        [("d", 2), ("e", 64)],
        [("d", 129), ("f", 3)],                      # d, e complete
        [("f", 1)], [("f", 36)],
    ]
    at = {k: 0 for k in seqs}
    got = {k: [] for k in seqs}
    for step in plan:
        entries = [(k, seqs[k][at[k]:at[k] + n], range(n)) for k, n in step]
        out = eng.run_step(entries)
        o = 0
        for k, n in step:
            got[k].append(out[o:o + n]); o += n; at[k] += n
            if at[k] == lens[k]:
                eng.release(k)
    assert eng.cache.pages.free == 7 and eng.cache.slots.free == 3
    for k in seqs:
        if tol is not None:
            close(torch.cat(got[k]), ref[k], tol)
        else:                                        # rounding to 16 bits costs a request in a batch what it costs alone
            off = lambda x: float((x.double().cpu() - ref[k]).pow(2).mean().sqrt() / ref[k].pow(2).mean().sqrt())
            alone = off(whole(eng, seqs[k]))
            assert off(torch.cat(got[k])) < 1.5 * alone + 0.02 and alone < 0.15, (k, off(torch.cat(got[k])), alone)
    with pytest.raises(MemoryError):
        eng.run_step([("big", toks(8 * 64, cfg["vocab"], 1), [])])


# ------------------------------------------------------------------------------------------------ one key that dominates: page borders, window edges, kept tokens
def _axes(cfg, seed):
    """Weights and embeddings in which token 1 (the beacon) lives on axis 0 alone, token 2 (the asker) on axis 1 alone and every other token on neither."""
    w = U.make_weights(cfg, seed=seed)
    w["l0.norm1"].fill_(1.0)
    e = torch.randn(cfg["vocab"], cfg["width"], generator=torch.Generator().manual_seed(seed + 1))
    e[:, :2] = 0.0
    e[1], e[2] = 0.0, 0.0
    e[1, 0], e[2, 1] = 1.0, 1.0
    w["embed"] = e
    return w


def _window_beacon(window, keep, heads=2, kv_heads=1, dim=32, vdim=16):
    """The key of the beacon and the query of the asker meet in one unrotated channel that every other token leaves empty: the asker's score for the
    beacon stands out by about ten, and the beacon's value is far from the others'."""
    cfg = U.make_config([U.window_layer(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, rot_dims=8, window=window, keep=keep, scale=1.0)], vocab=40, width=32)
    w = _axes(cfg, 17)
    p, c = "l0.mix.", dim - 1                            # the channel: beyond the rotary span
    for n in ("q", "k"):
        w[p + n] *= 0.3
        w[p + n + ".norm"].fill_(0.4)
    for j in range(kv_heads):
        w[p + "k"][j * dim + c] = 0.0
        w[p + "k"][j * dim + c, 0] = 2.0
    for h in range(heads):
        w[p + "q"][h * dim + c] = 0.0
        w[p + "q"][h * dim + c, 1] = 2.0
    w[p + "sink"].fill_(-1.0)
    w[p + "v"][:, 0] = 3.0 * torch.randn(kv_heads * vdim, generator=torch.Generator().manual_seed(19))
    return cfg, {k: v.bfloat16().float() for k, v in w.items()}


def _latent_beacon(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=24, q_rank=20):
    """The same for latent attention: the beacon's latent is nearly one-hot on channel 0, the asker's query latent on channel 1; the absorbed product of the
    two stands out."""
    cfg = U.make_config([U.latent_layer(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=1.0)], vocab=40, width=32)
    w = _axes(cfg, 27)
    p = "l0.mix."
    for n in ("dq", "dkv", "uq", "uk"):
        w[p + n] *= 0.15
    w[p + "dkv.norm"].fill_(1.0); w[p + "dq.norm"].fill_(1.0)
    w[p + "dkv"][0] = 0.0; w[p + "dkv"][0, 0] = 4.0
    w[p + "dq"][1] = 0.0; w[p + "dq"][1, 1] = 4.0
    w[p + "g"].zero_()
    for h in range(heads):
        w[p + "uk"][h * dim] = 0.0; w[p + "uk"][h * dim, 0] = 1.0
        w[p + "uq"][h * (dim + rot_dim)] = 0.0; w[p + "uq"][h * (dim + rot_dim), 1] = 12.0 / (q_rank ** 0.5 * kv_rank ** 0.5)
    w[p + "uv"][:, 0] = 3.0
    return cfg, {k: v.bfloat16().float() for k, v in w.items()}


def _ask(cfg, w, t, asker, ref, beacon):
    for dtype, tol in ((torch.float32, 3e-4), (torch.bfloat16, 0.05 * float(ref[asker].abs().max()) + 0.05)):
        eng = engine(cfg, w, dtype)
        close(eng.run_step([("w", t, [asker])]), ref[asker:asker + 1], tol)              # in a prompt
        eng.release("w")
        eng.run_step([("d", t[:asker], [])])
        close(eng.run_step([("d", [t[asker]], [0])]), ref[asker:asker + 1], tol)         # decoded alone
        eng.release("d")
        cut = max(1, beacon)                                                              # a portion that starts at the beacon
        eng.run_step([("p", t[:cut], [])])
        close(eng.run_step([("p", t[cut:], [asker - cut])]), ref[asker:asker + 1], tol)
        eng.release("p")
        if asker - beacon > 3:                                                            # decoding from just after the beacon to the asker
            eng.run_step([("q", t[:beacon + 2], [])])
            for tk in t[beacon + 2:asker]:
                eng.run_step([("q", [tk], [])])
            close(eng.run_step([("q", [t[asker]], [0])]), ref[asker:asker + 1], tol)


def _check_beacon(cfg, w, beacon, asker, seen):
    """The oracle confirms that swapping the beacon moves the asker's logits exactly when it is to be seen; the engine matches the oracle."""
    t = [3 + (i % 30) for i in range(asker + 1)]
    t[beacon], t[asker] = 1, 2
    ref = U.oracle_logits(cfg, w, t)
    t2 = list(t)
    t2[beacon] = 5
    moved = float((U.oracle_logits(cfg, w, t2)[asker] - ref[asker]).abs().max())
    assert (moved > 0.05) == seen, f"beacon {beacon}, asker {asker}: the oracle's logits moved by {moved}"
    _ask(cfg, w, t, asker, ref, beacon)


@pytest.mark.parametrize("window,keep,asker", [(40, 5, 100), (40, 0, 39), (40, 1, 40), (64, 20, 127), (64, 2, 128), (65, 33, 200), (16, 70, 170), (2, 3, 9), (97, 64, 230), (130, 10, 320)])
def test_dominant_key_just_inside_and_just_outside_the_window(window, keep, asker):
    """The beacon as the oldest key the window holds (distance window - 1), and one further back (seen only if it is a kept one)."""
    cfg, w = _window_beacon(window, keep)
    for dist in (window - 1, window):
        beacon = asker - dist
        if beacon >= 0:
            _check_beacon(cfg, w, beacon, asker, dist < window or beacon < keep)


@pytest.mark.parametrize("window,keep,asker", [(10, 1, 90), (10, 20, 90), (24, 31, 120), (24, 32, 120), (24, 33, 120), (9, 64, 200), (9, 65, 130), (70, 63, 300), (1, 2, 7), (50, 5, 56)])
def test_dominant_key_among_the_first_tokens(window, keep, asker):
    """The first and the last of the kept tokens, and the one behind them, with the asker far away."""
    cfg, w = _window_beacon(window, keep)
    for beacon in sorted({0, keep - 1, keep}):
        _check_beacon(cfg, w, beacon, asker, beacon < keep or asker - beacon < window)


@pytest.mark.parametrize("kind", ["window", "latent"])
@pytest.mark.parametrize("beacon,asker", [(0, 250), (3, 299), (63, 290), (64, 290), (127, 128), (128, 191), (190, 191), (1, 2)])
def test_dominant_key_far_back_and_at_page_borders(kind, beacon, asker):
    cfg, w = _window_beacon(1000, 2) if kind == "window" else _latent_beacon()
    _check_beacon(cfg, w, beacon, asker, True)


def test_kept_tokens_keep_their_positions():
    """A rotated key among the kept tokens: its angle is that of its true distance, hundreds of tokens away, not of a place beside the window."""
    cfg = U.make_config([U.window_layer(heads=2, kv_heads=1, dim=32, vdim=16, rot_dims=32, base=30.0, window=20, keep=6, scale=0.8)], vocab=40, width=32)
    w = U.make_weights(cfg, seed=33)
    t = toks(260, 40, 34)
    ref = U.oracle_logits(cfg, w, t)
    for dtype in (torch.float32, torch.bfloat16):
        eng = engine(cfg, w, dtype)
        got = [whole(eng, t)]
        eng.run_step([("d", t[:230], [])])
        got.append(torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[230:]]))
        for x, r in zip(got, (ref, ref[230:])):
            close(x, r, 3e-4) if dtype == torch.float32 else bf16_close(x, r)


def test_a_sink_that_takes_most_of_the_weight():
    outs = []
    for sinks in ((9.0, -30.0), (-30.0, 9.0), (0.5, -0.5)):
        cfg, w = _window_beacon(30, 4)
        w["l0.mix.sink"] = torch.tensor(sinks)
        t = [3 + (i % 30) for i in range(100)]
        ref = U.oracle_logits(cfg, w, t)
        outs.append(ref)
        eng = engine(cfg, w)
        close(whole(eng, t), ref, 3e-4)
        eng.run_step([("d", t[:70], [])])
        close(torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[70:]]), ref[70:], 3e-4)
        close(whole(engine(cfg, w, torch.bfloat16), t), ref, 0.05 * float(ref.abs().max()) + 0.05)
    assert float((outs[0] - outs[1]).abs().max()) > 0.05 and float((outs[0] - outs[2]).abs().max()) > 0.05


# ------------------------------------------------------------------------------------------------ long contexts
def test_long_decoding():
    cfg = U.make_config([U.window_layer(window=50, keep=7, mlp=U.moe()), U.latent_layer(mlp=U.dense()), U.window_layer(heads=2, kv_heads=1, window=130, keep=40)], loop=(0, 2, 2))
    w = U.make_weights(cfg, seed=23)
    t = toks(330, cfg["vocab"], 24)
    ref = U.oracle_logits(cfg, w, t)
    eng = engine(cfg, w)
    eng.run_step([("d", t[:10], [])])
    out = torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[10:]])
    close(out, ref[10:], 5e-4)


def test_contexts_beyond_a_thousand_tokens_split_decode_rows():
    """Past 1024 cached tokens a decode row's keys are dealt over several blocks and merged by a second launch: the kept tokens in front of the window and the
    head gates must survive that path."""
    cfg = U.make_config([U.window_layer(heads=2, kv_heads=1, window=1050, keep=40), U.latent_layer(heads=2)], vocab=50, width=32)
    w = U.make_weights(cfg, seed=41)
    t = toks(1240, 50, 42)
    ref = U.oracle_logits(cfg, w, t)
    eng = engine(cfg, w, max_tokens=1280)
    close(eng.run_step([("d", t[:1200], [0, 700, 1199])]), ref[[0, 700, 1199]], 5e-4)
    close(torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[1200:]]), ref[1200:], 5e-4)
    eng = engine(cfg, w, torch.bfloat16, max_tokens=1280)
    eng.run_step([("d", t[:1200], [])])
    bf16_close(torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[1200:]]), ref[1200:])


# ------------------------------------------------------------------------------------------------ generation
def _oracle_greedy(cfg, w, prompt, n):
    seq, margins = list(prompt), []
    for _ in range(n):
        lg = U.oracle_logits(cfg, w, seq)[-1]
        top = lg.topk(2).values
        margins.append(float(top[0] - top[1]))
        seq.append(int(lg.argmax()))
    return seq[len(prompt):], margins


def test_greedy_generation_through_the_scheduler():
    cfg = U.make_config([U.window_layer(window=20, mlp=U.dense()), U.latent_layer(mlp=U.moe(top=1))], vocab=64, width=48, loop=(0, 1, 2))
    w = U.make_weights(cfg, seed=29)
    prompts = [toks(n, 64, 30 + n) for n in (5, 40, 1, 70, 18, 33)]            # six requests over three slots: some wait their turn
    eng = engine(cfg, w, max_tokens=5 * 64, max_seqs=3, max_step_tokens=48)     # prompts are cut into portions of the step budget
    outs = eng.generate(prompts, 8)
    assert eng.cache.pages.free == 5 and eng.cache.slots.free == 3 and not eng.running and not eng.waiting
    for p, o in zip(prompts, outs):
        ref, margins = _oracle_greedy(cfg, w, p, 8)
        for i, (a, b) in enumerate(zip(o, ref)):
            if a != b:
                assert margins[i] < 1e-3, f"token {i}: {a} != {b} with a top-2 margin of {margins[i]}"
                break
    eng.use_graphs = True                                                        # decode-only steps as replayed graphs give the same tokens
    assert eng.generate(prompts[:3], 8) == outs[:3]
    sampled = eng.generate(prompts[:2], 6, top_k=5, top_p=0.9, temperature=0.8, seed=3)
    assert sampled == eng.generate(prompts[:2], 6, top_k=5, top_p=0.9, temperature=0.8, seed=3)
    assert all(len(o) == 6 and all(0 <= x < 64 for x in o) for o in sampled)


def test_command_line_generate_and_trace(tmp_path):
    from safetensors.torch import save_file
    cfg = U.make_config([U.latent_layer(mlp=None), U.window_layer(window=7, keep=2, mlp=U.moe())], vocab=64, width=48, loop=(1, 2, 2))
    w = U.make_weights(cfg, seed=31)
    d = tmp_path / "model"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.bfloat16().contiguous() for k, v in w.items()}, str(d / "model.safetensors"))
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = toks(21, 64, 32)
    r = subprocess.run([sys.executable, "-m", "rtp_llm_amd.cli", "generate", "--model", str(d), "--dtype", "float32", "--max-new-tokens", "5",
                        "--prompt-ids", ",".join(map(str, p))], cwd=root, capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    gen = json.loads(r.stdout.strip().splitlines()[-1])["generated"]
    ref, margins = _oracle_greedy(cfg, w, p, 5)
    assert gen == ref or min(margins) < 1e-3
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": p[:9], "want": [8]}, {"id": "b", "tokens": p[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": p[9:], "want": [0, 11]}], "end": ["a", "b"]}]
    out = tmp_path / "out"
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(d), "--dtype", "float32", "--out", str(out), "--max-tokens", "128"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", cwd=root, capture_output=True, text=True, timeout=300)
    assert r.returncode == 0 and "done 0" in r.stdout and "done 1" in r.stdout, r.stderr[-2000:]
    import numpy as np
    full = U.oracle_logits(cfg, w, p)
    close(torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(1, -1)), full[8:9], 3e-4)
    close(torch.from_numpy(np.fromfile(out / "1.f32", dtype="<f4").reshape(2, -1)), full[[9, 20]], 3e-4)


def test_graph_replayed_decode_steps_match_eager_and_oracle():
    """Decode steps through the captured graph with eager prompt portions and eager decode steps between the replays."""
    cfg = U.make_config(FULL, loop=LOOP)
    w = U.make_weights(cfg, seed=37)
    seqs = {k: toks(n, cfg["vocab"], 40 + i) for i, (k, n) in enumerate({"a": 90, "b": 61, "c": 75}.items())}
    ref = {k: U.oracle_logits(cfg, w, v) for k, v in seqs.items()}
    eng = engine(cfg, w)
    eng.run_step([("a", seqs["a"][:50], []), ("b", seqs["b"][:30], [])])
    at = {"a": 50, "b": 30, "c": 0}
    for i in range(30):
        eng.use_graphs = i % 3 != 2                                   # every third decode step runs eagerly
        out = eng.run_step([(k, [seqs[k][at[k]]], [0]) for k in ("a", "b")])
        for j, k in enumerate(("a", "b")):
            close(out[j:j + 1], ref[k][at[k]:at[k] + 1], 5e-4)
            at[k] += 1
        if i == 10:                                                   # an eager prefill step between replays
            eng.use_graphs = True
            eng.run_step([("c", seqs["c"][:70], [])]); at["c"] = 70
    eng.use_graphs = True
    out = eng.run_step([(k, [seqs[k][at[k]]], [0]) for k in ("a", "b", "c")])     # another shape: a second graph
    for j, k in enumerate(("a", "b", "c")):
        close(out[j:j + 1], ref[k][at[k]:at[k] + 1], 5e-4)
    assert len(eng._graphs) == 2
