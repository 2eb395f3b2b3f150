"""The Dupenex member of the hybrid family on the GPU against the plain implementation in dupenex_oracle (float64, CPU): single operations, every
mechanism alone in many shapes, whole prompts against token-by-token decoding, portions down to two tokens, unequal batches, reused pages and slots,
a key just inside / just outside the sliding window and at page borders with weights built so that it dominates, a token carried for hundreds of steps
by either recurrence, long decoding, graph replay, and greedy generation through the scheduler and the command line."""
import json
import os
import subprocess
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import dupenex_oracle as O  # noqa: E402
import dupenex_util as U  # noqa: E402

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


def bf16_close(got, ref, median=0.05, tail=0.1):
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


FULL = [U.parallel_layer(mlp=U.dense()),
        U.delta_layer(mlp=U.moe()),
        U.parallel_layer(U.window_side(heads=3, kv_heads=1, dim=32, vdim=16, rot_dims=32, window=70), U.memory_side(heads=2, dim=8, vdim=72, cap=4.0), mlp=U.moe(experts=5, top=3, ff=33)),
        U.delta_layer(heads=3, kv_heads=3, dim=40, vdim=12, conv=2, mlp=None)]
LOOP = (1, 3, 2)
# without routers, whose close calls rounding to 16 bits may turn over
NO_ROUTER = [dict(L, mlp=U.dense(48) if L["mlp"] else None) for L in FULL]


# ------------------------------------------------------------------------------------------------ single operations
@pytest.mark.parametrize("S", [1, 2, 3, 4, 7, 16])
def test_streams_boundary(S):
    """Start, write-back of every kind of result, read and norm, gathered rows, for widths with and without 16-byte rows."""
    from rtp_llm_amd import hybrid_ops as hops
    g = torch.Generator().manual_seed(S)
    d = lambda t: t.to(DEV)
    for W in (8, 50, 64, 1100):
        T, top = 7, 3
        X, a, b = torch.randn(T, S, W, generator=g), torch.randn(T, W, generator=g) * 3.0, torch.randn(T, W, generator=g) * 0.2
        mix, wr, rd = torch.randn(S, S, generator=g), torch.randn(S, generator=g), torch.randn(S, generator=g)
        y = torch.randn(T * top, W, generator=g)
        place = torch.randperm(T * top, generator=g).to(torch.int32).reshape(T, top)
        wts = torch.rand(T, top, generator=g)
        msum = (wts.double()[:, :, None] * y.double()[place.long()]).sum(1)
        for dt in (torch.float32, torch.bfloat16):
            w, na, nb = ((1.0 + 0.3 * torch.randn(W, generator=g)).to(dt) for _ in range(3))
            wd, nad, nbd = w.double(), na.double(), nb.double()
            htol = 3e-5 if dt == torch.float32 else 0.05
            cases = {
                "one branch": (dict(a=d(a)), a.double()),
                "two normed branches": (dict(a=d(a), ca=0.5, na=d(na), b=d(b), cb=0.25, nb=d(nb), branch_eps=1e-4),
                                        0.5 * O.rms_norm(a.double(), nad, 1e-4) + 0.25 * O.rms_norm(b.double(), nbd, 1e-4)),
                "mixture": (dict(moe=hops.MoeSum(d(y), d(place), d(wts))), msum),
                "mixture and an ungated shared branch": (dict(moe=hops.MoeSum(d(y), d(place), d(wts), d(a))), msum + a.double()),
            }
            for name, (kw, res) in cases.items():
                Xo = O.stream_write(X.double().transpose(0, 1), mix.double(), wr.double(), res)
                want = O.rms_norm(O.stream_read(Xo, rd.double()), wd, 1e-5)
                Xd = d(X)
                h = hops.streams(Xd, mix=d(mix), write=d(wr), read=d(rd), w=d(w), eps=1e-5, **kw)
                close(Xd, Xo.transpose(0, 1), 5e-5)
                assert h.dtype == dt
                close(h, want, htol)
                rows = I([5, 0, 5])
                Xd = d(X)
                h = hops.streams(Xd, mix=d(mix), write=d(wr), w=d(w), eps=1e-5, rows=rows, **kw)      # the last norm: sum of the streams, nothing written
                close(h, O.rms_norm(Xo.sum(0), wd, 1e-5)[[5, 0, 5]], htol)
                assert torch.equal(Xd.cpu(), X), name
            h = hops.streams(d(X), rows=I([2]), w=d(w), eps=1e-5)
            close(h, O.rms_norm(X.double().sum(1), wd, 1e-5)[[2]], htol)
            table = torch.randn(30, W, generator=g).to(dt)
            ids = torch.randint(0, 30, (T,), generator=g).to(torch.int32)
            Xd = torch.full((T, S, W), 7.0, device=DEV)
            h = hops.streams(Xd, ids=d(ids), table=d(table), read=d(rd), w=d(w), eps=1e-5)
            e = table.double()[ids.long()]
            close(Xd, e[:, None].expand(T, S, W), 0.0)
            close(h, O.rms_norm(e * rd.double().sum(), wd, 1e-5), htol)


@pytest.mark.parametrize("G,dim,rest,taps", [(2, 16, 40, 4), (1, 20, 7, 3), (3, 64, 200, 2), (2, 130, 260, 4), (1, 8, 8, 1), (2, 24, 50, 6)])
def test_short_convolutions_histories_and_unit_heads(G, dim, rest, taps):
    """Sequences of unequal length in one launch, cut into steps shorter than the taps and long enough for the sliding form; the histories are moved
    on by the recurrence's kernel."""
    from rtp_llm_amd import hybrid_ops as hops
    g = torch.Generator().manual_seed(dim * taps)
    C, R = 2 * G * dim + rest, 10
    lens, slots = [150, 1, 75, 9], [2, 0, 4, 3]
    steps = [[1, 1, 1, 2], [1, 0, 2, 2], [2, 0, 1, 0], [137, 0, 70, 5], [9, 0, 1, 0]]
    xs = [torch.randn(n, C, generator=g) for n in lens]
    for dt in (torch.float32, torch.bfloat16):
        w = torch.randn(C, taps, generator=g).to(dt)
        want = []
        for x in xs:
            y = O.short_conv(x.double(), w.double())
            for j in range(2 * G):
                y[:, j * dim:(j + 1) * dim] = O.unit(y[:, j * dim:(j + 1) * dim]) * (dim ** -0.5 if j < G else 1.0)
            want.append(y)
        hist = torch.full((5, taps - 1, C), 9.0, device=DEV)                       # what an earlier owner of the slot left must not matter
        H, vd = 1, 4
        state = torch.zeros(5, H, 4, vd, device=DEV)
        at = [0] * 4
        for st in steps:
            keep = [i for i in range(4) if st[i]]
            rows = torch.cat([torch.cat([xs[i][at[i]:at[i] + st[i]], torch.arange(R).expand(st[i], R) * 1.0], 1) for i in keep])
            rs = [0]
            for i in keep:
                rs.append(rs[-1] + st[i])
            seq = [n for n, i in enumerate(keep) for _ in range(st[i])]
            sl, fp = I([slots[i] for i in keep]), I([at[i] for i in keep])
            proj = rows.to(DEV)
            out, low = hops.short_conv(proj, C, w.to(DEV), hist, I(seq), I(rs), sl, fp, unit_heads=2 * G, query_heads=G, dim=dim, qscale=dim ** -0.5, low=(C + 1, R - 2))
            close(out, torch.cat([want[i][at[i]:at[i] + st[i]] for i in keep]), 3e-5)
            assert low.dtype == dt and torch.equal(low.float().cpu(), torch.arange(1, R - 1).expand(len(seq), R - 2).float())
            z = torch.zeros(len(seq), 12, device=DEV)                              # any recurrence: here only its hold on the histories counts
            hops.channel_delta_scan(torch.zeros(len(seq), 12, device=DEV), 0, 4, 8, z[:, :4], torch.zeros(4, device=DEV), torch.ones(1, device=DEV), z[:, 5:6], H, 1, 4, vd,
                                    I(rs), sl, fp, state, raw=proj, hist=hist if taps > 1 else None)
            for i in keep:
                at[i] += st[i]
                for j in range(taps - 1):
                    t = at[i] - (taps - 1) + j
                    close(hist[slots[i], j], xs[i][t].double() if t >= 0 else torch.zeros(C, dtype=torch.float64), 0.0)
        if taps > 1:
            assert float((hist[1] - 9.0).abs().max()) == 0.0


@pytest.mark.parametrize("H,G,dim,vdim", [(4, 2, 16, 24), (1, 1, 8, 8), (3, 1, 20, 12), (2, 2, 64, 64), (2, 1, 130, 72), (6, 3, 32, 100), (1, 1, 256, 16), (2, 1, 170, 33)])
def test_channel_delta_scan_states_and_outputs(H, G, dim, vdim):
    """The recurrence alone: three sequences of unequal length, continued from the states an earlier launch left."""
    from rtp_llm_amd import hybrid_ops as hops
    g = torch.Generator().manual_seed(dim + vdim)
    lens, slots, cut = [37, 1, 18], [3, 0, 4], [20, 1, 5]
    T, gd = sum(lens), G * dim
    x = torch.randn(T, 2 * gd + H * vdim + 5, generator=g)
    ro, ko, vo = 1, 1 + gd, 3 + 2 * gd
    for j in range(G):
        for o, f in ((ro, dim ** -0.5), (ko, 1.0)):
            x[:, o + j * dim:o + (j + 1) * dim] = O.unit(x[:, o + j * dim:o + (j + 1) * dim]) * f
    z, zb, rate = torch.randn(T, H * dim, generator=g) * 3.0, torch.randn(H * dim, generator=g) - 2.0, torch.exp(torch.randn(H, generator=g))
    z[:, 0] = 40.0; z[:, 1] = -60.0                                                # a channel that forgets at once and one that never forgets
    steps = torch.randn(T, H + 2, generator=g) * 2.0
    sd = torch.zeros(5, H, dim, vdim, device=DEV)
    S = [torch.zeros(H, dim, vdim, dtype=torch.float64) for _ in lens]
    starts = [0, lens[0], lens[0] + lens[1], T]

    def ref(rows, St):
        out = torch.zeros(len(rows), H, vdim, dtype=torch.float64)
        for n, t in enumerate(rows):
            for h in range(H):
                j = h // (H // G)
                dec = torch.exp(-rate[h].double() * O.softplus(z[t, h * dim:(h + 1) * dim].double() + zb[h * dim:(h + 1) * dim].double()))
                St[h], out[n, h] = O.delta_step(St[h], x[t, ro + j * dim:ro + (j + 1) * dim].double(), x[t, ko + j * dim:ko + (j + 1) * dim].double(),
                                                x[t, vo + h * vdim:vo + (h + 1) * vdim].double(), dec, torch.sigmoid(steps[t, 1 + h].double()))
        return out.reshape(len(rows), H * vdim)

    for part in (0, 1):
        rows = [list(range(starts[i] + (0 if part == 0 else cut[i]), starts[i] + (cut[i] if part == 0 else lens[i]))) for i in range(3)]
        keep = [i for i in range(3) if rows[i]]
        flat = [t for i in keep for t in rows[i]]
        rs = [0]
        for i in keep:
            rs.append(rs[-1] + len(rows[i]))
        out = hops.channel_delta_scan(x[flat].to(DEV), ro, ko, vo, z[flat].to(DEV), zb.to(DEV), rate.to(DEV), steps[flat].to(DEV)[:, 1:1 + H], H, G, dim, vdim, I(rs),
                                      I([slots[i] for i in keep]), I([0 if part == 0 else cut[i] for i in keep]), sd)
        close(out, torch.cat([ref(rows[i], S[i]) for i in keep]), 5e-5)
    for i in range(3):
        close(sd[slots[i]], S[i], 5e-5)
    assert float(sd[1].abs().max()) == 0.0 and float(sd[2].abs().max()) == 0.0


@pytest.mark.parametrize("H,dim,vdim,cap,chunk", [(2, 16, 24, 15.0, 64), (1, 64, 64, 2.0, 64), (3, 20, 12, 7.0, 128), (2, 136, 72, 15.0, 64), (2, 8, 140, 30.0, 64), (1, 260, 40, 5.0, 64)])
def test_matrix_memory_walk_and_chunks(H, dim, vdim, cap, chunk):
    """Both forms of the scan against the definition: sequences that start fresh or continue states, lengths on both sides of chunk borders, single rows
    between long ones; one head whose input gates reach the cap (the running maximum climbs), one whose forget gates let it sink below zero."""
    from rtp_llm_amd import hybrid_ops as hops
    g = torch.Generator().manual_seed(dim * 7 + vdim)
    lens, slots, first = [200, 1, 64, 65, 330, 2, 127], [6, 0, 3, 1, 5, 2, 4], [0, 9, 0, 40, 7, 0, 1]
    T, hd, hv, nz = sum(lens), H * dim, H * vdim, (vdim + 63) // 64
    proj = torch.randn(T, 2 * hd + hv + 2 * H + 4, generator=g)
    qo, ko, vo, io, fo = 0, hd, 2 * hd + 4, 2 * hd + hv + 4, 2 * hd + hv + 4 + H
    proj[:, io:io + H] = proj[:, io:io + H] * 6.0
    proj[:, fo:fo + H] = proj[:, fo:fo + H] * 2.0 + 2.0
    if H > 1:
        proj[:, io + 1], proj[:, fo + 1] = proj[:, io + 1] - 40.0, proj[:, fo + 1] - 3.0
    Sm = [{} for _ in range(7)]
    start = torch.zeros(7, H, dim * vdim + dim)
    mstart = torch.randn(7, H, 1, generator=g).expand(7, H, nz).contiguous() * 2.0
    start[:, :, :dim * vdim], start[:, :, dim * vdim:] = torch.randn(7, H, dim * vdim, generator=g), torch.randn(7, H, dim, generator=g)
    rs = [0]
    for n in lens:
        rs.append(rs[-1] + n)
    want = torch.zeros(T, H, vdim, dtype=torch.float64)
    for i, n in enumerate(lens):
        for h in range(H):
            fresh = first[i] == 0
            S = torch.zeros(dim, vdim, dtype=torch.float64) if fresh else start[slots[i], h, :dim * vdim].double().view(dim, vdim)
            nn = torch.zeros(dim, dtype=torch.float64) if fresh else start[slots[i], h, dim * vdim:].double()
            m = 0.0 if fresh else float(mstart[slots[i], h, 0])
            for t in range(rs[i], rs[i + 1]):
                p = proj[t].double()
                li = float(cap * torch.tanh(p[io + h] / cap))
                lf = float(O.log_sigmoid(cap * torch.tanh(p[fo + h] / cap)))
                S, nn, m, want[t, h] = O.memory_step(S, nn, m, p[qo + h * dim:qo + (h + 1) * dim] * dim ** -0.5, p[ko + h * dim:ko + (h + 1) * dim],
                                                     p[vo + h * vdim:vo + (h + 1) * vdim], li, lf)
            Sm[i][h] = (S, nn, m)
    old = hops.SCAN_CHUNK
    hops.SCAN_CHUNK = chunk
    try:
        for chunked in (True, False):
            sd, md, plans = start.clone().to(DEV), mstart.clone().to(DEV), {}
            out, den = hops.memory_scan(proj.to(DEV), qo, ko, vo, io, fo, cap, dim ** -0.5, 1e-6, H, dim, vdim, I(rs), I(slots), I(first), sd, md, plans=plans, chunked=chunked)
            assert (len(plans) == 1) == chunked
            o = out.double().cpu().view(T, H, vdim) / den.double().cpu()[:, :, None]
            err = (o - want).abs() / (1.0 + want.abs())
            assert float(err.max()) < 1e-3 and float(err.flatten().quantile(0.99)) < 5e-5, (float(err.max()), chunked)
            for i in range(len(lens)):
                for h in range(H):
                    S, nn, m = Sm[i][h]
                    close(md[slots[i], h], torch.full((nz,), m, dtype=torch.float64), 2e-5)
                    scale = float(S.abs().max()) + 1e-3
                    close(sd[slots[i], h, :dim * vdim] / scale, S.flatten() / scale, 5e-5)
                    close(sd[slots[i], h, dim * vdim:] / scale, nn / scale, 5e-5)
    finally:
        hops.SCAN_CHUNK = old


@pytest.mark.parametrize("E,top", [(6, 2), (12, 12), (5, 1), (100, 7), (64, 3)])
def test_router_weighs_by_the_softmax_over_the_chosen(E, top):
    from rtp_llm_amd import hybrid_ops as hops
    g = torch.Generator().manual_seed(E)
    for T in (1, 40, 130):                                                         # one launch for a few tokens, two for many
        z = torch.randn(T, E + 3, generator=g) * 4.0
        z[0, 1:] -= 200.0 * torch.arange(E + 2)                                    # exponentials of the chosen far below the largest underflow
        ids, wts, offs, src, place, tiles = hops.moe_route_sorted(z.to(DEV)[:, 1:1 + E], E, 1, 1, top, chosen=True)
        for t in range(T):
            rid, rw = O.route(z[t, 1:1 + E].double(), top)
            assert ids[t].cpu().tolist() == rid
            close(wts[t], torch.tensor(rw, dtype=torch.float64), 1e-6)


def test_squared_relu_in_the_linears_and_groups_over_column_slices():
    """The plain activation in the tile, skinny, row and grouped kernels; groups that read and write column slices at every number of rows; a grid of
    tiles that is no multiple of the XCDs or the bands."""
    from rtp_llm_amd import hybrid_ops as hops
    g = torch.Generator().manual_seed(3)
    K, N, G = 48, 40, 3
    w, bias = torch.randn(G, N, K, generator=g) * 0.3, torch.randn(N, generator=g)
    for M in (1, 2, 5, 16, 70):
        x = torch.randn(M, G * K, generator=g)
        ref = torch.clamp(x[:, :K].double() @ w[0].double().T, min=0.0) ** 2
        close(hops.dense_linear(x[:, :K].to(DEV), w[0].to(DEV), act=hops.ACT_RELU2), ref, 2e-5)
        bx, bw = x[:, :K].bfloat16(), w[0].bfloat16()
        close(hops.dense_linear(bx.to(DEV), bw.to(DEV), act=hops.ACT_RELU2, out_dtype=torch.float32), torch.clamp(bx.double() @ bw.double().T, min=0.0) ** 2, 2e-5)
        for dt in (torch.float32, torch.bfloat16):
            xd, wd = x.to(dt), w.to(dt)
            got = hops.dense_grouped(xd.to(DEV), wd.to(DEV), x_step=K, y_step=N + 8, out_dtype=torch.float32)
            for j in range(G):
                close(got[:, j * (N + 8):j * (N + 8) + N], xd[:, j * K:(j + 1) * K].double() @ wd[j].double().T, 2e-5)
        ids = (torch.arange(M) % G).to(torch.int32).reshape(M, 1).to(DEV)
        offs, src, place, tiles = hops.moe_align(ids, G)
        out = hops.dense_grouped(x[:, :K].contiguous().to(DEV), w.to(DEV), offs=offs, gather=src, tiles=tiles, rows=M, act=hops.ACT_RELU2)
        for r in range(M):
            close(out[place[r].long()].reshape(1, -1), torch.clamp(x[r:r + 1, :K].double() @ w[r % G].double().T, min=0.0) ** 2, 2e-5)
    for M, N in ((64 * 19 + 5, 128 * 11 + 3), (17, 64), (64 * 35, 128 * 3)):
        x, wt = torch.randn(M, 40, generator=g), torch.randn(N, 40, generator=g)
        close(hops.dense_linear(x.to(DEV), wt.to(DEV)), x.double() @ wt.double().T, 5e-5)
        xb, wb = x.bfloat16(), wt.bfloat16()
        close(hops.dense_linear(xb.to(DEV), wb.to(DEV), out_dtype=torch.float32), xb.double() @ wb.double().T, 5e-5)


# ------------------------------------------------------------------------------------------------ mechanisms alone
ALONE = {
    "parallel": (U.parallel_layer(), {}),
    "parallel_dense": (U.parallel_layer(mlp=U.dense()), {}),
    "parallel_experts": (U.parallel_layer(mlp=U.moe()), dict(streams=2)),
    "one_kv_head_odd_sizes": (U.parallel_layer(U.window_side(heads=3, kv_heads=1, dim=20, vdim=12, rot_dims=10, window=17), U.memory_side(heads=1, dim=20, vdim=12)), dict(streams=1)),
    "mha_no_rotary": (U.parallel_layer(U.window_side(heads=2, kv_heads=2, dim=12, vdim=20, rot_dims=0, window=33), U.memory_side(heads=5, dim=8, vdim=8)), {}),
    "window_of_one": (U.parallel_layer(U.window_side(window=1)), {}),
    "window_wider_than_the_prompt": (U.parallel_layer(U.window_side(window=500, base=1e6, rot_dims=16)), {}),
    "matrix_core_sizes": (U.parallel_layer(U.window_side(heads=4, kv_heads=2, dim=64, vdim=32, rot_dims=32, window=64), U.memory_side(heads=2, dim=64, vdim=64), mlp=U.dense(64)), {}),
    "wide_heads": (U.parallel_layer(U.window_side(heads=2, kv_heads=1, dim=160, vdim=136, window=40, rot_dims=20), U.memory_side(heads=1, dim=136, vdim=200)), dict(streams=6)),
    "one_value_channel": (U.parallel_layer(U.window_side(heads=2, kv_heads=1, dim=8, vdim=1), U.memory_side(heads=2, dim=4, vdim=1)), {}),
    "tight_gates": (U.parallel_layer(right=U.memory_side(cap=0.5)), {}),
    "delta": (U.delta_layer(), {}),
    "delta_experts": (U.delta_layer(mlp=U.moe(experts=7, top=7, ff=17)), {}),
    "delta_one_tap": (U.delta_layer(heads=2, kv_heads=1, dim=8, vdim=40, conv=1, mlp=U.dense(33)), dict(streams=2)),
    "delta_many_taps": (U.delta_layer(heads=3, kv_heads=3, dim=33, vdim=17, conv=7), {}),
    "delta_grouped_heads": (U.delta_layer(heads=6, kv_heads=2, dim=64, vdim=72, conv=2), dict(streams=4)),
    "delta_wide_heads": (U.delta_layer(heads=1, kv_heads=1, dim=200, vdim=130, conv=3), {}),
    "experts_top_one": (U.delta_layer(mlp=U.moe(experts=5, top=1, ff=64)), {}),
    "single_expert": (U.parallel_layer(mlp=U.moe(experts=1, top=1)), {}),
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


def test_other_widths_ranks_and_constants():
    """Widths that are no multiple of four or eight, ranks of one and wider than the heads, another eps."""
    for width, ra, rg, S in ((50, 1, 3, 2), (36, 30, 2, 1), (130, 16, 8, 5)):
        cfg = U.make_config([U.delta_layer(mlp=U.dense(30)), U.parallel_layer(U.window_side(window=11), mlp=U.moe(ff=33))], vocab=61, width=width, eps=1e-3, streams=S)
        w = U.make_weights(cfg, seed=width, rank_a=ra, rank_g=rg)
        t = toks(40, 61, width)
        ref = U.oracle_logits(cfg, w, t)
        eng = engine(cfg, w)
        close(whole(eng, t), ref, 3e-4)
        eng.run_step([("d", t[:25], [])])
        close(torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[25:]]), ref[25:], 3e-4)


@pytest.mark.parametrize("loop", [None, (0, 1, 1), (0, 4, 2), (1, 2, 3), (3, 4, 2), (1, 3, 0), (2, 2, 5)])
def test_layer_loops(loop):
    """A span at the start, in the middle, at the end, the whole stack, once, never; every run keeps keys and states of its own."""
    cfg = U.make_config(FULL, width=48, loop=loop)
    w = U.make_weights(cfg, seed=4)
    t = toks(60, cfg["vocab"], 5)
    col, ocol = [], []
    ref = U.oracle_logits(cfg, w, t, ocol)
    eng = engine(cfg, w)
    got = eng.run_step([("x", t, range(len(t)))], collect=col)
    assert len(col) == len(ocol) == len(O.layer_runs(cfg))
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
            if L.kind == "parallel":
                mixer.left.use_tiles = tiles
        bf16_close(whole(eng, t), ref)


def test_every_part_of_the_model_matters():
    """The oracle itself: changing a constant, or a tensor of the kind that is easily left out, moves the logits, so a part the engine lost would show in
    the comparisons above."""
    cfg = U.make_config(FULL[:2], loop=(0, 2, 2))
    w = U.make_weights(cfg, seed=7)
    t = toks(40, cfg["vocab"], 8)
    ref = U.oracle_logits(cfg, w, t)
    moved = lambda c, ww: float((U.oracle_logits(c, ww, t) - ref).abs().max())
    for name in ("l0.mix.left.g", "l0.mix.left.out", "l0.mix.right.out", "l0.mix.right.i.b", "l0.mix.right.f.b", "l0.mix.right.norm", "l0.mix.right.g", "l1.mix.dt_bias", "l1.mix.A_log",
                 "l1.mix.b", "l1.mix.g2", "l1.mix.norm", "l1.mix.q.conv", "l1.mix.k.conv", "l1.mix.v.conv", "l1.mlp.router", "l0.hc1.in", "l0.hc1.out", "l1.hc2.out"):
        w2 = dict(w); w2[name] = w[name] * 0.5 + 0.1
        assert moved(cfg, w2) > 0.01, name
    for name in ("l0.hc1.mix", "l1.hc2.mix"):
        w2 = dict(w); w2[name] = w[name].T.contiguous()                 # the mix is indexed [from, to]
        assert moved(cfg, w2) > 0.01, name
    for path, val in ((("layers", 0, "mixer", "right", "gate_cap"), 1.0), (("layers", 0, "mixer", "left", "mask", "size"), 5), (("layers", 0, "mixer", "left", "scale"), 0.6),
                      (("layers", 0, "mixer", "left", "rot", "base"), 10.0), (("layers", 0, "mixer", "left", "rot", "dims"), 4), (("layers", 1, "mlp", "router", "top"), 3),
                      (("loop", "times"), 3), (("loop", "start"), 1)):
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


@pytest.mark.parametrize("sizes", [[2] * 40, [33, 2, 31, 5, 64, 1, 1, 2, 60], [63, 1, 64, 65, 6], [1, 198], [23, 1, 24, 25, 47, 70], [3, 2, 2, 130, 2, 1, 62]])
def test_portions(sizes):
    cfg = U.make_config(FULL, loop=LOOP)
    w = U.make_weights(cfg, seed=11)
    n = sum(sizes)
    t = toks(n, cfg["vocab"], 12)
    ref = U.oracle_logits(cfg, w, t)
    eng = engine(cfg, w)
    at, outs = 0, []
    for s in sizes:
        outs.append(eng.run_step([("p", t[at:at + s], range(s))]))
        at += s
    close(torch.cat(outs), ref, 5e-4)


def test_long_portions_take_the_chunked_memory():
    """A prompt long enough for the chunked form, whole and in two long portions, with a decoded tail: the same logits as the walk gives."""
    from rtp_llm_amd import hybrid_ops as hops
    cfg = U.make_config([U.parallel_layer(), U.delta_layer(heads=2, kv_heads=1)], width=32, vocab=60)
    w = U.make_weights(cfg, seed=12)
    t = toks(620, 60, 13)
    assert hops.scan_prefers_chunks(600, 1, 600, 3, 20, hops.SCAN_CHUNK) and hops.scan_prefers_chunks(300, 1, 300, 3, 20, hops.SCAN_CHUNK)
    ref = U.oracle_logits(cfg, w, t)
    eng = engine(cfg, w)
    close(whole(eng, t), ref, 5e-4)
    outs = [eng.run_step([("p", t[:300], range(300))]), eng.run_step([("p", t[300:602], range(302))])]
    outs += [eng.run_step([("p", [tk], [0])]) for tk in t[602:]]
    close(torch.cat(outs), ref, 5e-4)


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


def test_a_state_slot_that_comes_back_starts_from_zero():
    """One slot, two requests after each other: the second must not see what the first left in a state, a running maximum, a convolution or the pages."""
    cfg = U.make_config([U.parallel_layer(), U.delta_layer(conv=5)], vocab=50, width=32)
    w = U.make_weights(cfg, seed=15)
    w["l0.mix.right.f.b"] += 6.0
    w["l1.mix.dt_bias"] -= 5.0                                       # long memories
    a, b = toks(70, 50, 16), toks(66, 50, 17)
    eng = engine(cfg, w, max_tokens=128, max_seqs=1)
    close(whole(eng, a, "a"), U.oracle_logits(cfg, w, a), 3e-4)
    ref = U.oracle_logits(cfg, w, b)
    outs = [eng.run_step([("b", b[:1], [0])]), eng.run_step([("b", b[1:3], [0, 1])]), eng.run_step([("b", b[3:40], range(37))])]
    outs += [eng.run_step([("b", [tk], [0])]) for tk in b[40:]]
    close(torch.cat(outs), ref, 3e-4)


# ------------------------------------------------------------------------------------------------ one key that dominates: page borders, window edges
def _axes_model(layer, width, vocab, seed):
    """Embeddings in which token 1 (the beacon) lives on axis 0 alone, token 2 (the asker) on axis 1 alone and every other token on neither."""
    cfg = U.make_config([layer], vocab=vocab, width=width, streams=2)
    w = U.make_weights(cfg, seed=seed)
    w["l0.norm1"].fill_(1.0)
    e = torch.randn(vocab, width, generator=torch.Generator().manual_seed(seed + 1))
    e[:, :2] = 0.0
    e[1], e[2] = 0.0, 0.0
    e[1, 0], e[2, 1] = 1.0, 1.0
    w["embed"] = e
    return cfg, w


def _beacon_model(window=40, heads=2, kv_heads=1, dim=16, vdim=16):
    """The key of the beacon and the query of the asker meet in one un-rotated channel that every other token leaves empty: the asker scores the beacon
    near 16 and every other key near zero, and the beacon's value is far from the others'.  The memory side weighs nothing."""
    width, c = 32, dim - 1                               # the channel: beyond the rotary span
    cfg, w = _axes_model(U.parallel_layer(U.window_side(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, rot_dims=8, window=window, scale=0.5), U.memory_side(heads=1, dim=8, vdim=8)),
                         width, 40, 17)
    p = "l0.mix.left."
    w["l0.mix.right.out"].fill_(0.0)
    for n in ("q", "k"):
        w[p + n] *= 0.05
    for g in range(kv_heads):
        w[p + "k"][g * dim + c] = 0.0
        w[p + "k"][g * dim + c, 0] = 1.0
    for h in range(heads):
        w[p + "q"][h * dim + c] = 0.0
        w[p + "q"][h * dim + c, 1] = 1.0
    w[p + "v"][:, 0] = 3.0 * torch.randn(kv_heads * vdim, generator=torch.Generator().manual_seed(19))
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


@pytest.mark.parametrize("window,asker", [(40, 100), (40, 39), (40, 40), (64, 127), (64, 128), (65, 200), (16, 70), (2, 9), (97, 230), (130, 320)])
def test_dominant_key_just_inside_and_just_outside_the_window(window, asker):
    """The beacon as the oldest key the asker still sees (distance window - 1), and one further back (not seen any more): the oracle confirms
    that the first moves the asker's logits and the second does not, and the engine matches it in a prompt, decoded, and in portions."""
    cfg, w = _beacon_model(window=window)
    for dist, seen in ((window - 1, True), (window, False)):
        beacon = asker - dist
        if beacon < 0:
            continue
        t = [3 + (i % 30) for i in range(asker + 1)]
        t[beacon], t[asker] = 1, 2
        ref = U.oracle_logits(cfg, w, t)
        t2 = list(t)
        t2[beacon] = 5
        moved = float((U.oracle_logits(cfg, w, t2)[asker] - ref[asker]).abs().max())
        assert (moved > 0.05) == seen, f"distance {dist}: the oracle's logits moved by {moved}"
        _ask(cfg, w, t, asker, ref, beacon)


@pytest.mark.parametrize("beacon,asker", [(0, 250), (3, 299), (63, 290), (64, 290), (127, 128), (128, 191), (190, 191), (1, 2)])
def test_dominant_key_far_back_and_at_page_borders(beacon, asker):
    """A window wider than the sequence: the beacon at the first positions and on both sides of page borders, hundreds of keys back."""
    cfg, w = _beacon_model(window=1000)
    t = [3 + (i % 30) for i in range(asker + 1)]
    t[beacon], t[asker] = 1, 2
    ref = U.oracle_logits(cfg, w, t)
    t2 = list(t); t2[beacon] = 5
    assert float((U.oracle_logits(cfg, w, t2)[asker] - ref[asker]).abs().max()) > 0.05, "the beacon must move the asker's logits"
    _ask(cfg, w, t, asker, ref, beacon)


def _carried(cfg, w, n, check):
    t = [3 + (i % 30) for i in range(n)]
    t[2], t[n - 1] = 1, 2
    ref = U.oracle_logits(cfg, w, t)
    t2 = list(t); t2[2] = 7
    assert float((U.oracle_logits(cfg, w, t2)[-1] - ref[-1]).abs().max()) > 0.05, "the carried token must move the asker's logits"
    check(t, t2)
    eng = engine(cfg, w)
    close(whole(eng, t)[-1:], ref[-1:], 5e-4)
    eng.run_step([("d", t[:n - 50], [])])
    close(torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[n - 50:]]), ref[n - 50:], 5e-4)
    eng.release("d")
    eng.run_step([("p", t[:2], [])])                                    # a portion that starts at the beacon, then two-token portions
    eng.run_step([("p", t[2:n - 5], [])])
    out = torch.cat([eng.run_step([("p", t[n - 5:n - 3], [0, 1])]), eng.run_step([("p", t[n - 3:n - 1], [0, 1])]), eng.run_step([("p", t[n - 1:], [0])])])
    close(out, ref[n - 5:], 5e-4)
    bf16_close(whole(engine(cfg, w, torch.bfloat16), t), ref, 0.1, 0.3)


def test_matrix_memory_carries_a_far_token():
    """The beacon opens the input gate wide and writes into a key channel no other token touches; the forget gates stay near one and the others' input gates
    near zero, so the running maximum keeps the beacon's scale for hundreds of tokens.  The window has long passed (and the left side weighs nothing)."""
    d = 16
    cfg, w = _axes_model(U.parallel_layer(U.window_side(window=8), U.memory_side(heads=2, dim=d, vdim=12, cap=15.0)), 32, 40, 23)
    w["l0.mix.left.out"].fill_(0.0)
    p = "l0.mix.right."
    w[p + "k"] *= 0.2; w[p + "q"] *= 0.2
    for h in range(2):
        w[p + "k"][h * d + d - 1] = 0.0
        w[p + "q"][h * d + d - 1] = 0.0
        w[p + "k"][h * d + d - 1, 0] = 1.0
        w[p + "q"][h * d + d - 1, 1] = 1.0
    w[p + "i"] *= 0.1; w[p + "f"] *= 0.1
    w[p + "i"][:, 0] = 1.0
    w[p + "i.b"].fill_(-3.0)
    w[p + "f.b"] = torch.tensor([7.0, -1.0])                             # the second head forgets
    w = {k: v.bfloat16().float() for k, v in w.items()}

    def check(t, t2):
        w2 = dict(w); w2[p + "f.b"] = torch.tensor([-1.0, -1.0])
        assert float((U.oracle_logits(cfg, w2, t2)[-1] - U.oracle_logits(cfg, w2, t)[-1]).abs().max()) < 1e-6      # only the first head remembers
    _carried(cfg, w, 400, check)


def test_channel_delta_carries_a_far_token():
    """The beacon writes into a key channel no other token touches and that decays slowly; the rest of the state decays at once."""
    d = 16
    cfg, w = _axes_model(U.delta_layer(heads=2, kv_heads=1, dim=d, vdim=12, conv=3), 32, 40, 29)
    p = "l0.mix."
    for n in ("q", "k"):
        w[p + n] = w[p + n].abs() * 0.3
        w[p + n + ".conv"][:] = torch.tensor([0.1, 0.1, 1.0])
        w[p + n][d - 1] = 0.0
    w[p + "k"][d - 1, 0] = 2.0
    w[p + "q"][d - 1, 1] = 2.0
    w[p + "a2"] *= 0.1
    w[p + "A_log"].fill_(0.0)
    w[p + "dt_bias"].fill_(2.0)
    w[p + "dt_bias"].view(2, d)[:, d - 1] = -7.0
    w = {k: v.bfloat16().float() for k, v in w.items()}

    def check(t, t2):
        w2 = dict(w); w2[p + "dt_bias"] = torch.full((2 * d,), 2.0)
        assert float((U.oracle_logits(cfg, w2, t2)[-1] - U.oracle_logits(cfg, w2, t)[-1]).abs().max()) < 1e-6      # only the slow channel remembers
    _carried(cfg, w, 400, check)


def test_long_decoding():
    cfg = U.make_config([U.parallel_layer(U.window_side(window=50), mlp=U.moe()), U.delta_layer(mlp=U.dense()),
                         U.parallel_layer(U.window_side(heads=2, kv_heads=1, window=130))], loop=(0, 2, 2))
    w = U.make_weights(cfg, seed=23)
    w["l1.mix.dt_bias"] -= 3.0
    t = toks(330, cfg["vocab"], 24)
    ref = U.oracle_logits(cfg, w, t)
    eng = engine(cfg, w)
    eng.run_step([("d", t[:10], [])])
    out = torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[10:]])
    close(out, ref[10:], 5e-4)


def test_contexts_beyond_a_thousand_tokens_split_decode_rows():
    """Past 1024 cached tokens a decode row's keys are dealt over several blocks and merged by a second launch: the channel gates and the window's start must
    survive that path."""
    cfg = U.make_config([U.parallel_layer(U.window_side(heads=2, kv_heads=1, window=1100), U.memory_side(heads=1))], vocab=50, width=32, streams=2)
    w = U.make_weights(cfg, seed=41)
    t = toks(1180, 50, 42)
    ref = U.oracle_logits(cfg, w, t)
    eng = engine(cfg, w, max_tokens=1280)
    close(eng.run_step([("d", t[:1140], [0, 700, 1139])]), ref[[0, 700, 1139]], 5e-4)
    out = torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[1140:]])
    close(out, ref[1140:], 5e-4)
    eng = engine(cfg, w, torch.bfloat16, max_tokens=1280)
    eng.run_step([("d", t[:1140], [])])
    bf16_close(torch.cat([eng.run_step([("d", [tk], [0])]) for tk in t[1140:]]), ref[1140:])


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
    cfg = U.make_config([U.parallel_layer(U.window_side(window=20)), U.delta_layer(mlp=U.moe(top=1))], vocab=64, width=48, loop=(0, 1, 2))
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
    cfg = U.make_config([U.delta_layer(mlp=None), U.parallel_layer(U.window_side(window=7), mlp=U.moe())], vocab=64, width=48, streams=2)
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
