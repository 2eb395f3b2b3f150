"""Host-side pieces of the Dupenex member (CPU): configuration reading and its errors, the registry, the order of layer runs, the cache layout, and the
plain implementation against closed forms."""
import json
import math
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import dupenex_oracle as O  # noqa: E402
import dupenex_util as U  # noqa: E402


def test_config_reading():
    from rtp_llm_amd.hybrid import HybridConfig, ParallelSpec
    from rtp_llm_amd.mixers import AttentionSpec, ChannelDeltaSpec, MatrixMemorySpec
    cfg = U.make_config([U.parallel_layer(U.window_side(heads=6, kv_heads=3, dim=20, vdim=12, rot_dims=10, window=33, scale=0.3), U.memory_side(heads=5, dim=8, vdim=40, cap=7.5),
                                          mlp=U.moe(experts=12, top=5, ff=72)),
                         U.delta_layer(heads=6, kv_heads=2, dim=24, vdim=10, conv=3, mlp=U.dense(56)), U.delta_layer()],
                        width=80, vocab=77, eps=1e-4, streams=5, loop=(1, 3, 4))
    c = HybridConfig.from_json(cfg)
    assert c.sequential and c.streams == 5 and c.loop == (1, 3, 4) and c.eps == 1e-4 and c.norm_offset == 0.0 and c.norm_kind == "rms"
    assert not (c.out_norm or c.depth_mix or c.branch_gates or c.tied_head or c.shared_norm) and c.logit_softcap == 0.0
    assert c.layer_runs() == [0, 1, 2, 1, 2, 1, 2, 1, 2] == O.layer_runs(cfg)
    L0, L1, L2 = c.layers
    assert isinstance(L0.mixer, ParallelSpec) and L0.mixer.out_norms and (L0.mixer.left_scale, L0.mixer.right_scale) == (0.5, 0.5)
    a, b = L0.mixer.left, L0.mixer.right
    assert isinstance(a, AttentionSpec) and (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.chunk, a.scale) == (6, 3, 20, 12, 33, 0, 0.3)
    assert a.out_gate and a.gate_channels and not (a.sink or a.qk_norm or a.bias) and (a.rot.layout, a.rot.dims, a.rot.scaling) == ("interleaved", 10, None)
    assert isinstance(b, MatrixMemorySpec) and (b.heads, b.dim, b.vdim, b.gate_cap) == (5, 8, 40, 7.5)
    assert (L0.ff, L0.mlp_kind, L0.mlp_act, L0.shared_ff) == (72, "plain_experts", "relu2", None)
    assert (L0.router.experts, L0.router.top, L0.router.score, L0.router.groups) == (12, 5, "softmax_chosen", 1)
    assert isinstance(L1.mixer, ChannelDeltaSpec) and (L1.mixer.heads, L1.mixer.kv_heads, L1.mixer.dim, L1.mixer.vdim, L1.mixer.conv) == (6, 2, 24, 10, 3)
    assert (L1.ff, L1.mlp_kind, L1.mlp_act) == (56, "gated", "silu") and L2.ff is None
    plain = json.loads(json.dumps(cfg)); del plain["loop"]
    assert HybridConfig.from_json(plain).layer_runs() == [0, 1, 2]
    for path, val, err in ((("layers", 0, "type"), "conv", NotImplementedError), (("layers", 1, "mlp", "kind"), "glu", NotImplementedError), (("loop", "stop"), 4, ValueError)):
        bad = json.loads(json.dumps(cfg))
        node = bad
        for k in path[:-1]:
            node = node[k]
        node[path[-1]] = val
        with pytest.raises(err):
            HybridConfig.from_json(bad)


def test_registry_names_the_member():
    from rtp_llm_amd import registry
    assert "dupenex" in registry.families()


def test_every_layer_run_has_a_cache_of_its_own():
    """Weights on the CPU are enough to lay out the caches: pages and two states for a parallel layer, two states for a delta layer, per run."""
    from rtp_llm_amd.hybrid import HybridConfig, HybridModel
    cfg = U.make_config([U.parallel_layer(right=U.memory_side(heads=3, dim=16, vdim=70)), U.delta_layer(heads=4, kv_heads=2, dim=16, vdim=24, conv=3, mlp=U.moe())],
                        loop=(0, 2, 3))
    m = HybridModel(HybridConfig.from_json(cfg), U.make_weights(cfg), torch.float32, "cpu")
    lay = m.cache_layout()
    assert len(lay) == 6 and lay[0] == lay[2] == lay[4] and lay[1] == lay[3] == lay[5]
    assert lay[0] == ("sides", [("kv", (2, 64, 16), (2, 64, 24)), ("state", (3, 16 * 70 + 16), (3, 2))])
    assert lay[1] == ("state", (4, 16, 24), (2, 2 * 2 * 16 + 4 * 24))
    caches = m.alloc_cache(5, 3)
    assert [len(c) for c in caches] == [4, 2] * 3 and caches[0][0].shape == (5, 2, 64, 16) and caches[0][2].shape == (3, 3, 16 * 71)
    assert len({t.data_ptr() for c in caches for t in c}) == 18


def test_weights_that_do_not_fit_are_refused():
    from rtp_llm_amd.hybrid import HybridConfig, HybridModel
    cfg = U.make_config([U.parallel_layer(mlp=U.moe()), U.delta_layer()])
    for name, change in (("l0.mix.left.g", lambda t: t[:-1]), ("l0.mix.right.norm", lambda t: t[:-1]), ("l1.mix.q.conv", lambda t: t[:, :-1]), ("l1.mix.A_log", lambda t: t[:-1]),
                         ("l0.hc2.mix", lambda t: t[:-1]), ("l0.mlp.router", lambda t: t[:-1])):
        w = U.make_weights(cfg)
        w[name] = change(w[name])
        with pytest.raises((ValueError, RuntimeError)):
            HybridModel(HybridConfig.from_json(cfg), w, torch.float32, "cpu")
    w = U.make_weights(cfg)
    del w["l1.mix.dt_bias"]
    with pytest.raises(KeyError):
        HybridModel(HybridConfig.from_json(cfg), w, torch.float32, "cpu")


def test_oracle_against_closed_forms():
    g = torch.Generator().manual_seed(1)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    # one delta step writes v where beta = 1, whatever the state was, and leaves what is orthogonal to k
    S, k, v = r(4, 3), torch.tensor([0.0, 1.0, 0.0, 0.0], dtype=torch.float64), r(3)
    S2, o = O.delta_step(S, k, k, v, torch.ones(4, dtype=torch.float64), 1.0)
    assert torch.allclose(o, v) and torch.allclose(S2[[0, 2, 3]], S[[0, 2, 3]])
    S2, _ = O.delta_step(S, k, k, v, torch.tensor([0.5, 1.0, 1.0, 1.0], dtype=torch.float64), 0.0)
    assert torch.allclose(S2[0], 0.5 * S[0]) and torch.allclose(S2[1:], S[1:])
    # the matrix memory is sum_j e^(i_j + f_(j+1) + .. + f_t) k_j v_j^T over max(|n . q|, 1), in a common scale
    T, d, dv = 6, 3, 2
    q, k, v, li, lf = r(T, d), r(T, d), r(T, dv), 3.0 * r(T), -r(T).abs()
    S, n, m = torch.zeros(d, dv, dtype=torch.float64), torch.zeros(d, dtype=torch.float64), 0.0
    for t in range(T):
        S, n, m, o = O.memory_step(S, n, m, q[t], k[t], v[t], float(li[t]), float(lf[t]))
        c = [math.exp(float(li[j] + lf[j + 1:t + 1].sum())) for j in range(t + 1)]
        num = sum(c[j] * float(k[j] @ q[t]) * v[j] for j in range(t + 1))
        nq = abs(sum(c[j] * float(k[j] @ q[t]) for j in range(t + 1)))
        want = num / max(nq, 1.0)
        assert torch.allclose(o, want, rtol=1e-4, atol=1e-6)
    assert m >= float(lf.sum()) - 1e-12
    # convolution: the last tap is the current token, and a history continues the sequence
    x, w = r(7, 2), r(2, 3)
    full = O.short_conv(x, w)
    assert torch.allclose(full[0], O.silu(w[:, 2] * x[0]))
    assert torch.allclose(O.short_conv(x[4:], w, x[2:4]), full[4:])
    # streams: the mix is indexed [from, to]
    X, M = r(2, 1, 1), torch.tensor([[1.0, 2.0], [3.0, 4.0]], dtype=torch.float64)
    Y = O.stream_write(X, M, torch.zeros(2, dtype=torch.float64), r(1, 1))
    assert torch.allclose(Y[1], 2.0 * X[0] + 4.0 * X[1])
    ids, wts = O.route(torch.tensor([0.1, 3.0, -1.0, 2.0], dtype=torch.float64), 2)
    assert ids == [1, 3] and abs(sum(wts) - 1.0) < 1e-12 and abs(wts[0] / wts[1] - math.e) < 1e-9
