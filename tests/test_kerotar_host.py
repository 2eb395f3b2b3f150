"""Host-side pieces of the Kerotar member (CPU): configuration reading and its errors, the registry, the order of layer runs and passes, the cache layout,
and the plain implementation against closed forms."""
import json
import math
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import kerotar_oracle as O  # noqa: E402
import kerotar_util as U  # noqa: E402


def test_config_reading():
    from rtp_llm_amd.hybrid import HybridConfig
    from rtp_llm_amd.mixers import AttentionSpec, LatentAttentionSpec
    cfg = U.make_config([U.window_layer(heads=6, kv_heads=3, dim=20, vdim=12, rot_dims=10, window=33, keep=7, scale=0.3, mlp=U.moe(experts=12, top=5, ff=72)),
                         U.latent_layer(heads=5, dim=12, rot_dim=6, vdim=10, kv_rank=18, q_rank=26, scale=0.21, base=77.0, mlp=U.dense(56, limit=2.5)), U.latent_layer()],
                        width=80, vocab=77, eps=1e-4, scale=2.25, loop=(1, 3, 4))
    c = HybridConfig.from_json(cfg)
    assert not c.sequential and c.shared_norm and not c.branch_gates and c.loop == (1, 3, 4) and c.loop_input and c.eps == 1e-4 and c.norm_offset == 0.0
    assert c.embed_scale == 2.25 and not (c.out_norm or c.depth_mix or c.tied_head or c.streams) and c.logit_softcap == 0.0 and c.residual_mult == 1.0
    assert c.layer_runs() == [0, 1, 2, 1, 2, 1, 2, 1, 2] == [i for i, _ in O.schedule(cfg)]
    assert c.pass_starts() == {1: 0, 3: 1, 5: 2, 7: 3} == {n: t for n, (_, t) in enumerate(O.schedule(cfg)) if t is not None}
    L0, L1, L2 = c.layers
    a = L0.mixer
    assert isinstance(a, AttentionSpec) and (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.keep_first, a.chunk, a.scale) == (6, 3, 20, 12, 33, 7, 0, 0.3)
    assert a.sink and a.learned_sink and a.qk_norm and a.qk_norm_whole and not (a.bias or a.out_gate or a.value_norm) and (a.rot.layout, a.rot.dims) == ("halves", 10)
    assert (L0.ff, L0.mlp_kind, L0.mlp_act, L0.router.experts, L0.router.top, L0.router.score, L0.shared_ff) == (72, "experts", "silu", 12, 5, "softmax_chosen", None)
    b = L1.mixer
    assert isinstance(b, LatentAttentionSpec) and (b.heads, b.dim, b.rot_dim, b.vdim, b.kv_rank, b.scale) == (5, 12, 6, 10, 18, 0.21)
    assert b.query_latent and b.out_gate and not b.gate_channels and not b.sink and (b.rot.layout, b.rot.dims, b.rot.base) == ("halves", 6, 77.0)
    assert (L1.ff, L1.mlp_kind, L1.mlp_act, L1.act_param) == (56, "gated", "swiglu_clamp", 2.5) and L2.ff is None
    plain = json.loads(json.dumps(cfg)); del plain["loop"]
    p = HybridConfig.from_json(plain)
    assert p.layer_runs() == [0, 1, 2] and p.pass_starts() == {} and not p.loop_input
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
    assert "kerotar" in registry.families()


def test_every_layer_run_has_a_cache_of_its_own():
    from rtp_llm_amd.hybrid import HybridConfig, HybridModel
    cfg = U.make_config([U.window_layer(), U.latent_layer(kv_rank=20, rot_dim=8, mlp=U.moe())], loop=(0, 2, 3))
    m = HybridModel(HybridConfig.from_json(cfg), U.make_weights(cfg), torch.float32, "cpu")
    lay = m.cache_layout()
    assert lay == [("kv", (2, 64, 16), (2, 64, 24)), ("latent", (64, 32))] * 3 and not m.has_state
    caches = m.alloc_cache(5, 3)
    assert caches[0][0].shape == (5, 2, 64, 16) and caches[1][0].shape == (5, 64, 32)
    assert len({t.data_ptr() for c in caches for t in c if t is not None}) == 9


def test_weights_that_do_not_fit_are_refused():
    from rtp_llm_amd.hybrid import HybridConfig, HybridModel
    cfg = U.make_config([U.window_layer(mlp=U.dense()), U.latent_layer(mlp=U.moe())], loop=(0, 1, 2))
    for name, change in (("l0.mix.q.norm", lambda t: t[:-1]), ("l0.mix.sink", lambda t: t[:-1]), ("l1.mix.dq.norm", lambda t: t[:-1]), ("l1.mix.uq", lambda t: t[:, :-1]),
                         ("l1.mix.g", lambda t: t[:-1]), ("l1.mlp.router", lambda t: t[:-1]), ("loop.in", lambda t: t[:, :-1]), ("loop.step", lambda t: t[:-1])):
        w = U.make_weights(cfg)
        w[name] = change(w[name])
        with pytest.raises((ValueError, RuntimeError)):
            HybridModel(HybridConfig.from_json(cfg), w, torch.float32, "cpu")
    w = U.make_weights(cfg)
    del w["l1.mix.uk"]
    with pytest.raises(KeyError):
        HybridModel(HybridConfig.from_json(cfg), w, torch.float32, "cpu")


def test_oracle_against_closed_forms():
    g = torch.Generator().manual_seed(1)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    see = O.visible(12, 3, 2)
    assert see[11].nonzero().flatten().tolist() == [0, 1, 9, 10, 11] and see[3].nonzero().flatten().tolist() == [0, 1, 2, 3] and see[0].nonzero().flatten().tolist() == [0]
    assert O.visible(5, 0, 0).sum() == 15 and O.visible(6, 2, 0)[5].nonzero().flatten().tolist() == [4, 5]
    # a sink takes its share and nothing else; scores and sink may be shifted together
    s = r(2, 4)
    p = O.softmax_sink(s, torch.tensor(0.7, dtype=torch.float64))
    assert torch.allclose(p, torch.exp(s) / (torch.exp(s).sum(-1, keepdim=True) + math.exp(0.7)))
    assert torch.allclose(O.softmax_sink(s), torch.softmax(s, -1))
    # the turn keeps lengths and makes products depend on the distance only; channels behind the span stay
    q = r(1, 1, 6).expand(9, 1, 6).contiguous()
    k = r(1, 1, 6).expand(9, 1, 6).contiguous()
    a, b = O.rotate(q, 4, 50.0), O.rotate(k, 4, 50.0)
    assert torch.allclose(a[7, 0] @ b[4, 0], a[3, 0] @ b[0, 0]) and torch.equal(a[..., 4:], q[..., 4:])
    c, t = math.cos(5.0), math.sin(5.0)
    assert torch.allclose(a[5, 0, 0], q[5, 0, 0] * c - q[5, 0, 2] * t) and torch.allclose(a[5, 0, 2], q[5, 0, 2] * c + q[5, 0, 0] * t)
    # renormalised softmax weights are the softmax over the chosen
    ids, wts = O.route(torch.tensor([0.1, 3.0, -1.0, 2.0], dtype=torch.float64), 2)
    assert ids == [1, 3] and abs(sum(wts) - 1.0) < 1e-12 and abs(wts[0] / wts[1] - math.e) < 1e-9
    # the clamped unit: gate from above, up from both sides
    one = torch.eye(1, dtype=torch.float64)
    w = {"gate": 1.0 * one, "up": -3.0 * one, "down": one}
    lim = 0.5
    y = O.clamped_mlp(2.0 * one, w, "", lim)
    assert torch.allclose(y, lim / (1 + torch.exp(torch.tensor(-1.702 * lim, dtype=torch.float64))) * (1.0 - lim) * one)
    y = O.clamped_mlp(-2.0 * one, w, "", lim)
    assert torch.allclose(y, -2.0 / (1 + torch.exp(torch.tensor(3.404, dtype=torch.float64))) * (1.0 + lim) * one)
    x, x0, A, st = r(3, 2), r(3, 2), r(2, 4), r(2)
    assert torch.allclose(O.inject(x, x0, A, st), x @ A[:, :2].T + x0 @ A[:, 2:].T + st)
