"""The Bapavik design of the hybrid family without a GPU: the reader of config.json and its refusals, the weight
layout, page accounting, the plan of which chunks attend with expanded keys, and properties of the plain
restatement that the GPU tests lean on."""
import math

import numpy as np
import pytest
import torch

from oracle import bapavik_ref as R


def _cfg():
    att = {"heads": 6, "kv_heads": 2, "dim": 10, "vdim": 12, "scale": 0.3, "softcap": 11.0, "q_temp": {"coef": 0.7, "every": 9}}
    lat = {"heads": 3, "dim": 16, "rot_dim": 8, "vdim": 24, "kv_rank": 40, "scale": 0.2, "rot": {"dims": 8, "base": 700.0}}
    return {"architecture": "Bapavik", "width": 96, "vocab": 50, "norm": {"eps": 1e-5}, "embedding": {"scale": 9.5},
            "loop": {"start": 1, "stop": 3, "times": 3},
            "layers": [{"type": "attention", "mixer": att, "mlp": {"kind": "moe", "expert": {"ff": 20}, "router": {"experts": 5, "top": 2}}},
                       {"type": "latent_attention", "mixer": lat, "mlp": None},
                       {"type": "attention", "mixer": {k: v for k, v in att.items() if k not in ("softcap", "q_temp")},
                        "mlp": {"kind": "dense", "ff": 80, "limit": 1.25}},
                       {"type": "latent_attention", "mixer": lat, "mlp": {"kind": "moe", "expert": {"ff": 24}, "router": {"experts": 3, "top": 1}}}]}


def test_config_reader():
    from mi355_decode.config import NO_WINDOW, ModelConfig
    cfg = ModelConfig.from_dict(_cfg())
    spec = cfg.hybrid
    assert cfg.family == "hybrid" and cfg.architecture == "Bapavik" and (cfg.vocab_size, cfg.hidden_size) == (50, 96)
    assert cfg.rms_norm_eps == 1e-5 and not cfg.tie_word_embeddings and cfg.torch_dtype == "bfloat16"
    assert (spec.arrangement, spec.embed_scale, spec.layer_norm, spec.loop_plain) == ("pre", 9.5, True, True)
    assert [i for i, _ in spec.runs()] == [0, 1, 2, 1, 2, 1, 2, 3]
    a, c, lat = spec.layers[0].battn, spec.layers[2].battn, spec.layers[1].lattn
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.softcap, a.temp_coef, a.temp_every) == (6, 2, 10, 12, 0.3, 11.0, 0.7, 9.0)
    assert a.row_norm and a.learned_sink and not (a.qk_norm or a.penalty or a.values_are_keys or a.bias or a.rot_dims or a.window or a.block)
    assert (c.softcap, c.temp_every) == (0.0, 0.0)
    assert (lat.heads, lat.dim, lat.rot_dim, lat.vdim, lat.kv_rank, lat.rot_dims, lat.rot_base, lat.scale) == (3, 16, 8, 24, 40, 8, 700.0, 0.2)
    assert lat.q_direct and lat.interleaved and not lat.sink and not lat.gate and lat.window == NO_WINDOW
    m = spec.layers[0].moe
    assert (m.experts, m.top, m.ff, m.score, m.gated) == (5, 2, 20, "table", False)
    assert (spec.layers[2].ff, spec.layers[2].ff_act, spec.layers[2].ff_limit) == (80, "limited", 1.25)
    plain = {k: v for k, v in _cfg().items() if k not in ("embedding", "loop")}
    plain = ModelConfig.from_dict(plain).hybrid
    assert plain.embed_scale == 1.0 and plain.runs() == [(i, None) for i in range(4)]
    for layer, part, change in ((0, "mixer", {"kv_heads": 4}), (0, "mixer", {"softcap": -1.0}), (1, "mixer", {"rot": {"dims": 10, "base": 5.0}}),
                                (1, "mixer", {"rot": {"dims": 7, "base": 5.0}}), (0, "mlp", {"router": {"experts": 5, "top": 6}}),
                                (2, "mlp", {"kind": "sparse"})):
        bad = _cfg()
        bad["layers"][layer][part].update(change)
        with pytest.raises(ValueError):
            ModelConfig.from_dict(bad)
    bad = _cfg()
    bad["layers"][1]["type"] = "mlstm"
    with pytest.raises(ValueError):
        ModelConfig.from_dict(bad)
    bad = _cfg()
    bad["loop"]["stop"] = 5
    with pytest.raises(ValueError):
        ModelConfig.from_dict(bad)


def test_weight_layout_and_page_accounting():
    from mi355_decode import weights as W
    from mi355_decode.config import ModelConfig
    d = _cfg()
    cfg = ModelConfig.from_dict(d)
    st = R.random_state(d, seed=1)
    w = W.from_state_dict(cfg, st, torch.bfloat16, "cpu")
    l0, l1, l2, l3 = w.layers
    assert list(l0.seg) == ["q", "k", "v"] and list(l1.seg) == ["q", "dkv"] and all(a % 8 == 0 for lw in w.layers for a, _ in lw.seg.values())
    a, n = l0.seg["k"]
    assert n == 20 and torch.equal(l0.in_w[a:a + n].float(), st["l0.mix.k"])
    assert l0.sink.dtype == torch.float32 and torch.equal(l0.sink, st["l0.mix.sink"]) and l0.q_norm.shape == (60,) and l0.k_norm.shape == (20,)
    a, n = l1.seg["dkv"]
    assert n == 48 and torch.equal(l1.in_w[a:a + n].float(), st["l1.mix.dkv"])
    # per-head products: natural and transposed key up-projection, natural value up-projection
    uk, uv = st["l1.mix.uk"].view(3, 16, 40), st["l1.mix.uv"].view(3, 24, 40)
    assert torch.equal(l1.uk_w.float(), uk) and torch.equal(l1.uk_t.float(), uk.transpose(1, 2)) and torch.equal(l1.uv_w.float(), uv) and l1.uv_t is None
    f32 = W.from_state_dict(cfg, st, torch.float32, "cpu").layers[1]
    assert f32.uk_t is None and torch.equal(f32.uv_t, uv.transpose(1, 2))
    assert l0.table.dtype == torch.int32 and torch.equal(l0.table, st["l0.mlp.table"]) and l0.up_w.shape == (5, 20, 96) and l0.down_w.shape == (5, 96, 20)
    assert torch.equal(l0.up_w[3].float(), st["l0.mlp.e3.up"]) and l2.gate_up_w.shape == (160, 96) and torch.equal(l2.gate_up_w[80:].float(), st["l2.mlp.up"])
    assert l1.norm2 is None and torch.equal(w.lm_head.float(), st["head"]) and l3.table.shape == (50, 1)
    assert set(W.hybrid_synthetic_state(cfg, seed=0)) == set(st)
    for e in W.hybrid_synthetic_state(cfg, seed=0)["l0.mlp.table"].tolist():
        assert len(set(e)) == 2 and min(e) >= 0 and max(e) < 5
    for name, change in (("l0.mix.sink", lambda t: t[:-1]), ("l0.mlp.table", lambda t: t + 1), ("l1.mix.dkv", lambda t: t[:-8])):
        with pytest.raises(ValueError):
            W.from_state_dict(cfg, dict(st, **{name: change(st[name])}), torch.float32, "cpu")


def test_plan_of_expanded_chunks():
    """Long chunks get pages of their own over their whole context; the others keep their rows, in packed order."""
    from mi355_decode.hybrid_runner import LatentPlan
    least = LatentPlan.EXPAND_MIN_ROWS
    cu = np.cumsum([0, least, 1, least + 5, 3])
    ctx = [least, 40, 100, 3]
    bt = np.arange(4 * 10).reshape(4, 10)[:, ::-1].copy()
    p = LatentPlan(cu, ctx, bt, "cpu")
    n0, n2 = -(-least // 16), 7
    assert p.fits and p.pages == n0 + n2 and p.max_q_len == least + 5 and p.ctx.tolist() == [least, 0, 100, 0]
    index = p.index.view(-1, 16)
    assert index[:, 0].tolist() == [int(x) * 16 for x in list(bt[0, :n0]) + list(bt[2, :n2])]
    assert torch.equal(index - index[:, :1], torch.arange(16, dtype=torch.int32).expand(n0 + n2, 16))
    assert p.tables[0, :n0].tolist() == list(range(n0)) and p.tables[2, :n2].tolist() == list(range(n0, n0 + n2))
    assert int(p.tables.max()) < p.pages and int(p.tables.min()) >= 0
    rows, tables, seq = p.short
    assert rows.tolist() == [int(cu[1])] + list(range(int(cu[3]), int(cu[4]))) and seq.tolist() == [0, 1, 1, 1]
    assert tables.tolist() == bt[[1, 3]].tolist()
    assert p.short_tiles(3).tolist() == [[0, 0, 3], [1, 3, 9]] and p.short_tiles(17)[:3].tolist() == [[0, 0, 16], [0, 16, 1], [1, 17, 16]]
    assert not LatentPlan([0, 1, 2], [9, 9], bt, "cpu").fits
    assert LatentPlan([0, 64], [64], bt, "cpu").short is None


def test_restatement_norms_temperature_and_rotation():
    g = torch.Generator().manual_seed(0)
    x = torch.randn(5, 12, generator=g, dtype=torch.float64) * 3 + 7
    y = R.layer_norm(x, torch.ones(12, dtype=torch.float64), 0.0)
    assert torch.allclose(y.mean(-1), torch.zeros(5, dtype=torch.float64), atol=1e-12) and torch.allclose((y ** 2).mean(-1), torch.ones(5, dtype=torch.float64))
    assert torch.allclose(R.layer_norm(x * 0 + 2.0, torch.ones(12, dtype=torch.float64), 1e-6), torch.zeros(5, 12, dtype=torch.float64))
    t = R.query_temperature(40, {"coef": 0.5, "every": 8}, torch.float64)
    assert t[:7].tolist() == [1.0] * 7 and abs(float(t[7]) - (1 + 0.5 * math.log(2))) < 1e-12 and abs(float(t[39]) - (1 + 0.5 * math.log(6))) < 1e-12
    assert R.query_temperature(3, None).tolist() == [1.0, 1.0, 1.0]
    # a turn keeps lengths of neighbours, position 0 stays, and scores depend on the distance alone
    rot = {"dims": 6, "base": 30.0}
    q = torch.randn(1, 8, generator=g, dtype=torch.float64).expand(20, 8)
    k = torch.randn(1, 8, generator=g, dtype=torch.float64).expand(20, 8)
    a, b = R.rotate_neighbours(q, rot), R.rotate_neighbours(k, rot)
    assert torch.equal(a[0], q[0]) and torch.equal(a[:, 6:], q[:, 6:])
    assert torch.allclose(a[:, 0] ** 2 + a[:, 1] ** 2, q[:, 0] ** 2 + q[:, 1] ** 2)
    assert torch.allclose(a[9] @ b[4], a[14] @ b[9]) and not torch.allclose(a[9] @ b[4], a[9] @ b[5])
    c = math.cos(3 * 30.0 ** (-2 / 6)) * q[3, 2] - math.sin(3 * 30.0 ** (-2 / 6)) * q[3, 3]
    assert abs(float(a[3, 2] - c)) < 1e-12


def test_restatement_attention_sinks_and_caps():
    T, H, d = 6, 2, 4
    q, k = torch.zeros(T, H, d), torch.zeros(T, 1, d)
    v = torch.arange(T, dtype=torch.float32).view(T, 1, 1)
    o = R.attention(q, k, v, 1.0, 5.0, torch.tensor([0.0, math.log(6.0)]))
    assert abs(float(o[5, 0]) - 15 / 7) < 1e-6 and abs(float(o[5, 1]) - 15 / 12) < 1e-6      # equal scores: the sink counts e^sink keys
    assert abs(float(R.attention(q, k, v, 1.0, None, None)[5, 0]) - 2.5) < 1e-6
    s = torch.tensor([-100.0, 0.0, 1.0, 100.0])
    assert torch.allclose(R.capped(s, 8.0), torch.tensor([-8.0, 0.0, 8 * math.tanh(1 / 8), 8.0])) and torch.equal(R.capped(s, None), s)


def test_restatement_feed_forwards():
    g = torch.Generator().manual_seed(3)
    h = torch.randn(4, 6, generator=g)
    wt = {"gate": torch.randn(5, 6, generator=g) * 3, "up": torch.randn(5, 6, generator=g) * 3, "down": torch.randn(6, 5, generator=g)}
    y = R.dense_ff(wt, "", {"limit": 0.5}, h)
    gte, up = (h @ wt["gate"].T), (h @ wt["up"].T)
    assert float(gte.min()) < -0.5 and float(up.min()) < -0.5                                # the gate is limited above only
    gte, up = torch.minimum(gte, torch.tensor(0.5)), up.clamp(-0.5, 0.5)
    assert torch.allclose(y, (gte / (1 + torch.exp(-1.702 * gte)) * (up + 1)) @ wt["down"].T, atol=1e-6)
    ex = {"table": torch.tensor([[0, 2], [1, 0], [2, 1]], dtype=torch.int32)}
    for e in range(3):
        ex[f"e{e}.up"], ex[f"e{e}.down"] = torch.randn(5, 6, generator=g), torch.randn(6, 5, generator=g)
    y = R.table_moe_ff(ex, "", {"router": {"top": 2}}, h, [1, 0, 1, 2])
    want = 0.5 * (R.expert(ex, "e1.", h[2:3]) + R.expert(ex, "e0.", h[2:3]))
    assert torch.allclose(y[2:3], want, atol=1e-5)


def test_restatement_is_causal_and_loops():
    d = _cfg()
    st = R.random_state(d, seed=3)
    toks = np.random.default_rng(0).integers(0, 50, 30).tolist()
    trace = []
    z = R.forward(st, d, toks, trace)
    assert z.shape == (30, 50) and len(trace) == 8
    other = toks[:20] + [(t + 1) % 50 for t in toks[20:]]
    z2 = R.forward(st, d, other)
    assert torch.allclose(z[:20], z2[:20], atol=1e-5) and not torch.allclose(z[20], z2[20], atol=1e-3)
    unrolled = dict(d, layers=[d["layers"][i] for i in (0, 1, 2, 1, 2, 1, 2, 3)], loop=None)
    names = {f"l{n}.{k.split('.', 1)[1]}": v for n, i in enumerate((0, 1, 2, 1, 2, 1, 2, 3)) for k, v in st.items() if k.startswith(f"l{i}.")}
    assert torch.equal(R.forward({**{k: v for k, v in st.items() if not k.startswith("l")}, **names}, unrolled, toks), z)
