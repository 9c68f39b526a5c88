"""The Rigazen design of the hybrid family without a GPU: the reader of config.json and its refusals, the
weight layout (one input matrix with its bias row, one output matrix over both mixers' heads, norm weights
stored around zero, the tied head), page accounting, the tile lists of the recurrences, the exact rotary table,
and properties of the plain restatement that the GPU tests lean on."""
import math

import numpy as np
import pytest
import torch

from oracle import rigazen_ref as R


def _cfg():
    left = {"heads": 6, "kv_heads": 2, "dim": 16, "vdim": 9, "mask": {"size": 20, "keep_first": 3}, "rot": {"dims": 8, "base": 500.0}, "scale": 0.3}
    right = {"heads": 2, "dim": 12, "vdim": 20, "decay": [0.0, 0.97]}
    par = {"left": left, "right": right, "left_scale": 0.6, "right_scale": 1.5}
    return {"architecture": "Rigazen", "width": 96, "vocab": 160, "norm": {"eps": 1e-5}, "embedding": {"scale": 9.5}, "token_side": {"dim": 10},
            "layers": [{"type": "parallel", "mixer": par, "mlp": {"kind": "dense", "ff": 80}},
                       {"type": "mlstm", "mixer": {"heads": 3, "dim": 16, "vdim": 24, "gate_cap": 7.5}, "mlp": None},
                       {"type": "parallel", "mixer": dict(par, left=dict(left, mask=None, rot=None)), "mlp": None}]}


def test_config_reader():
    from mi355_decode.config import ModelConfig
    cfg = ModelConfig.from_dict(_cfg())
    spec = cfg.hybrid
    assert cfg.family == "hybrid" and cfg.architecture == "Rigazen" and cfg.vocab_size == 160 and cfg.hidden_size == 96
    assert cfg.rms_norm_eps == 1e-5 and cfg.tie_word_embeddings and cfg.torch_dtype == "bfloat16"
    assert (spec.arrangement, spec.embed_scale, spec.token_side) == ("post", 9.5, 10)
    a, c = spec.layers[0].battn, spec.layers[2].battn
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.block, a.window, a.keep_first, a.scale) == (6, 2, 16, 9, 0, 20, 3, 0.3)
    assert a.bias and a.row_norm and not a.qk_norm and not a.penalty and (a.rot_dims, a.rot_base) == (8, 500.0)
    assert (c.window, c.keep_first, c.rot_dims) == (0, 0, 0)
    d, m = spec.layers[0].lin, spec.layers[1].mem
    assert (d.heads, d.dim, d.vdim, d.decay) == (2, 12, 20, (0.0, 0.97))
    assert (m.heads, m.dim, m.vdim, m.gate_cap) == (3, 16, 24, 7.5)
    assert (spec.layers[0].left_scale, spec.layers[0].right_scale) == (0.6, 1.5)
    assert (spec.layers[0].ff, spec.layers[0].ff_act, spec.layers[1].ff) == (80, "relu2", None)
    assert [L.kind for L in spec.layers] == ["attention_decay", "mlstm", "attention_decay"] and spec.runs() == [(i, None) for i in range(3)]
    plain = {k: v for k, v in _cfg().items() if k not in ("embedding", "token_side")}
    plain = ModelConfig.from_dict(plain).hybrid
    assert plain.embed_scale == 1.0 and plain.token_side == 0
    for layer, side, change in ((0, "left", {"kv_heads": 4}), (0, "left", {"rot": {"dims": 18, "base": 10.0}}), (0, "left", {"rot": {"dims": 7, "base": 10.0}}),
                                (0, "right", {"decay": [0.5]}), (0, "right", {"decay": [0.5, -0.1]}), (1, None, {"gate_cap": 0.0})):
        bad = _cfg()
        mix = bad["layers"][layer]["mixer"]
        (mix if side is None else mix[side]).update(change)
        with pytest.raises(ValueError):
            ModelConfig.from_dict(bad)
    bad = _cfg()
    bad["layers"][1]["type"] = "mingru"
    with pytest.raises(ValueError):
        ModelConfig.from_dict(bad)
    bad = _cfg()
    bad["layers"][0]["mlp"]["kind"] = "moe"
    with pytest.raises(ValueError):
        ModelConfig.from_dict(bad)


def test_weight_layout_and_page_accounting():
    from mi355_decode import weights as W
    from mi355_decode.config import ModelConfig
    d = _cfg()
    cfg = ModelConfig.from_dict(d)
    st = R.random_state(d, seed=1)
    w = W.from_state_dict(cfg, st, torch.float32, "cpu")
    l0, l1, l2 = w.layers
    assert list(l0.seg) == ["lq", "lk", "lv", "q", "k", "v", "g"] and list(l1.seg) == ["q", "k", "v", "g"]
    for lw in w.layers:
        assert all(a % 8 == 0 for a, _ in lw.seg.values())
    a, n = l0.seg["lk"]
    assert n == 32 and torch.equal(l0.in_w[a:a + n], st["l0.mix.left.k"]) and torch.equal(l0.in_b[a:a + n], st["l0.mix.left.k.b"])
    a, n = l0.seg["q"]
    assert torch.equal(l0.in_w[a:a + n], st["l0.mix.right.q"]) and float(l0.in_b[a:].abs().max()) == 0.0       # no bias on the right
    # heads of the attention (6 x 9 = 54 columns, padded to 56), then those of the linear attention
    assert l0.out_w.shape == (96, 56 + 40) and torch.equal(l0.out_w[:, :54], st["l0.mix.left.o"])
    assert float(l0.out_w[:, 54:56].abs().max()) == 0.0 and torch.equal(l0.out_w[:, 56:], st["l0.mix.right.o"])
    assert torch.equal(l0.norm1, 1.0 + st["l0.norm1"]) and torch.equal(l0.head_norm, 1.5 * st["l0.mix.right.norm"])
    assert l0.log_decay.dtype == torch.float64 and float(l0.log_decay[0]) == -1e30 and abs(float(l0.log_decay[1]) - math.log(0.97)) < 1e-16
    assert torch.equal(l1.gate_w, torch.cat([st["l1.mix.i"], st["l1.mix.f"]])) and torch.equal(l1.gate_b[3:], st["l1.mix.f.b"])
    assert l1.norm2 is None and l1.up_w is None and torch.equal(l1.side_norm, st["l1.side.norm"]) and l1.in_b is None
    assert w.lm_head is w.embed and torch.equal(w.final_norm, 1.0 + st["final.norm"]) and w.side_embed.shape == (160, 30)
    # a 16-bit engine keeps norm weights in 32 bits: one plus a small weight is no 16-bit number
    h = W.from_state_dict(cfg, st, torch.bfloat16, "cpu")
    assert h.layers[0].norm1.dtype == torch.float32 and torch.equal(h.layers[0].norm1, l0.norm1) and h.layers[0].in_w.dtype == torch.bfloat16
    assert h.layers[1].gate_w32.dtype == torch.float32
    # the head counts once
    assert w.nbytes() == sum(t.numel() * t.element_size() for t in [w.embed, w.final_norm, w.side_embed] + [t for lw in w.layers for t in lw.tensors()])
    assert set(W.hybrid_synthetic_state(cfg, seed=0)) == set(st)
    bad = dict(st)
    bad["l1.mix.f.b"] = bad["l1.mix.f.b"][:-1]
    with pytest.raises(ValueError):
        W.from_state_dict(cfg, bad, torch.float32, "cpu")
    runs = [cfg.hybrid.layers[i] for i, _ in cfg.hybrid.runs()]
    assert sum(x.kv_heads * (x.dim + x.vdim) for L in runs for x in (L.battn,) if x is not None) == 2 * 2 * 25


def test_row_tiles_and_state_sizes():
    from mi355_decode import ops
    t = ops.RowTiles([0, 70, 70, 71, 135], 32, "cpu")
    assert t.tiles.tolist() == [[0, 0, 32], [0, 32, 32], [0, 64, 6], [2, 70, 1], [3, 71, 32], [3, 103, 32]]
    assert t.start.tolist() == [0, 3, 3, 4, 6] and t.count == 6 and t.rows == 32
    assert ops.query_tiles([0, 17, 18]).tolist() == [[0, 0, 16], [0, 16, 1], [1, 17, 1]]
    assert ops.linear_attn_state_floats(5, 7, False) == 36 and ops.linear_attn_state_floats(5, 7, True) == 40
    assert ops.linear_attn_state_floats(8, 4, True) == 40
    assert ops.linear_attn_tile_rows(16, 16) == 64 and ops.linear_attn_tile_rows(128, 128) == 64
    assert ops.linear_attn_tile_rows(256, 256) == 32 and ops.linear_attn_tile_rows(4096, 4096) == 0


def test_exact_rotary_table():
    from mi355_decode.hybrid_runner import rotary_table
    t = rotary_table(6, 77.0, 5000, "cpu", exact=True)
    for p, i in ((0, 0), (1, 2), (4999, 1), (3141, 0)):
        a = p * 77.0 ** (-2.0 * i / 6)
        assert abs(float(t[p, i]) - math.cos(a)) < 1e-7 and abs(float(t[p, 3 + i]) - math.sin(a)) < 1e-7
    assert rotary_table(0, 1.0, 16, "cpu", exact=True).shape == (16, 0)


def test_restatement_window_and_kept_tokens():
    m = R.window_mask(40, 7, 3)
    for i in range(40):
        assert [j for j in range(40) if m[i, j]] == sorted(set(range(max(i - 6, 0), i + 1)) | set(range(min(3, i + 1))))
    assert R.window_mask(5, 1, 0).tolist() == torch.eye(5, dtype=torch.bool).tolist()
    assert bool(R.window_mask(9, 0, 0)[8, 0])
    # equal scores: the mean over the visible values
    v = torch.arange(12, dtype=torch.float32).view(12, 1, 1)
    o = R.attend(torch.zeros(12, 2, 4), torch.zeros(12, 1, 4), v, 1.0, 4, 2)
    assert abs(float(o[11, 0]) - (0 + 1 + 8 + 9 + 10 + 11) / 6) < 1e-6 and float(o[11, 1]) == float(o[11, 0])


def test_restatement_norms_sit_on_the_outputs():
    x = torch.randn(4, 30, generator=torch.Generator().manual_seed(0))
    assert torch.allclose((R.rms(x, 0.0) ** 2).mean(-1), torch.ones(4), atol=1e-5)
    assert torch.allclose(R.rms(x * 1e-6, 1e-4), x * 1e-4, rtol=1e-4)            # eps sits inside the root
    o = torch.randn(3, 2, 5, generator=torch.Generator().manual_seed(1))
    w, g = torch.ones(10), torch.full((3, 10), 50.0)
    per, all_ = R.head_norm_gate(o, w, g, 0.0).view(3, 2, 5), R.all_norm_gate(o, w, g, 0.0).view(3, 2, 5)
    assert torch.allclose((per ** 2).mean(-1), torch.ones(3, 2), atol=1e-5)
    assert torch.allclose((all_ ** 2).mean((1, 2)), torch.ones(3), atol=1e-5) and not torch.allclose(per, all_)
    assert abs(float(R.gelu_tanh(torch.tensor(1.0))) - 0.841192) < 1e-6


def test_restatement_recurrences():
    g = torch.Generator().manual_seed(2)
    T, H, d, dv = 9, 2, 3, 4
    q, k, v = (torch.randn(T, H, n, generator=g, dtype=torch.float64) for n in (d, d, dv))
    # constant decay: the closed sum
    o, S = R.decayed_memory(q, k, v, (0.5, 1.0))
    for t in (0, 4, 8):
        want = sum(torch.tensor([0.5, 1.0], dtype=torch.float64)[:, None] ** (t - j) * (q[t] * k[j]).sum(-1, keepdim=True) * v[j] for j in range(t + 1))
        assert torch.allclose(o[t], want)
    o1, S1 = R.decayed_memory(q[:4], k[:4], v[:4], (0.5, 1.0))
    o2, S2 = R.decayed_memory(q[4:], k[4:], v[4:], (0.5, 1.0), S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)
    # matrix memory: the stabiliser only scales, so the ratio follows from plain exponentials
    a, b = R.mlstm_gates(torch.randn(T, H, generator=g, dtype=torch.float64) * 3, torch.randn(T, H, generator=g, dtype=torch.float64) * 3, 5.0)
    assert float(a.abs().max()) < 5.0 and float(b.max()) < 0.0
    o, (C, n, m) = R.mlstm_memory(q, k, v, a, b)
    Fs = torch.cumsum(b, 0)
    for t in (0, 3, 8):
        mt = torch.maximum(Fs[t], torch.stack([Fs[t] - Fs[j] + a[j] for j in range(t + 1)]).amax(0))       # the maximum starts at 0
        wgt = [torch.exp(Fs[t] - Fs[j] + a[j] - mt) for j in range(t + 1)]
        num = sum(wgt[j][:, None] * (q[t] * k[j]).sum(-1, keepdim=True) * v[j] for j in range(t + 1))
        nq = sum(wgt[j] * (q[t] * k[j]).sum(-1) for j in range(t + 1))
        assert torch.allclose(o[t], num / (torch.maximum(nq.abs(), torch.exp(-mt)) + 1e-6)[:, None])
    o1, s1 = R.mlstm_memory(q[:4], k[:4], v[:4], a[:4], b[:4])
    o2, s2 = R.mlstm_memory(q[4:], k[4:], v[4:], a[4:], b[4:], s1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(s2[2], m)


def test_restatement_is_causal_and_uses_the_tied_table():
    d = _cfg()
    st = R.random_state(d, seed=3)
    toks = np.random.default_rng(0).integers(0, 160, 30).tolist()
    z = R.forward(st, d, toks)
    assert z.shape == (30, 160)
    other = toks[:20] + [(t + 1) % 160 for t in toks[20:]]
    z2 = R.forward(st, d, other)
    assert torch.allclose(z[:20], z2[:20], atol=1e-5) and not torch.allclose(z[20], z2[20], atol=1e-3)
    st2 = dict(st, embed=st["embed"].clone())
    unused = next(t for t in range(160) if t not in toks)
    st2["embed"][unused] = 0.0                                # only the head reads this row
    z3 = R.forward(st2, d, toks)
    rest = [t for t in range(160) if t != unused]
    assert float(z3[:, unused].abs().max()) == 0.0 and torch.equal(z3[:, rest], z[:, rest])
