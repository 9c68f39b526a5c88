"""Hybrid decoders of the Rigazen design on the GPU against the plain restatement in
oracle/rigazen_ref.py: every mechanism alone -- the norm on a sub-layer's output with its activation
copy, whole-row norms with rotation and page writes, the windowed attention with kept first tokens in
its three forms, the linear attention with constant decays and the matrix memory with exponential
gates in their tiled and their one-token form, the per-layer token input in both forms -- then the
whole model through the engine: whole prompts, token-by-token decoding, portions down to two tokens,
mixed batches, reused pages and slots, window and page edges, other sizes, and greedy generation
through LLM.generate.  Small seeded configurations made here; float32 runs carry the sharp bars,
bfloat16 a loose one."""
import numpy as np
import pytest
import torch

pytestmark = pytest.mark.gpu

from oracle import rigazen_ref as R  # noqa: E402


def _par(left, right, scales=(0.9, 1.2)):
    return {"left": left, "right": right, "left_scale": scales[0], "right_scale": scales[1]}


def _left(heads, kv_heads, dim, vdim, size, keep, rot=None, scale=0.25):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size:
        m["mask"] = {"size": size, "keep_first": keep}
    if rot:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
    return m


def _right(dim, vdim, decay):
    return {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}


def _mem(heads, dim, vdim, cap):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


CONFIGS = {
    # grouped heads, values wider and narrower than keys, windows that end inside a page, one to nine kept tokens,
    # part of a head rotated, no feed-forward in one layer, a matrix memory first
    "mix": {"architecture": "Rigazen", "width": 80, "vocab": 150, "norm": {"eps": 1e-5}, "embedding": {"scale": 6.0},
            "token_side": {"dim": 12},
            "layers": [{"type": "mlstm", "mixer": _mem(3, 16, 24, 8.0), "mlp": _dense(96)},
                       {"type": "parallel", "mixer": _par(_left(6, 2, 16, 24, 20, 3, (8, 500.0)), _right(16, 12, (0.4, 0.97, 1.0))), "mlp": None},
                       {"type": "parallel", "mixer": _par(_left(3, 3, 24, 8, 7, 9, (24, 10000.0)), _right(8, 20, (0.999,)), (-0.5, 0.7)),
                        "mlp": _dense(56)},
                       {"type": "mlstm", "mixer": _mem(2, 24, 16, 15.0), "mlp": _dense(40)}]},
    # one head of everything, a window of one token, no window at all, no rotation, a decay of zero, no embedding
    # scale, one side number, equal scales of one
    "plain": {"architecture": "Rigazen", "width": 48, "vocab": 99, "norm": {"eps": 1e-6}, "token_side": {"dim": 1},
              "layers": [{"type": "parallel", "mixer": _par(_left(2, 1, 16, 16, 1, 1), _right(16, 16, (0.0, 0.9)), (1.0, 1.0)), "mlp": _dense(48)},
                         {"type": "mlstm", "mixer": _mem(1, 8, 8, 1.0), "mlp": None},
                         {"type": "parallel", "mixer": _par(_left(1, 1, 136, 40, 0, 0, (64, 10000.0), 0.1), _right(8, 8, (1.0,))), "mlp": None},
                         {"type": "parallel", "mixer": _par(_left(4, 4, 8, 12, 33, 0, (8, 100.0), 0.5), _right(20, 4, (0.5,))), "mlp": _dense(24)}]},
    # sizes that the matrix-core attentions (LDS-staged with equal and unequal key and value sizes, tiles with 32-wide
    # keys), the tiled weight stream (width 512) and the two-product token input (512 x 384 numbers) cover in 16 bits
    "wide": {"architecture": "Rigazen", "width": 512, "vocab": 384, "norm": {"eps": 1e-6}, "embedding": {"scale": 20.0},
             "token_side": {"dim": 384},
             "layers": [{"type": "parallel", "mixer": _par(_left(8, 2, 64, 64, 40, 5, (32, 10000.0), 0.125), _right(64, 64, (0.7, 0.98, 0.999))),
                         "mlp": _dense(1024)},
                        {"type": "mlstm", "mixer": _mem(4, 64, 128, 10.0), "mlp": _dense(512)},
                        {"type": "parallel", "mixer": _par(_left(6, 3, 128, 64, 100, 2, (128, 1e6), 0.1), _right(32, 48, (0.9, 0.99))), "mlp": None},
                        {"type": "parallel", "mixer": _par(_left(6, 2, 32, 48, 50, 40, (16, 1000.0), 0.2), _right(128, 16, (0.95,))),
                         "mlp": _dense(256)}]},
    # a width that is no multiple of 8, head sizes that no tile covers, heads * vdim that is no multiple of 8, no
    # token input
    "odd": {"architecture": "Rigazen", "width": 90, "vocab": 101, "norm": {"eps": 1e-5}, "embedding": {"scale": 3.0},
            "layers": [{"type": "parallel", "mixer": _par(_left(5, 5, 24, 7, 96, 11, (10, 77.0)), _right(21, 9, (0.6, 0.95, 0.99))), "mlp": _dense(50)},
                       {"type": "mlstm", "mixer": _mem(5, 22, 13, 6.5), "mlp": _dense(30)},
                       {"type": "parallel", "mixer": _par(_left(3, 1, 20, 9, 10, 2, (20, 10000.0)), _right(5, 33, (0.9,))), "mlp": None}]},
}
_cache = {}


def _weights(name):
    if ("w", name) not in _cache:
        _cache[("w", name)] = R.random_state(CONFIGS[name], seed=len(name))
    return _cache[("w", name)]


def _engine(name, dtype="float32", pages=40, max_model_len=320):
    from mi355_decode.config import EngineArgs, ModelConfig
    from mi355_decode.llm import build_engine
    key = (name, dtype, pages, max_model_len)
    if key not in _cache:
        torch.backends.cuda.matmul.allow_tf32 = False
        _cache[key] = build_engine(EngineArgs(model=name, dtype=dtype, max_num_seqs=4, max_model_len=max_model_len,
                                              num_gpu_blocks_override=pages, gpu_memory_utilization=0.0,
                                              max_num_batched_tokens=1 << 20),
                                   state_dict=_weights(name), model_config=ModelConfig.from_dict(CONFIGS[name]))
    eng = _cache[key]
    assert not eng.seqs and eng.alloc.num_free == pages and eng.slots.num_free == 4
    return eng


def _tokens(name, n, seed):
    return np.random.default_rng(seed).integers(0, CONFIGS[name]["vocab"], n).tolist()


def _ref(name, toks):
    key = ("ref", name, tuple(toks))
    if key not in _cache:
        with torch.no_grad():
            _cache[key] = R.forward(_weights(name), CONFIGS[name], toks, torch.float64).float().numpy()
    return _cache[key]


def _close(got, want, tol=3e-4):
    scale = float(np.abs(want).max())
    err = float(np.abs(got - want).max())
    assert err <= tol * scale, f"max |diff| {err:.3e} on a scale of {scale:.3f}"


def _near(got, want, tol):
    """Tensors; the difference relative to the largest number."""
    got, want = got.float().cpu(), want.float().cpu()
    assert torch.isfinite(got).all()
    err, scale = float((got - want).abs().max()), float(want.abs().max())
    assert err <= tol * scale, f"max |diff| {err:.3e} on a scale of {scale:.3f}"


def _run_cuts(eng, rid, toks, cuts):
    """Feeds toks in portions `cuts` (the last portion takes the rest), all positions wanted."""
    rows, at = [], 0
    sizes = list(cuts)
    while at < len(toks):
        n = min(sizes.pop(0) if sizes else len(toks) - at, len(toks) - at)
        rows.append(eng.forced_step([(rid, toks[at:at + n], list(range(n)))], [rid] if at + n == len(toks) else []))
        at += n
    return np.concatenate(rows)


def b16(t):
    return t.to(torch.bfloat16)


# ------------------------------------------------------------------------------------------ #
# mechanisms alone: pointwise
# ------------------------------------------------------------------------------------------ #
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W", [9, 64, 90, 2056, 4104, 8200])
def test_norm_of_a_sub_layers_output(dtype, W):
    """resid += rms(y * c) * w for widths with and without the vector form, small y (so that eps counts), and
    the activation copy of the new residual."""
    from mi355_decode import ops
    g = torch.Generator().manual_seed(W)
    x, y, w = torch.randn(5, W, generator=g) * 4, (torch.randn(5, W, generator=g) * 3).to(dtype), torch.randn(W, generator=g) * 0.2 + 1.0
    y[3] *= 1e-3
    for c in (1.0, -0.4):
        want = x.double() + R.rms(y.double() * c, 1e-5) * w.double()
        got, act = x.cuda(), torch.full((5, W), float("nan"), dtype=dtype, device="cuda")
        ops.norm_resid_f32(got, y.cuda(), w.cuda(), 1e-5, y_scale=c, act_out=act)
        _near(got, want, 1e-6)
        assert torch.equal(act.cpu(), got.cpu().to(dtype))
        got2 = x.cuda()
        ops.norm_resid_f32(got2, y.cuda(), w.cuda(), 1e-5, y_scale=c)
        assert torch.equal(got, got2)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_scaled_embedding_with_its_activation_copy(dtype):
    from mi355_decode import ops
    embed = torch.randn(31, 45, generator=torch.Generator().manual_seed(0)).to(dtype)
    ids = torch.tensor([3, 30, 0, 3, 17])
    act = torch.full((5, 45), float("nan"), dtype=dtype, device="cuda")
    got = ops.embed_scale_f32(embed.cuda(), ids.cuda(), 7.3, act_out=act)
    _near(got, embed.float()[ids] * 7.3, 1e-6)
    assert torch.equal(act.cpu(), got.cpu().to(dtype))


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-6), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("W,n,layers", [(40, 8, 3), (90, 5, 2), (33, 1, 4), (512, 48, 2), (264, 130, 2)])
def test_per_layer_token_input_in_both_forms(dtype, tol, W, n, layers):
    from mi355_decode import ops
    g = torch.Generator().manual_seed(W + n)
    V, T = 23, 7
    st = {"side.embed": torch.randn(V, layers * n, generator=g).to(dtype), "side.gate": (torch.randn(n, W, generator=g) * W ** -0.5).to(dtype),
          "side.proj": (torch.randn(W, n, generator=g) * n ** -0.5).to(dtype), "side.norm": torch.randn(W, generator=g)}
    x, ids = torch.randn(T, W, generator=g) * 2, torch.randint(0, V, (T,), generator=g)
    d = lambda k: st[k].cuda()                                # noqa: E731
    for i in range(layers):
        want = x.double() + R.token_side({k: v.double() for k, v in st.items()}, "", i, n, ids, x.double(), 1e-5)
        got, act = x.cuda(), torch.empty(T, W, dtype=dtype, device="cuda")
        ops.token_side_f32(got, d("side.gate"), d("side.proj"), d("side.norm"), d("side.embed"), i * n, ids.cuda(), 1e-5, act_out=act)
        _near(got, want, 3e-6)                                # (float32 inside whatever the storage type)
        assert torch.equal(act.cpu(), got.cpu().to(dtype))
        got = x.cuda()
        z = torch.mm(x.cuda().to(dtype), d("side.gate").t())
        y = torch.mm(ops.token_gate_rows(z, d("side.embed"), i * n, ids.cuda()), d("side.proj").t())
        ops.norm_resid_f32(got, y, d("side.norm"), 1e-5)
        _near(got, want, tol)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 3e-6), (torch.bfloat16, 1e-2)])
@pytest.mark.parametrize("n", [12, 515, 1000, 2048, 3000, 8192])
def test_gated_norm_over_all_heads_at_once(dtype, tol, n):
    """One norm over the whole row, into a column slice of a wider row that keeps its other columns."""
    from mi355_decode import ops
    g = torch.Generator().manual_seed(n)
    o, gate, w = torch.randn(3, n, generator=g), (torch.randn(3, n + 8, generator=g) * 2).to(dtype), torch.randn(n, generator=g)
    row = torch.full((3, n + 24), 7.0, dtype=dtype, device="cuda")
    ops.gated_head_rms_norm(o.view(3, 1, n).cuda(), gate.cuda()[:, 8:], w.cuda(), 1e-5, ops.ACT_SIGMOID, out=row[:, 16: 16 + n])
    _near(row[:, 16: 16 + n], R.all_norm_gate(o.view(3, 4 if n % 4 == 0 else 1, -1), w, gate.float()[:, 8:], 1e-5), tol)
    assert (row[:, :16] == 7.0).all() and (row[:, 16 + n:] == 7.0).all()


# ------------------------------------------------------------------------------------------ #
# mechanisms alone: the attention
# ------------------------------------------------------------------------------------------ #
def _pages(T, G, d, dv, dtype, spare=3, seed=0):
    """A shuffled page table for one sequence of T tokens over NaN-filled pools."""
    n = -(-T // 16)
    order = torch.randperm(n + spare, generator=torch.Generator().manual_seed(seed))[:n]
    kc = torch.full((n + spare, G, 16, d), float("nan"), dtype=dtype, device="cuda")
    vc = torch.full((n + spare, G, dv, 16), float("nan"), dtype=dtype, device="cuda")
    slots = (order[torch.arange(T) // 16] * 16 + torch.arange(T) % 16).cuda()
    return kc, vc, order.to(torch.int32).view(1, n).cuda(), slots


def _table(rot, T):
    from mi355_decode.hybrid_runner import rotary_table
    return rotary_table(rot[0] if rot else 0, rot[1] if rot else 1.0, T + 16, "cuda", exact=True)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-6), (torch.bfloat16, 1e-2)])
@pytest.mark.parametrize("H,G,d,dv,rot", [(6, 2, 16, 24, (8, 500.0)), (3, 3, 24, 8, (24, 1e4)), (5, 1, 20, 9, None), (16, 4, 128, 64, (64, 1e6)),
                                          (1, 1, 7, 3, (6, 30.0))])
def test_row_norms_rotation_and_page_writes(dtype, tol, H, G, d, dv, rot):
    """The norms run over all heads of a row (one loud head quiets the others), weights differ per channel, and
    rotation follows them; a row without a slot leaves the pages alone."""
    from mi355_decode import ops
    g = torch.Generator().manual_seed(H * 10 + d)
    T = 37
    q, k, v = torch.randn(T, H * d, generator=g), torch.randn(T, G * d, generator=g), torch.randn(T, G * dv, generator=g)
    q[:, :d] *= 6.0
    wq, wk = torch.randn(H * d, generator=g) + 1.0, torch.randn(G * d, generator=g) + 1.0
    q, k, v = q.to(dtype), k.to(dtype), v.to(dtype)
    spec = {"dims": rot[0], "base": rot[1]} if rot else None
    qr = R.rotate((R.rms(q.double(), 1e-5) * wq).view(T, H, d), spec)
    kr = R.rotate((R.rms(k.double(), 1e-5) * wk).view(T, G, d), spec)
    kc, vc, bt, slots = _pages(T, G, d, dv, dtype)
    slots = slots.clone()
    slots[5] = -1
    width = H * d + G * d + G * dv
    buf = torch.cat([q, k, v, torch.zeros(T, 5, dtype=dtype)], dim=1).cuda().contiguous()
    ops.row_norm_rope_kv_write(buf[:, : H * d], buf[:, H * d: H * d + G * d], buf[:, H * d + G * d: width], wq.cuda(), wk.cuda(),
                               _table(rot, T), torch.arange(T).cuda(), slots, kc, vc, H, G, d, dv, 1e-5)
    _near(buf[:, : H * d], qr.reshape(T, -1), tol)
    assert torch.equal(buf[:, H * d: width].cpu(), torch.cat([k, v], 1)) and (buf[:, width:] == 0).all()
    at = slots.cpu()
    for t in range(T):
        if t == 5:
            p = int(bt[0, 0])
            assert torch.isnan(kc[p, :, 5].float()).all() and torch.isnan(vc[p, :, :, 5].float()).all()
            continue
        page, off = int(at[t]) // 16, int(at[t]) % 16
        _near(kc[page, :, off], kr[t], tol * 3)
        assert torch.equal(vc[page, :, :, off].cpu().reshape(-1), v[t])


FORMS = ("rows", "tiles", "staged")


def _attend_in_cuts(q, k, v, cuts, size, keep, scale, rot=None, form="rows", splits=0, out_scale=1.0):
    """q [T, H, d], k [T, G, d], v [T, G, dv] unrotated: rotation, page write and attention through the
    product's kernels, portion by portion, over shuffled NaN-filled pages; the output lands in a column
    slice of a wider NaN-filled row."""
    from mi355_decode import ops
    T, H, d = q.shape
    G, dv, dt = k.shape[1], v.shape[2], q.dtype
    kc, vc, bt, slots = _pages(T, G, d, dv, dt)
    table = _table(rot, T)
    outs, at = [], 0
    cuts = list(cuts) + ([T - sum(cuts)] if sum(cuts) < T else [])
    for n in cuts:
        pos = torch.arange(at, at + n, dtype=torch.int64, device="cuda")
        width = (H + G) * d + G * dv
        buf = torch.cat([q[at:at + n].reshape(n, -1), k[at:at + n].reshape(n, -1), v[at:at + n].reshape(n, -1),
                         torch.zeros(n, -width % 8, dtype=dt)], dim=1).cuda().contiguous()
        qs, ks, vs = buf[:, : H * d], buf[:, H * d: (H + G) * d], buf[:, (H + G) * d: width]
        ops.rope_partial_kv_write(qs, ks, vs, table, pos, slots[at:at + n], kc, vc, H, G, d, dv)
        row = torch.full((n, H * dv + 16), float("nan"), dtype=dt, device="cuda")
        out = row[:, 8: 8 + H * dv]
        if form == "staged":
            assert ops.chunk_attn_prefill_ok(dt, H, G, d, dv)
            ops.paged_attn_prefill_ext(qs, kc, vc, bt, torch.tensor([0, n], dtype=torch.int32, device="cuda"),
                                       torch.tensor([at + n], dtype=torch.int32, device="cuda"), n, H, G, d, scale, window=size,
                                       keep=keep, out=out, out_scale=out_scale)
        else:
            tiles = torch.from_numpy(ops.query_tiles(np.array([0, n]))).cuda() if form == "tiles" else None
            ops.softmax_bias_attn(qs, kc, vc, bt, torch.zeros(n, dtype=torch.int32, device="cuda"), pos, None, None, None, H, scale,
                                  window=size, keep=keep, tiles=tiles, num_splits=splits, out=out, out_scale=out_scale)
        assert torch.isnan(row[:, :8]).all() and torch.isnan(row[:, 8 + H * dv:]).all()
        outs.append(out.float().cpu())
        at += n
    return torch.cat(outs)


def _attend_ref(q, k, v, size, keep, scale, rot=None):
    spec = {"dims": rot[0], "base": rot[1]} if rot else None
    q, k, v = q.double(), k.double(), v.double()
    return R.attend(R.rotate(q, spec), R.rotate(k, spec), v, scale, size, keep).float()


CUTS = ([1] * 90, [2, 3, 1, 30, 2, 16, 21], [90])


@pytest.mark.parametrize("H,G,d,dv,size,keep,rot", [(6, 2, 16, 24, 20, 3, (8, 500.0)), (3, 3, 24, 8, 7, 9, (24, 1e4)), (2, 1, 32, 48, 64, 2, (32, 100.0)),
                                                    (4, 4, 20, 20, 1, 1, None), (4, 1, 8, 12, 0, 0, (8, 100.0)), (1, 1, 136, 40, 30, 40, (64, 1e4)),
                                                    (2, 2, 8, 300, 17, 66, None), (5, 5, 24, 7, 1000, 4, None), (4, 2, 12, 10, 13, 0, None)])
def test_window_attention_by_rows(H, G, d, dv, size, keep, rot):
    g = torch.Generator().manual_seed(H * 100 + d)
    T = 90
    q, k, v = torch.randn(T, H, d, generator=g), torch.randn(T, G, d, generator=g), torch.randn(T, G, dv, generator=g)
    ref = _attend_ref(q, k, v, size, keep, 0.3, rot)
    for cuts in CUTS:
        _near(_attend_in_cuts(q, k, v, cuts, size, keep, 0.3, rot), ref, 3e-5)
    _near(_attend_in_cuts(q, k, v, [90], size, keep, 0.3, rot, out_scale=-0.7), ref * -0.7, 3e-5)
    q, k, v = b16(q), b16(k), b16(v)
    _near(_attend_in_cuts(q, k, v, [40, 2, 1, 47], size, keep, 0.3, rot), _attend_ref(q, k, v, size, keep, 0.3, rot), 3e-2)


@pytest.mark.parametrize("H,G,d,dv,size,keep,rot", [(6, 2, 32, 16, 20, 3, (8, 500.0)), (3, 3, 64, 48, 7, 33, (24, 1e4)), (8, 2, 64, 32, 48, 17, (32, 1e4)),
                                                    (4, 4, 96, 16, 1, 1, None), (8, 1, 32, 64, 0, 0, (32, 100.0)), (2, 1, 128, 128, 40, 5, (64, 1e4)),
                                                    (12, 2, 32, 80, 17, 70, None), (5, 1, 64, 128, 33, 0, (64, 1e6))])
def test_window_attention_on_the_matrix_cores(H, G, d, dv, size, keep, rot):
    """bfloat16; the restatement sees the same rounded inputs.  Keys spread over one, three and seven workgroups,
    so that some of them hold kept keys only, or none."""
    g = torch.Generator().manual_seed(H * 100 + d)
    T = 150
    q, k, v = b16(torch.randn(T, H, d, generator=g)), b16(torch.randn(T, G, d, generator=g)), b16(torch.randn(T, G, dv, generator=g))
    ref = _attend_ref(q, k, v, size, keep, 0.3, rot)
    for splits in (0, 3, 7):
        for cuts in ([T], [1] * T, [2, 3, 1, 30, 2, 16, 21, 1]):
            _near(_attend_in_cuts(q, k, v, cuts, size, keep, 0.3, rot, form="tiles", splits=splits, out_scale=1.5), ref * 1.5, 3e-2)


@pytest.mark.parametrize("T", [75, 300])
@pytest.mark.parametrize("H,G,d,dv,size,keep,rot", [(8, 2, 64, 64, 48, 3, (32, 1e4)), (4, 4, 64, 128, 7, 17, (24, 1e4)), (16, 4, 128, 64, 20, 70, (8, 500.0)),
                                                    (6, 1, 128, 128, 0, 0, (64, 1e4)), (3, 1, 64, 128, 33, 1, None), (16, 1, 128, 128, 100, 4, (128, 100.0)),
                                                    (2, 2, 128, 64, 1, 0, None), (12, 3, 64, 64, 64, 130, (64, 5e5)), (5, 1, 64, 64, 129, 64, None)])
def test_window_attention_staged_through_lds(H, G, d, dv, size, keep, rot, T):
    """The form for prompts and portions: walks that take the kept keys' intervals first and then start several
    steps into the sequence, equal and unequal key and value sizes."""
    g = torch.Generator().manual_seed(H * 100 + d + T)
    q, k, v = b16(torch.randn(T, H, d, generator=g)), b16(torch.randn(T, G, d, generator=g)), b16(torch.randn(T, G, dv, generator=g))
    ref = _attend_ref(q, k, v, size, keep, 0.3, rot)
    for cuts in ([T], [2, 3, 1, 30, 2, 16, 21], [T // 2 + 3, 1, 1, 2]) + (([1] * T,) if T == 75 else ()):
        _near(_attend_in_cuts(q, k, v, cuts, size, keep, 0.3, rot, form="staged", out_scale=0.6), ref * 0.6, 3e-2)


@pytest.mark.parametrize("size,keep", [(16, 3), (17, 1), (31, 16), (48, 17), (64, 4), (65, 40), (200, 2)])
def test_window_and_kept_edges_show_with_one_loud_key(size, keep):
    """Keys that every query scores far above all others, each with a value channel of its own: the last kept token
    (heard by everyone after it), the first token that is not kept and one in the middle (heard while inside the
    window: at a distance of size - 1 and not at size)."""
    H, G, d, dv = 2, 1, 64, 64
    mid = keep + size + 5
    T = mid + size + 20
    g = torch.Generator().manual_seed(size)
    base = torch.zeros(T, H, d), torch.randn(T, G, d, generator=g) * 0.1, torch.randn(T, G, dv, generator=g) * 0.1
    rot = (8, 100.0)
    for loud, channel in ((keep - 1, 5), (keep, 6), (mid, 7)):
        q, k, v = (t.clone() for t in base)
        k[:, :, 30] = 0.0                                    # (an unrotated coordinate: rotation covers the first 8)
        k[loud, 0] = 0.0
        k[loud, 0, 30] = 4.0
        q[:, :, 30] = 4.0                                    # score 16 on that key, near 0 on all others
        v[:, :, channel] = 0.0
        v[loud, 0, channel] = 5.0
        ref = _attend_ref(q, k, v, size, keep, 1.0, rot)
        heard = [t for t in range(T) if float(ref[t, channel]) > 4.9 and float(ref[t, dv + channel]) > 4.9]
        quiet = [t for t in range(T) if abs(float(ref[t, channel])) < 1e-3]
        assert heard == list(range(loud, T if loud < keep else loud + size)) and len(heard) + len(quiet) == T
        edge = (heard[-1] if loud >= keep else loud + size) - 1
        for cuts in ([T], [edge, 1, 1, 1, 1], [5, 2] + [1] * (T - 7), [loud + 1, size - 2, 2, 2] if size > 2 else [loud + 1, 2, 2]):
            _near(_attend_in_cuts(q, k, v, cuts, size, keep, 1.0, rot), ref, 1e-4)
            r16 = _attend_ref(b16(q), b16(k), b16(v), size, keep, 1.0, rot)
            _near(_attend_in_cuts(b16(q), b16(k), b16(v), cuts, size, keep, 1.0, rot, form="tiles", splits=4), r16, 3e-2)
            if len(cuts) < 20:
                _near(_attend_in_cuts(b16(q), b16(k), b16(v), cuts, size, keep, 1.0, rot, form="staged"), r16, 3e-2)


def test_far_positions_keep_the_digits_of_their_angles():
    from mi355_decode.hybrid_runner import rotary_table
    rot = {"dims": 12, "base": 50.0}
    x = torch.randn(3, 1, 12, generator=torch.Generator().manual_seed(0), dtype=torch.float64)
    table = rotary_table(12, 50.0, 40003, "cuda", exact=True).cpu().double()[40000:]
    want = R.rotate(x, rot, first=40000)
    c, s = table[:, None, :6], table[:, None, 6:]
    got = torch.cat([x[..., :6] * c - x[..., 6:] * s, x[..., 6:] * c + x[..., :6] * s], -1)
    assert (got - want).abs().max() < 1e-6


# ------------------------------------------------------------------------------------------ #
# mechanisms alone: the recurrences
# ------------------------------------------------------------------------------------------ #
def _chunk(at, n, slot):
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device="cuda")     # noqa: E731
    return i32([0, n]), torch.arange(at, at + n, dtype=torch.int64, device="cuda"), i32([slot])


def _decay_in_cuts(q, k, v, decay, cuts, tiled, rows=None, slot=1):
    """Pre-activation q, k [T, H, d], v [T, H, dv]: the constant-decay recurrence in portions on a junk-filled slot."""
    from mi355_decode import ops
    T, H, d = q.shape
    dv = v.shape[2]
    ld = torch.tensor([np.log(x) if x > 0 else -1e30 for x in decay], dtype=torch.float64, device="cuda")
    state = torch.full((3, H, ops.linear_attn_state_floats(d, dv, False)), 1e30, device="cuda")
    rows = rows or ops.linear_attn_tile_rows(d, dv)
    outs, at = [], 0
    cuts = list(cuts) + ([T - sum(cuts)] if sum(cuts) < T else [])
    for n in cuts:
        buf = torch.cat([q[at:at + n].reshape(n, -1), k[at:at + n].reshape(n, -1), v[at:at + n].reshape(n, -1)], 1).cuda().contiguous()
        cu, pos, sl = _chunk(at, n, slot)
        o = ops.decay_attn(buf[:, : H * d], buf[:, H * d: 2 * H * d], buf[:, 2 * H * d:], ld, state, cu, pos, sl, H, d, dv,
                           tiles=ops.RowTiles([0, n], rows, "cuda") if tiled else None)
        outs.append(o.cpu())
        at += n
    assert (state[0] == 1e30).all() and (state[2] == 1e30).all(), "another slot was touched"
    return torch.cat(outs)


def _decay_ref(q, k, v, decay):
    s = torch.nn.functional.silu
    return R.decayed_memory(s(q.double()), s(k.double()), s(v.double()), decay)[0].float()


@pytest.mark.parametrize("d,dv,decay", [(16, 16, (0.5, 0.99)), (8, 20, (1.0,)), (21, 9, (0.6, 0.95, 0.999)), (64, 48, (0.0, 0.9)), (128, 128, (0.97,)),
                                        (5, 33, (0.2, 1.0)), (200, 24, (0.99,)), (256, 256, (0.999,)), (24, 300, (0.9,))])
def test_constant_decay_in_both_forms(d, dv, decay):
    g = torch.Generator().manual_seed(d + dv)
    T, H = 150, len(decay)
    q, k, v = torch.randn(T, H, d, generator=g), torch.randn(T, H, d, generator=g), torch.randn(T, H, dv, generator=g)
    ref = _decay_ref(q, k, v, decay)
    for cuts in ([T], [2, 3, 64, 1, 63, 2], [65, 85], [1] * 20):
        _near(_decay_in_cuts(q, k, v, decay, cuts, True), ref, 5e-6)
    for cuts in ([1] * T, [2, 3, 1, 4, 2, 138]):
        _near(_decay_in_cuts(q, k, v, decay, cuts, False), ref, 5e-6)
    _near(_decay_in_cuts(q, k, v, decay, [70], True, rows=16), ref, 5e-6)
    q, k, v = b16(q), b16(k), b16(v)
    ref = _decay_ref(q, k, v, decay)
    for cuts, tiled in (([100, 50], True), ([1] * T, False), ([40, 2, 2, 60], True)):
        _near(_decay_in_cuts(q, k, v, decay, cuts, tiled), ref, 5e-6)      # (float32 inside: only the inputs are rounded)


def test_a_value_written_early_is_read_far_behind():
    """Decay one: the first token's value comes back 400 tokens later through a key that nothing else uses; with
    a decay of 0.9 it is gone."""
    T, H, d, dv = 401, 2, 8, 8
    q, k, v = torch.full((T, H, d), -30.0), torch.full((T, H, d), -30.0), torch.randn(T, H, dv, generator=torch.Generator().manual_seed(1))
    k[0, :, 3], q[T - 1, :, 3] = 3.0, 3.0                       # (silu(-30) is zero)
    ref = _decay_ref(q, k, v, (1.0, 0.9))
    assert float(ref[-1, 0].abs().max()) > 1.0 and float(ref[-1, 1].abs().max()) < 1e-6
    for cuts, tiled in (([T], True), ([200, 2, 2, 197], True), ([1] * T, False)):
        got = _decay_in_cuts(q, k, v, (1.0, 0.9), cuts, tiled)
        _near(got[-1, 0], ref[-1, 0], 1e-5)
        assert float(got[-1, 1].abs().max()) < 1e-6


def _mem_case(T, H, d, dv, W, seed, dtype=torch.float32, ib=0.0, fb=2.0, spread=3.0):
    g = torch.Generator().manual_seed(seed)
    r = lambda *s, m=1.0: (torch.randn(*s, generator=g) * m).to(dtype)     # noqa: E731
    x = torch.randn(T, W, generator=g)
    return {"q": r(T, H, d), "k": r(T, H, d), "v": r(T, H, dv), "g": r(T, H * dv, m=2.0), "x": x,
            "w": r(2 * H, W, m=spread * W ** -0.5), "b": torch.cat([torch.full((H,), ib), torch.full((H,), fb)]) + torch.randn(2 * H, generator=g),
            "norm": torch.randn(H * dv, generator=g) + 1.0}


def _mem_in_cuts(c, cap, cuts, tiled, rows=None, eps=1e-5, slot=1):
    """The matrix memory with its gates, norm and output gate in portions on a junk-filled slot."""
    from mi355_decode import ops
    T, H, d = c["q"].shape
    dv = c["v"].shape[2]
    state = torch.full((3, H, ops.linear_attn_state_floats(d, dv, True)), 1e30, device="cuda")
    mst = torch.full((3, H), 1e30, device="cuda")
    rows = rows or ops.linear_attn_tile_rows(d, dv)
    w, b, nrm = c["w"].cuda(), c["b"].float().cuda(), c["norm"].cuda()
    outs, at = [], 0
    cuts = list(cuts) + ([T - sum(cuts)] if sum(cuts) < T else [])
    for n in cuts:
        s = slice(at, at + n)
        buf = torch.cat([c["q"][s].reshape(n, -1), c["k"][s].reshape(n, -1), c["v"][s].reshape(n, -1), c["g"][s]], 1).cuda().contiguous()
        q, k, v, gt = buf[:, : H * d], buf[:, H * d: 2 * H * d], buf[:, 2 * H * d: 2 * H * d + H * dv], buf[:, 2 * H * d + H * dv:]
        x = c["x"][s].cuda().contiguous()
        cu, pos, sl = _chunk(at, n, slot)
        if tiled:
            o = ops.mlstm_chunks(q, k, v, d ** -0.5, torch.mm(x, w.float().t()), b, cap, state, mst, cu, pos, sl, H, d, dv,
                                 ops.RowTiles([0, n], rows, "cuda"))
            o = ops.gated_head_rms_norm(o, gt, nrm, eps, ops.ACT_SIGMOID)
        else:
            o = ops.mlstm_step(q, k, v, d ** -0.5, x, w, b, cap, gt, nrm, eps, state, mst, cu, pos, sl, H, d, dv)
        outs.append(o.float().cpu())
        at += n
    assert (state[0] == 1e30).all() and (state[2] == 1e30).all() and (mst[[0, 2]] == 1e30).all(), "another slot was touched"
    return torch.cat(outs)


def _mem_ref(c, cap, eps=1e-5):
    H, d = c["q"].shape[1:]
    z = c["x"].double() @ c["w"].double().T + c["b"].double()
    a, b = R.mlstm_gates(z[:, :H], z[:, H:], cap)
    o, _ = R.mlstm_memory(c["q"].double() * d ** -0.5, c["k"].double(), c["v"].double(), a, b)
    return R.head_norm_gate(o, c["norm"].double(), c["g"].double(), eps).float()


@pytest.mark.parametrize("H,d,dv,W,cap,ib,fb", [(2, 16, 16, 40, 8.0, 0.0, 2.0), (3, 24, 13, 33, 15.0, 2.0, 4.0), (1, 8, 40, 64, 1.0, -3.0, -2.0),
                                                (2, 64, 128, 64, 10.0, -6.0, 6.0), (1, 128, 128, 96, 6.5, 0.0, 5.0), (5, 22, 20, 21, 30.0, 3.0, 0.0),
                                                (1, 200, 24, 16, 12.0, 0.0, 3.0), (1, 256, 256, 16, 12.0, 0.0, 3.0), (4, 5, 7, 9, 4.0, 5.0, 9.0)])
def test_matrix_memory_in_both_forms(H, d, dv, W, cap, ib, fb):
    """Gates open and shut, weak and strong (input gates that overtake the running maximum, forget gates that
    wipe the state), in portions of every size."""
    T = 150
    c = _mem_case(T, H, d, dv, W, seed=d * 7 + dv, ib=ib, fb=fb)
    ref = _mem_ref(c, cap)
    for cuts in ([T], [2, 3, 64, 1, 63, 2], [65, 85], [1] * 20):
        _near(_mem_in_cuts(c, cap, cuts, True), ref, 2e-4)
    for cuts in ([1] * T, [2, 3, 1, 4, 2, 138]):
        _near(_mem_in_cuts(c, cap, cuts, False), ref, 2e-4)
    _near(_mem_in_cuts(c, cap, [70], True, rows=16), ref, 2e-4)
    c = _mem_case(T, H, d, dv, W, seed=d * 7 + dv, ib=ib, fb=fb, dtype=torch.bfloat16)
    ref = _mem_ref(c, cap)
    for cuts, tiled in (([100, 50], True), ([1] * T, False), ([40, 2, 2, 60], True)):
        _near(_mem_in_cuts(c, cap, cuts, tiled), ref, 1e-2)


def test_matrix_memory_over_long_prompts():
    """1 500 tokens: more tiles than one turn of the gate scan's waves, and log decays that add up to thousands
    while neighbouring tokens still differ by a fraction."""
    c = _mem_case(1500, 2, 16, 16, 24, seed=5, ib=1.0, fb=-1.0)
    ref = _mem_ref(c, 12.0)
    _near(_mem_in_cuts(c, 12.0, [1500], True), ref, 2e-4)
    _near(_mem_in_cuts(c, 12.0, [1030, 2, 400], True), ref, 2e-4)
    _near(_mem_in_cuts(c, 12.0, [1500], False), ref, 2e-4)


def test_running_maximum_starts_at_zero():
    """First tokens with shut input gates: the maximum stays at the forget gate's (near zero), so the output shrinks
    with the input gate and the denominator is exp(-m), not |n . q|: seen ahead of the norm, whose eps it meets."""
    from mi355_decode import ops
    H, d, dv, T = 1, 8, 8, 3
    c = _mem_case(T, H, d, dv, 4, seed=3)
    c["w"] *= 0.0
    c["b"] = torch.tensor([-9.0, 20.0])                         # a = -9 and f = 0, nearly, under a wide cap
    cap, eps = 100.0, 1e-5
    z = torch.zeros(T, 2 * H, dtype=torch.float64) + c["b"].double()
    a, b = R.mlstm_gates(z[:, :H], z[:, H:], cap)
    o, (_, _, m) = R.mlstm_memory(c["q"].double() * d ** -0.5, c["k"].double(), c["v"].double(), a, b)
    assert float(o.abs().max()) < 5e-3 and abs(float(m)) < 1e-6
    closed = torch.exp(a[0]) * (c["q"][0, 0].double() * d ** -0.5 @ c["k"][0, 0].double()) * c["v"][0, 0].double()
    assert torch.allclose(o[0, 0], closed, rtol=1e-3)           # (a minus-infinite start would give q.k / |q.k| v: of order one)
    state, mst = torch.zeros(1, H, ops.linear_attn_state_floats(d, dv, True), device="cuda"), torch.zeros(1, H, device="cuda")
    cu, pos, sl = _chunk(0, T, 0)
    rows = [c[n].reshape(T, -1).cuda() for n in "qkv"]
    got = ops.mlstm_chunks(*rows, d ** -0.5, torch.zeros(T, 2 * H, device="cuda"), c["b"].cuda(), cap, state, mst, cu, pos, sl, H, d, dv,
                           ops.RowTiles([0, T], 64, "cuda"))
    _near(got, o, 1e-5)
    for cuts, tiled in (([T], True), ([1] * T, False)):
        _near(_mem_in_cuts(c, cap, cuts, tiled, eps=eps), R.head_norm_gate(o, c["norm"].double(), c["g"].double(), eps), 1e-4)


def test_a_memory_held_for_four_hundred_tokens():
    """One token with an open input gate, then shut input and open forget gates: its value comes back 400 tokens
    later; the second head forgets."""
    T, H, d, dv, W, cap = 401, 2, 8, 8, 3, 40.0
    c = _mem_case(T, H, d, dv, W, seed=9)
    c["x"] = torch.zeros(T, W)
    c["x"][0, 0], c["x"][1:, 1] = 1.0, 1.0
    c["w"] = torch.zeros(2 * H, W)
    c["w"][:H, 0], c["w"][:H, 1] = 6.0, -25.0                   # input gates: open at token 0, shut after
    c["w"][H, :2] = 30.0                                        # head 0 keeps
    c["w"][H + 1, 1] = 0.5                                      # head 1 forgets a third at every token
    c["b"] = torch.zeros(2 * H)
    c["k"][0] = c["q"][-1]
    ref = _mem_ref(c, cap)
    v0 = R.head_norm_gate(c["v"][:1].double(), c["norm"].double(), c["g"][-1:].double(), 1e-5).float()[0]
    assert (ref[-1, :dv] - v0[:dv]).abs().max() < 1e-3 and (ref[-1, dv:] - v0[dv:]).abs().max() > 0.1
    for cuts, tiled in (([T], True), ([130, 2, 2, 267], True), ([1] * T, False)):
        _near(_mem_in_cuts(c, cap, cuts, tiled), ref, 5e-4)


@pytest.mark.parametrize("tiled", [True, False])
def test_packed_chunks_of_several_sequences(tiled):
    """Three sequences side by side: a portion that continues, a first token, a portion from the start on a slot that
    another sequence used; afterwards all continue with their slots permuted in the batch."""
    from mi355_decode import ops
    H, d, dv, W, cap, eps = 2, 12, 20, 10, 9.0, 1e-5
    lens = (100, 3, 70)
    cases = [_mem_case(n, H, d, dv, W, seed=40 + i) for i, n in enumerate(lens)]
    for c in cases[1:]:
        c.update(w=cases[0]["w"], b=cases[0]["b"], norm=cases[0]["norm"])
    refs = [_mem_ref(c, cap, eps) for c in cases]
    decay = (0.9, 0.99)
    drefs = [_decay_ref(c["q"], c["k"], c["v"], decay) for c in cases]
    ld = torch.tensor(np.log(decay), device="cuda")
    st, mst = torch.full((4, H, ops.linear_attn_state_floats(d, dv, True)), 3.0, device="cuda"), torch.full((4, H), 3.0, device="cuda")
    ds = torch.full((4, H, ops.linear_attn_state_floats(d, dv, False)), 3.0, device="cuda")
    slot = (2, 0, 3)
    at = [0, 0, 0]
    for order, sizes in (((0,), (41,)), ((0, 1, 2), (7, 1, 64)), ((2, 0, 1), (6, 52, 2))):
        part = {n: torch.cat([cases[s][n][at[s]: at[s] + m].reshape(m, -1) for s, m in zip(order, sizes)]).cuda() for n in "qkvgx"}
        cu_h = np.concatenate([[0], np.cumsum(sizes)])
        cu = torch.tensor(cu_h, dtype=torch.int32, device="cuda")
        pos = torch.cat([torch.arange(at[s], at[s] + m) for s, m in zip(order, sizes)]).cuda()
        sl = torch.tensor([slot[s] for s in order], dtype=torch.int32, device="cuda")
        q, k, v, g, x = (part[n].contiguous() for n in "qkvgx")
        w, b, nrm = cases[0]["w"].cuda(), cases[0]["b"].cuda(), cases[0]["norm"].cuda()
        rt = ops.RowTiles(cu_h, 32, "cuda") if tiled else None
        if tiled:
            o = ops.mlstm_chunks(q, k, v, d ** -0.5, torch.mm(x, w.t()), b, cap, st, mst, cu, pos, sl, H, d, dv, rt)
            o = ops.gated_head_rms_norm(o, g, nrm, eps, ops.ACT_SIGMOID)
        else:
            o = ops.mlstm_step(q, k, v, d ** -0.5, x, w, b, cap, g, nrm, eps, st, mst, cu, pos, sl, H, d, dv)
        do = ops.decay_attn(q, k, v, ld, ds, cu, pos, sl, H, d, dv, tiles=rt)
        for i, (s, m) in enumerate(zip(order, sizes)):
            r = slice(int(cu_h[i]), int(cu_h[i + 1]))
            _near(o[r], refs[s][at[s]: at[s] + m], 3e-4)
            _near(do[r], drefs[s][at[s]: at[s] + m], 1e-5)
            at[s] += m
    assert tuple(at) == lens


# ------------------------------------------------------------------------------------------ #
# the whole model through the engine
# ------------------------------------------------------------------------------------------ #
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_and_every_layer(name):
    eng = _engine(name)
    toks = _tokens(name, 90, 1)
    eng.runner.layer_trace = []
    try:
        got = eng.forced_step([("a", toks, list(range(len(toks))))], ["a"])
        trace = [t.cpu().numpy() for t in eng.runner.layer_trace]
    finally:
        eng.runner.layer_trace = None
    want = []
    with torch.no_grad():
        R.forward(_weights(name), CONFIGS[name], toks, torch.float64, layers_out=want)
    assert len(trace) == len(want)
    for i, (a, b) in enumerate(zip(trace, want)):
        assert np.abs(a - b.numpy()).max() <= 1e-4 * np.abs(b.numpy()).max(), f"layer {i}"
    _close(got, _ref(name, toks))


@pytest.mark.parametrize("name", list(CONFIGS))
def test_portions_and_token_by_token_equal_the_whole_prompt(name):
    eng = _engine(name)
    toks = _tokens(name, 70, 2)
    want = _ref(name, toks)
    for cuts in ([1] * 70, [2, 2, 3, 16, 1, 17, 2], [33, 2] + [1] * 35, [5] * 14):
        _close(_run_cuts(eng, "p", toks, cuts), want)


@pytest.mark.parametrize("name", ["mix", "plain"])
def test_first_tokens_and_one_token_requests(name):
    eng = _engine(name)
    for n in (1, 2, 3, 5):
        toks = _tokens(name, n, 10 + n)
        _close(_run_cuts(eng, "s", toks, [1] * n), _ref(name, toks))
        _close(_run_cuts(eng, "s", toks, [n]), _ref(name, toks))


def _run_mixed(eng, name):
    """Four requests of unequal length advance together, portions beside single tokens; requests end and new
    ones take their pages and slots.  Returns {request: (tokens, logits of all its positions)}."""
    lens = {"a": 60, "b": 23, "c": 91, "d": 2, "e": 47, "f": 35}
    toks = {r: _tokens(name, n, ord(r)) for r, n in lens.items()}
    plan = {"a": [30, 1, 1, 2, 26], "b": [2, 1, 20], "c": [16, 17, 1, 1, 1, 55], "d": [1, 1], "e": [2, 45], "f": [34, 1]}
    at = {r: 0 for r in lens}
    got = {r: [] for r in lens}
    live, waiting = ["a", "b", "c", "d"], ["e", "f"]
    step = 0
    while live:
        entries, end = [], []
        for r in list(live):
            if r == "b" and step % 2 == 1:
                continue                                            # b sits out every other step
            n = plan[r].pop(0)
            entries.append((r, toks[r][at[r]:at[r] + n], list(range(n))))
            at[r] += n
            if at[r] == lens[r]:
                end.append(r)
        out = eng.forced_step(entries, end)
        row = 0
        for r, t, _ in entries:
            got[r].append(out[row:row + len(t)])
            row += len(t)
        for r in end:
            live.remove(r)
            if waiting:
                live.append(waiting.pop(0))
        step += 1
    return {r: (toks[r], np.concatenate(got[r])) for r in lens}


@pytest.mark.parametrize("name", ["mix", "plain", "odd"])
def test_mixed_batches_equal_each_request_alone(name):
    for toks, got in _run_mixed(_engine(name, pages=24), name).values():
        _close(got, _ref(name, toks))


def _tracks(got, want, scale):
    """A head whose output nearly cancels is blown up by its norm, rounding and all: such positions (one in thirty)
    may differ by more; the others must be close."""
    d = got - want
    d = d - d.mean(1, keepdims=True)
    err = np.sqrt((d ** 2).mean(1)) / scale
    assert np.median(err) < 0.03 and (err > 0.12).sum() <= max(len(err) // 30, 1), (np.median(err), np.sort(err)[-6:])


def test_mixed_batches_in_bfloat16():
    """The same schedule in bfloat16 on the configuration whose layers take the LDS-staged attention for steps that
    hold a portion (single tokens of other requests ride along) and the tile form for single tokens only."""
    name = "wide"
    for toks, got in _run_mixed(_engine(name, dtype="bfloat16", pages=24), name).values():
        _tracks(got, _ref(name, toks), _ref(name, toks).std())


def test_pages_and_slots_are_reused_without_leaking():
    for name in ("plain", "mix"):
        eng = _engine(name, pages=8, max_model_len=128)         # one 100-token request nearly fills the pool
        for i in range(6):
            toks = _tokens(name, 100 - 7 * i, 50 + i)
            _close(_run_cuts(eng, f"r{i}", toks, [40, 3] + [1] * 10), _ref(name, toks))


@pytest.mark.parametrize("name", ["mix", "odd"])
def test_long_decoding_past_windows_and_pages(name):
    eng = _engine(name)
    toks = _tokens(name, 300, 9)
    _close(_run_cuts(eng, "long", toks, [10] + [1] * 290), _ref(name, toks), tol=6e-4)


def test_a_kept_token_and_a_window_through_the_whole_model():
    """The first tokens' value is made loud through the weights: the kept one is heard 250 tokens later, decoded
    token by token; the same token just past the kept ones is heard inside the window only."""
    from mi355_decode.config import EngineArgs, ModelConfig
    from mi355_decode.llm import build_engine
    cfg = {"architecture": "Rigazen", "width": 32, "vocab": 40, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
           "layers": [{"type": "parallel", "mixer": _par(_left(2, 1, 16, 8, 60, 3, (4, 100.0), 4.0), _right(8, 8, (0.5,)), (1.0, 0.1)), "mlp": None}]}
    w = R.random_state(cfg, seed=11)
    loud = 7
    w["embed"][:, 3] = 0.0
    w["embed"][loud, 3] = 3.0                               # only token `loud` lights coordinate 3
    L = "l0.mix.left."
    w[L + "k"][:], w[L + "k.b"][:], w[L + "k.norm"][:] = 0.0, 0.0, 1.0
    w[L + "k"][8, 3] = 4.0                                  # an unrotated key coordinate follows it; other keys are small noise
    w[L + "k.b"][9] = 0.5
    w[L + "q"][:], w[L + "q.b"][:], w[L + "q.norm"][:] = 0.0, 0.0, 1.0
    w[L + "q.b"][8] = w[L + "q.b"][16 + 8] = 1.5            # every query asks for that coordinate
    torch.backends.cuda.matmul.allow_tf32 = False
    eng = build_engine(EngineArgs(model="far", dtype="float32", max_num_seqs=4, max_model_len=320, num_gpu_blocks_override=20,
                                  gpu_memory_utilization=0.0, max_num_batched_tokens=1 << 20), state_dict=w,
                       model_config=ModelConfig.from_dict(cfg))
    for place in (2, 3):
        toks = [int(t) for t in np.random.default_rng(4).integers(8, 40, 260)]
        toks[place] = loud
        other = list(toks)
        other[place] = 9
        with torch.no_grad():
            want, quiet = R.forward(w, cfg, toks).numpy(), R.forward(w, cfg, other).numpy()
        gap = np.abs(want - quiet).max(1) / np.abs(want).max()
        assert gap[place + 59] > 0.05 and (gap[place + 60] > 0.05) == (place == 2) and (gap[-1] > 0.05) == (place == 2)
        for cuts in ([5] + [1] * 255, [place + 59, 1, 1, 1], [200, 2, 58]):
            _close(_run_cuts(eng, "f", toks, cuts), want)


@pytest.mark.parametrize("name", ["mix", "wide", "odd"])
def test_bfloat16_tracks_the_float32_restatement(name):
    """Whole prompts (library GEMMs, the staged attention, the tiled recurrences) and decode-sized steps (at width 512
    the tiled weight stream) in bfloat16 against the restatement and against each other."""
    eng = _engine(name, dtype="bfloat16")
    if name == "wide":
        assert eng.runner._tiled_w, "no tiled weight copies at width 512"
    toks = _tokens(name, 64, 4)
    want = _ref(name, toks)
    whole = _run_cuts(eng, "h", toks, [64])
    for got in (whole, _run_cuts(eng, "h", toks, [30, 2] + [1] * 32)):
        for a, b in ((got, want), (got, whole)):
            _tracks(a, b, want.std())


@pytest.mark.parametrize("name,dtype", [("mix", "float32"), ("plain", "float32"), ("wide", "bfloat16")])
def test_greedy_generation_through_the_engine(name, dtype):
    """LLM.generate: scheduler admission, prefill, then decode steps replayed from HIP graphs with
    run-ahead.  A token may leave the restatement's only where its own margin is inside the error."""
    from mi355_decode.llm import LLM
    from mi355_decode.sampling_params import SamplingParams
    eng = _engine(name, dtype=dtype)
    prompts = [_tokens(name, n, 70 + n) for n in (5, 33, 18, 1, 26)]     # five requests on four slots: one waits
    steps = 24
    for _ in range(2):                                                   # the second time every step is a replay
        outs = LLM(eng).generate(prompts, SamplingParams(max_tokens=steps, temperature=0.0, ignore_eos=True))
        assert eng.runner.use_graphs and eng.runner.graphs, "the decode steps did not run as HIP graphs"
        for p, o in zip(prompts, outs):
            assert len(o) == steps
            with torch.no_grad():
                z = R.forward(_weights(name), CONFIGS[name], p + o)[len(p) - 1: -1]
            tol = 2e-3 if dtype == "float32" else 0.3 * float(z.std())
            for t in range(steps):
                best = int(torch.argmax(z[t]))
                assert o[t] == best or float(z[t, best] - z[t, o[t]]) <= tol, f"token {t}: {o[t]} vs {best}"


def test_served_from_a_model_directory(tmp_path):
    """The OpenAI server started on a directory with config.json + model.safetensors of this design: the
    model class chosen by config.json, weights from the checkpoint names, greedy completions by token
    id against the restatement (margin rule), and a seeded sampled completion through the sampler."""
    import json
    import os
    import signal
    import socket
    import subprocess
    import sys
    import time
    from safetensors.torch import save_file
    from conftest import PKG, ROOT
    from mi355_decode.harness import BenchClient
    name = "mix"
    cfg, w = CONFIGS[name], _weights(name)
    model_dir = tmp_path / "model"
    model_dir.mkdir()
    json.dump(cfg, open(model_dir / "config.json", "w"))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in w.items()}, str(model_dir / "model.safetensors"))
    with socket.socket() as s:
        s.bind(("127.0.0.1", 0))
        port = s.getsockname()[1]
    args = ["--model", str(model_dir), "--served-model-name", "kept", "--host", "127.0.0.1", "--port", str(port),
            "--dtype", "float32", "--max-num-seqs", "4", "--max-model-len", "128"]
    env = dict(os.environ, PYTHONPATH=PKG + os.pathsep + ROOT)
    log = open(tmp_path / "server.log", "w")
    proc = subprocess.Popen([sys.executable, "-m", "mi355_decode.entrypoints.openai.api_server"] + args, env=env, stdout=log,
                            stderr=subprocess.STDOUT, start_new_session=True)
    url = f"http://127.0.0.1:{port}"
    try:
        client = BenchClient(url)
        t0 = time.time()
        while True:
            assert proc.poll() is None, open(tmp_path / "server.log").read()[-3000:]
            try:
                if client.health() == 200:
                    break
            except Exception:
                pass
            assert time.time() - t0 < 240, "server did not become healthy"
            time.sleep(0.2)
        post = lambda **body: client.http.post(f"{url}/v1/completions", json={"model": "kept", **body})   # noqa: E731
        prompt, steps = _tokens(name, 21, 5), 12
        r = post(prompt=prompt, max_tokens=steps, temperature=0, ignore_eos=True, logprobs=0, return_tokens_as_token_ids=True)
        assert r.status_code == 200, r.text
        got = [int(t.split(":")[1]) for t in r.json()["choices"][0]["logprobs"]["tokens"]]
        assert len(got) == steps
        with torch.no_grad():
            z = R.forward(w, cfg, prompt + got)[len(prompt) - 1: -1]
        for t in range(steps):
            best = int(torch.argmax(z[t]))
            assert got[t] == best or float(z[t, best] - z[t, got[t]]) <= 2e-3, f"token {t}"
        draws = [post(prompt=prompt, max_tokens=8, temperature=0.9, top_k=20, seed=7, ignore_eos=True, logprobs=0,
                      return_tokens_as_token_ids=True).json()["choices"][0]["logprobs"]["tokens"] for _ in range(2)]
        assert draws[0] == draws[1] and len(draws[0]) == 8
        assert "synthetic" not in open(tmp_path / "server.log").read()
    finally:
        os.killpg(proc.pid, signal.SIGTERM)
        try:
            proc.wait(timeout=20)
        except subprocess.TimeoutExpired:
            os.killpg(proc.pid, signal.SIGKILL)


def test_trace_replay_program(tmp_path):
    """bin/trace_run on a model directory of this design: steps as JSON lines on standard input (a
    portion beside a single token, a request that ends and one that takes its place), float32 logits
    of the wanted rows per step on disk, a 'done <step>' line after every step."""
    import json
    import os
    import subprocess
    from safetensors.torch import save_file
    from conftest import ROOT
    name = "plain"
    cfg, w = CONFIGS[name], _weights(name)
    model_dir, out_dir = tmp_path / "model", tmp_path / "out"
    model_dir.mkdir()
    json.dump(cfg, open(model_dir / "config.json", "w"))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in w.items()}, str(model_dir / "model.safetensors"))
    a, b, c = _tokens(name, 50, 1), _tokens(name, 20, 2), _tokens(name, 9, 3)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:33], "want": [0, 32]}, {"id": "b", "tokens": b[:1], "want": [0]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[1:], "want": [18]}, {"id": "a", "tokens": a[33:34], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[34:36], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "c", "tokens": c, "want": [8]}, {"id": "a", "tokens": a[36:], "want": [13]}], "end": ["a", "c"]}]
    p = subprocess.Popen([os.path.join(ROOT, "bin", "trace_run"), "--model", str(model_dir), "--dtype", "float32", "--out", str(out_dir),
                          "--max-tokens", "128"], stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    try:
        for st in steps:
            p.stdin.write(json.dumps(st) + "\n")
            p.stdin.flush()
            while True:
                line = p.stdout.readline()
                assert line, "the program ended early"
                if line.strip() == f"done {st['step']}":
                    break
        p.stdin.close()
        assert p.wait(timeout=60) == 0
    finally:
        if p.poll() is None:
            p.kill()
    V = cfg["vocab"]
    ra, rb, rc = _ref(name, a), _ref(name, b), _ref(name, c)
    want = {0: [ra[0], ra[32], rb[0]], 1: [rb[19], ra[33]], 3: [rc[8], ra[49]]}
    assert not (out_dir / "2.f32").exists()
    for n, rows in want.items():
        got = np.fromfile(out_dir / f"{n}.f32", dtype="<f4").reshape(-1, V)
        assert got.shape[0] == len(rows)
        _close(got, np.stack(rows))
