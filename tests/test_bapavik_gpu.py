"""Hybrid decoders of the Bapavik design on the GPU against the plain restatement in
oracle/bapavik_ref.py: every mechanism alone -- the layer norm with the rows it adds (a mixture's in expert
order too), whole-row norms with the query temperature, the capped attention with learned sinks in its three
forms, the latent attention with neighbours rotated on the latents (by rows and on the matrix cores) and with
expanded keys and values, the grouped products, expert orders from a table -- then the whole model through
the engine: whole prompts, token-by-token decoding, portions down to two tokens, mixed batches, reused pages
and slots, far keys and page edges, looped layers, other sizes, and greedy generation through LLM.generate.
Small seeded configurations made here; float32 runs carry the sharp bars, bfloat16 a loose one."""
from types import SimpleNamespace

import numpy as np
import pytest
import torch

pytestmark = pytest.mark.gpu

from oracle import bapavik_ref as R  # noqa: E402


def _att(heads, kv_heads, dim, vdim, scale=0.25, softcap=None, temp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if softcap:
        m["softcap"] = softcap
    if temp:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    return {"type": "attention", "mixer": m}


def _lat(heads, dim, rot, vdim, rank, base=10000.0, scale=0.2):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": scale,
                                                  "rot": {"dims": rot, "base": base}}}


def _dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def _moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def _cfg(width, vocab, layers, loop=None, scale=None, eps=1e-5):
    d = {"architecture": "Bapavik", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": [dict(a, mlp=m) for a, m in layers]}
    if scale:
        d["embedding"] = {"scale": scale}
    if loop:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


CONFIGS = {
    # grouped heads, values wider and narrower than keys, a low cap, temperatures that change every few tokens, a loop of
    # three passes in the middle, two and three experts per token, a layer without a feed-forward
    "mix": _cfg(80, 150, [(_att(6, 2, 16, 24, 0.3, 4.0, (0.7, 7)), _moe(5, 2, 24)), (_lat(3, 16, 8, 24, 32, 500.0, 0.3), None),
                          (_att(3, 3, 24, 8, 0.2, 9.0, (1.3, 16)), _dense(56, 1.2)), (_lat(5, 24, 4, 8, 16), _moe(7, 3, 40))], (1, 3, 3), 6.0),
    # one head of everything, no temperature, no cap, no loop, no embedding scale, one expert in all, a latent of one part
    "plain": _cfg(48, 99, [(_lat(1, 8, 2, 8, 8, 50.0, 0.5), _moe(1, 1, 16)), (_att(1, 1, 16, 16), _dense(48, 7.0)),
                           (_att(2, 1, 136, 40, 0.1, None, (0.4, 64)), None)], eps=1e-6),
    # sizes that the matrix cores cover in 16 bits: the LDS-staged attention with equal and unequal key and value sizes,
    # expanded latents with keys of 128 and of 192, expert tiles, the tiled weight stream (width 512); all layers loop
    "wide": _cfg(512, 384, [(_att(8, 2, 64, 64, 0.125, 20.0, (0.5, 40)), _moe(4, 1, 256)), (_lat(4, 96, 32, 64, 128, 1e4, 0.1), _dense(512, 2.0)),
                            (_att(6, 3, 128, 64, 0.1, 30.0), _moe(6, 2, 128)), (_lat(3, 128, 64, 128, 256, 1e6, 0.07), _moe(4, 1, 256))], (0, 4, 2), 20.0),
    # a width that is no multiple of 8, head sizes that no tile covers, a loop that runs once
    "odd": _cfg(90, 101, [(_att(5, 5, 21, 7, 0.3, 3.0, (0.9, 11)), _moe(3, 2, 30)), (_lat(3, 13, 6, 9, 22, 77.0), _dense(50, 0.8)),
                          (_lat(7, 20, 10, 12, 36), None)], (1, 2, 1), 3.0),
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
            _cache[key] = R.forward(_weights(name), CONFIGS[name], toks).numpy()
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


def _tracks(got, want, scale, most=0.15):
    d = got - want
    d = d - d.mean(1, keepdims=True)
    err = np.sqrt((d ** 2).mean(1)) / scale
    assert np.median(err) < most / 3 and err.max() < most, (np.median(err), np.sort(err)[-6:])


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
# mechanisms alone: norm, grouped products, expert orders
# ------------------------------------------------------------------------------------------ #
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-6), (torch.bfloat16, 1e-2), (torch.float16, 2e-3)])
@pytest.mark.parametrize("W", [9, 64, 90, 2056, 4104, 8200])
def test_layer_norm_and_what_it_adds(dtype, tol, W):
    """Widths with and without the vector form; rows far from zero mean (without the subtraction the result is wrong by
    the mean) and a row of tiny spread (eps counts); the addend none, plain rows, a mixture's rows in expert order."""
    from mi355_decode import ops
    g = torch.Generator().manual_seed(W)
    T = 5
    x, w = torch.randn(T, W, generator=g) + 20.0, (torch.randn(W, generator=g) * 0.2 + 1.0).to(dtype)
    x[3] = x[3] * 1e-3 + 0.1
    for top in (0, 1, 3):
        rows = torch.randn(T * max(top, 1), W, generator=g).to(dtype)
        if top == 0:
            want, kw = x.double(), {}
        else:
            perm = torch.randperm(T * top, generator=g)
            want = x.double() + rows.double()[perm].view(T, top, W).sum(1) * (0.3 if top > 1 else 1.0)
            kw = dict(add=rows.cuda(), inv=perm.to(torch.int32).cuda(), top=top, row_weight=0.3 if top > 1 else 1.0)
        got = x.cuda()
        out = ops.add_layer_norm_f32(got, w.cuda(), 1e-5, **kw)
        _near(got, want, 1e-6)
        _near(out, R.layer_norm(got.cpu().double(), w.double(), 1e-5), max(tol, 1e-5))
        if top:
            got = x.cuda()
            assert ops.add_layer_norm_f32(got, None, 1e-5, **kw) is None
            _near(got, want, 1e-6)
    add = torch.randn(T, W, generator=g).to(dtype)
    got = x.cuda()
    out = ops.add_layer_norm_f32(got, w.cuda(), 1e-5, add=add.cuda())
    _near(got, x.double() + add.double(), 1e-6)
    _near(out, R.layer_norm(got.cpu().double(), w.double(), 1e-5), max(tol, 1e-5))


@pytest.mark.parametrize("E,top,V,T,L", [(8, 1, 50, 200, 3), (5, 3, 11, 1, 1), (16, 2, 300, 700, 2), (1, 1, 7, 33, 1), (70, 4, 90, 64, 2)])
def test_expert_orders_from_tables(E, top, V, T, L):
    from mi355_decode import ops
    g = torch.Generator().manual_seed(E + T)
    tables = torch.stack([torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(V)]) for _ in range(L)]).to(torch.int32)
    ids = torch.randint(0, V, (T,), generator=g)
    r = ops.TableRoutes(tables.cuda(), ids.cuda(), E)
    assert r.rows == T * top
    for layer in range(L):
        want = tables[layer][ids].reshape(-1)
        counts = torch.bincount(want, minlength=E)
        assert r.offsets[layer].tolist() == [0] + counts.cumsum(0).tolist()
        assert r.tile_start[layer].tolist() == [0] + (-(-counts // ops.MOE_TILE_ROWS)).cumsum(0).tolist()
        perm, inv = r.perm[layer].cpu().long(), r.inv[layer].cpu().long()
        assert sorted(perm.tolist()) == list(range(T * top)) and torch.equal(inv[perm], torch.arange(T * top))
        assert torch.equal(want[perm], torch.repeat_interleave(torch.arange(E), counts).to(torch.int32))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
@pytest.mark.parametrize("E,top,T,W,F", [(4, 1, 600, 64, 96), (6, 2, 37, 96, 64), (5, 3, 300, 72, 40), (3, 2, 9, 90, 30), (9, 2, 1, 32, 16),
                                         (2, 1, 500, 136, 200)])
def test_table_mixture_of_ungated_experts(dtype, E, top, T, W, F):
    """Through the runner's feed-forward object: few rows per expert take the row kernels, many the tiles; one expert is
    left without rows; what is added to the residual against the restatement."""
    from mi355_decode import hybrid_runner as H
    from mi355_decode import ops
    from mi355_decode.config import MoESpec
    g = torch.Generator().manual_seed(T + E)
    V = 40
    names = torch.arange(1, E) if E > top else torch.arange(E)                                # expert 0 is never chosen
    table = torch.stack([names[torch.randperm(len(names), generator=g)[:top]] for _ in range(V)]).to(torch.int32)
    wt = {"table": table}
    for e in range(E):
        wt[f"e{e}.up"], wt[f"e{e}.down"] = torch.randn(F, W, generator=g) * W ** -0.5, torch.randn(W, F, generator=g) * F ** -0.5
    wt = {k: v if k == "table" else b16(v).float() for k, v in wt.items()}
    h, ids, x = torch.randn(T, W, generator=g).to(dtype), torch.randint(0, V, (T,), generator=g), torch.randn(T, W, generator=g)
    want = x + R.table_moe_ff(wt, "", {"router": {"top": top}}, h.float(), ids.tolist())
    lw = SimpleNamespace(up_w=torch.stack([wt[f"e{e}.up"] for e in range(E)]).to(dtype).cuda(),
                         down_w=torch.stack([wt[f"e{e}.down"] for e in range(E)]).to(dtype).cuda())
    spec = MoESpec(E, top, 1, 1, F, score="table", gated=False)
    ff = H.TableMoE(spec, lw, 1)
    b = SimpleNamespace(routes={(E, top): ops.TableRoutes(torch.stack([table.flip(0), table]).cuda(), ids.cuda(), E)})
    keep = H.EXPERT_GEMM_MIN_ROWS
    try:
        for least in (0, 1 << 20):
            H.EXPERT_GEMM_MIN_ROWS = least
            y = ff(h.cuda(), b)
            got = x.cuda()
            ops.add_layer_norm_f32(got, None, 1e-5, add=y.rows, inv=y.inv, top=y.top, row_weight=y.weight)
            _near(got, want, 2e-6 if dtype == torch.float32 else 2e-2)
    finally:
        H.EXPERT_GEMM_MIN_ROWS = keep


@pytest.mark.parametrize("dtype,tol", [(torch.bfloat16, 1e-2), (torch.float16, 2e-3)])
@pytest.mark.parametrize("rows", [1, 15, 33, 64, 65, 200])
@pytest.mark.parametrize("H,N,K", [(3, 64, 32), (2, 200, 136), (5, 12, 8), (1, 132, 512)])
def test_products_per_head(dtype, tol, rows, H, N, K):
    """Column slices in and out, rows through an index, pages of 16 rows with copied columns, transposed pages; nothing
    beside the outputs is touched."""
    from mi355_decode import ops
    g = torch.Generator().manual_seed(rows + N)
    w = (torch.randn(H, N, K, generator=g) * K ** -0.5).to(dtype)
    x = torch.randn(rows, H * K + 8, generator=g).to(dtype)
    want = torch.einsum("mhk,hnk->mhn", x[:, 8:].double().view(rows, H, K), w.double())
    buf = x.cuda()
    out = torch.full((rows, H * N + 8), 7.0, dtype=dtype, device="cuda")
    ops.head_gemm(buf[:, 8:], K, w.cuda(), out, 16 * (H * N + 8), H * N + 8, N, rows)
    _near(out[:, : H * N], want.reshape(rows, -1), tol)
    assert (out[:, H * N:] == 7.0).all()
    # one row for all heads, read through an index; N + copied columns per head, pages of 16 rows
    C = 24
    src = torch.randn(77, K + C, generator=g).to(dtype)
    index = torch.randint(0, 77, (rows,), generator=g).to(torch.int32)
    want = torch.einsum("mk,hnk->mhn", src[index.long(), :K].double(), w.double())
    pages = -(-rows // 16)
    if N % 8 == 0:
        out = torch.full((pages, H, 16, N + C), 7.0, dtype=dtype, device="cuda")
        ops.head_gemm(src.cuda(), 0, w.cuda(), out, H * 16 * (N + C), N + C, 16 * (N + C), rows, index=index.cuda(), copy=C)
        got = out.permute(0, 2, 1, 3).reshape(pages * 16, H, N + C).cpu()
        _near(got[:rows, :, :N], want, tol)
        assert torch.equal(got[:rows, :, N:], src[index.long(), K:][:, None].expand(rows, H, C)) and (got[rows:] == 7.0).all()
    out = torch.full((pages, H, N, 16), 7.0, dtype=dtype, device="cuda")
    ops.head_gemm(src.cuda(), 0, w.cuda(), out, H * N * 16, 0, N * 16, rows, index=index.cuda(), transposed=True)
    got = out.permute(0, 3, 1, 2).reshape(pages * 16, H, N).cpu()
    _near(got[:rows], want, tol)
    assert (got[rows:] == 7.0).all()


# ------------------------------------------------------------------------------------------ #
# mechanisms alone: the attention with row norms, temperature, cap and sinks
# ------------------------------------------------------------------------------------------ #
def _pages(T, G, d, dv, dtype, spare=3, seed=0):
    """A shuffled page table for one sequence of T tokens over NaN-filled pools."""
    n = -(-T // 16)
    order = torch.randperm(n + spare, generator=torch.Generator().manual_seed(seed))[:n]
    kc = torch.full((n + spare, G, 16, d), float("nan"), dtype=dtype, device="cuda")
    vc = torch.full((n + spare, G, dv, 16), float("nan"), dtype=dtype, device="cuda")
    slots = (order[torch.arange(T) // 16] * 16 + torch.arange(T) % 16).cuda()
    return kc, vc, order.to(torch.int32).view(1, n).cuda(), slots


def _attend_in_cuts(q, k, v, wq, wk, cuts, scale, cap=0.0, sink=None, temp=(0.0, 0.0), form="rows", splits=0):
    """q [T, H, d], k [T, G, d], v [T, G, dv] as projected: norms, temperature, page write and attention through the
    product's kernels, portion by portion, over shuffled NaN-filled pages."""
    from mi355_decode import ops
    T, H, d = q.shape
    G, dv, dt = k.shape[1], v.shape[2], q.dtype
    kc, vc, bt, slots = _pages(T, G, d, dv, dt)
    none = torch.empty(T + 16, 0, device="cuda")
    outs, at = [], 0
    cuts = list(cuts) + ([T - sum(cuts)] if sum(cuts) < T else [])
    sk = None if sink is None else sink.cuda()
    for n in cuts:
        pos = torch.arange(at, at + n, dtype=torch.int64, device="cuda")
        width = (H + G) * d + G * dv
        buf = torch.cat([q[at:at + n].reshape(n, -1), k[at:at + n].reshape(n, -1), v[at:at + n].reshape(n, -1),
                         torch.zeros(n, -width % 8, dtype=dt)], dim=1).cuda().contiguous()
        qs, ks, vs = buf[:, : H * d], buf[:, H * d: (H + G) * d], buf[:, (H + G) * d: width]
        ops.row_norm_rope_kv_write(qs, ks, vs, wq.cuda(), wk.cuda(), none, pos, slots[at:at + n], kc, vc, H, G, d, dv, 1e-5,
                                   temp_coef=temp[0], temp_every=temp[1])
        if form == "staged" and n == 1 and ops.attn_decode_ok(dt, H, G, d, dv):
            o = ops.paged_attn_decode(qs, kc, vc, bt, torch.tensor([at + 1], dtype=torch.int32, device="cuda"), H, G, d, scale,
                                      num_splits=max(splits, 1), sink=sk, softcap=cap)
        elif form == "staged":
            assert ops.chunk_attn_prefill_ok(dt, H, G, d, dv)
            o = ops.paged_attn_prefill_ext(qs, kc, vc, bt, torch.tensor([0, n], dtype=torch.int32, device="cuda"),
                                           torch.tensor([at + n], dtype=torch.int32, device="cuda"), n, H, G, d, scale, sink=sk, softcap=cap)
        else:
            tiles = torch.from_numpy(ops.query_tiles(np.array([0, n]))).cuda() if form == "tiles" else None
            o = ops.softmax_bias_attn(qs, kc, vc, bt, torch.zeros(n, dtype=torch.int32, device="cuda"), pos, None, None, None, H, scale,
                                      tiles=tiles, num_splits=splits, sink=sk, softcap=cap)
        outs.append(o.float().cpu())
        at += n
    return torch.cat(outs)


def _attend_ref(q, k, v, wq, wk, scale, cap=0.0, sink=None, temp=(0.0, 0.0)):
    T, H, d = q.shape
    q = R.rms_norm(q.double().reshape(T, -1), wq.double(), 1e-5)
    k = R.rms_norm(k.double().reshape(T, -1), wk.double(), 1e-5)
    q = q * R.query_temperature(T, {"coef": temp[0], "every": temp[1]} if temp[1] else None, torch.float64)[:, None]
    return R.attention(q.view(T, H, d), k.view(T, -1, d), v.double(), scale, cap, None if sink is None else sink.double())


CUTS = ([1] * 90, [2, 3, 1, 30, 2, 16, 21], [90])


def _qkv(H, G, d, dv, T=90):
    g = torch.Generator().manual_seed(H * 100 + d)
    return (torch.randn(T, H, d, generator=g), torch.randn(T, G, d, generator=g), torch.randn(T, G, dv, generator=g),
            torch.randn(H * d, generator=g) * 0.3 + 1.5, torch.randn(G * d, generator=g) * 0.3 + 1.5, torch.randn(H, generator=g) * 2)


@pytest.mark.parametrize("every,coef", [(7, 0.5), (1, 2.0), (2.5, -0.3), (45, 1.0), (1000, 3.0)])
def test_query_temperature_steps(every, coef):
    """Equal queries at all positions: the stored ones show the factor, which steps where position + 1 passes a multiple."""
    from mi355_decode import ops
    T, H, d = 100, 2, 8
    q, k, v = torch.ones(T, H * d), torch.ones(T, d), torch.ones(T, d)
    kc, vc, _, slots = _pages(T, 1, d, d, torch.float32)
    qs = q.cuda()
    ops.row_norm_rope_kv_write(qs, k.cuda(), v.cuda(), torch.ones(H * d).cuda(), torch.ones(d).cuda(), torch.empty(T, 0).cuda(),
                               torch.arange(T).cuda(), slots, kc, vc, H, 1, d, d, 0.0, temp_coef=coef, temp_every=every)
    want = R.query_temperature(T, {"coef": coef, "every": every})
    _near(qs, want[:, None].expand(T, H * d), 1e-6)
    assert (want[1:] != want[:-1]).nonzero().view(-1).tolist() == [p - 1 for p in range(1, T) if (p + 1) // every != p // every]
    flat = kc[torch.div(slots, 16, rounding_mode="floor"), 0, slots % 16]
    _near(flat, torch.ones(T, d), 1e-6)                       # keys keep their size


@pytest.mark.parametrize("H,G,d,dv,cap,temp", [(6, 2, 16, 24, 2.0, (0.7, 7)), (3, 3, 24, 8, 0.0, (0.5, 16)), (5, 5, 21, 7, 0.5, (0.0, 0.0)),
                                               (4, 1, 8, 12, 30.0, (1.0, 1)), (1, 1, 136, 40, 5.0, (0.3, 33)), (2, 2, 8, 300, 3.0, (0.0, 0.0))])
def test_capped_attention_by_rows(H, G, d, dv, cap, temp):
    q, k, v, wq, wk, sink = _qkv(H, G, d, dv)
    kw = dict(cap=cap, sink=sink, temp=temp)
    ref = _attend_ref(q, k, v, wq, wk, 0.4, **kw)
    assert (ref - _attend_ref(q, k, v, wq, wk, 0.4, cap=cap, temp=temp)).abs().max() > 0.05 * ref.abs().max()      # the sinks are heard
    for cuts in CUTS:
        _near(_attend_in_cuts(q, k, v, wq, wk, cuts, 0.4, **kw), ref, 3e-5)
    q, k, v = b16(q), b16(k), b16(v)
    _near(_attend_in_cuts(q, k, v, wq, wk, [40, 2, 1, 47], 0.4, **kw), _attend_ref(q, k, v, wq, wk, 0.4, **kw), 4e-2)


@pytest.mark.parametrize("H,G,d,dv,cap", [(6, 2, 32, 16, 2.0), (3, 3, 64, 48, 8.0), (8, 2, 48, 32, 30.0), (4, 4, 96, 16, 1.0), (8, 1, 8, 64, 4.0),
                                          (2, 1, 128, 128, 3.0), (3, 1, 40, 80, 0.0), (1, 1, 104, 112, 6.0)])
@pytest.mark.parametrize("splits", [0, 3])
def test_capped_attention_on_the_matrix_cores(H, G, d, dv, cap, splits):
    """Key sizes that do and do not fill the last fragment, in the tile form with and without key splits."""
    q, k, v, wq, wk, sink = _qkv(H, G, d, dv)
    q, k, v = b16(q), b16(k), b16(v)
    kw = dict(cap=cap, sink=sink, temp=(0.4, 20))
    ref = _attend_ref(q, k, v, wq, wk, 0.3, **kw)
    for cuts in CUTS:
        _near(_attend_in_cuts(q, k, v, wq, wk, cuts, 0.3, form="tiles", splits=splits, **kw), ref, 4e-2)


@pytest.mark.parametrize("H,G,d,dv,cap", [(8, 2, 64, 64, 2.0), (3, 3, 128, 64, 20.0), (4, 1, 64, 128, 5.0), (16, 1, 128, 128, 1.0), (2, 2, 192, 128, 4.0),
                                          (3, 3, 192, 64, 0.0)])
def test_capped_attention_staged_through_lds(H, G, d, dv, cap):
    q, k, v, wq, wk, sink = _qkv(H, G, d, dv)
    q, k, v = b16(q), b16(k), b16(v)
    kw = dict(cap=cap, sink=sink, temp=(0.4, 20))
    ref = _attend_ref(q, k, v, wq, wk, 0.3, **kw)
    for cuts, splits in (([2, 3, 1, 30, 2, 16, 36], 0), ([90], 0), ([1] * 90, 0), ([50] + [1] * 40, 3)):      # (single tokens: the decode launch)
        _near(_attend_in_cuts(q, k, v, wq, wk, cuts, 0.3, form="staged", splits=splits, **kw), ref, 4e-2)
    _near(_attend_in_cuts(q, k, v, wq, wk, [90], 0.3, form="staged", cap=cap), _attend_ref(q, k, v, wq, wk, 0.3, cap=cap), 4e-2)


@pytest.mark.parametrize("form", ["rows", "tiles", "staged"])
@pytest.mark.parametrize("at", [0, 15, 16, 130, 255])
def test_a_far_key_among_hundreds(form, at):
    """One key is matched by the query hundreds of tokens later (its capped score stands far above the others'), in a
    prompt, in a portion and decoded; without the cap the others' share would vanish, with it they keep a visible one."""
    T, H, G, d = 300, 4, 2, 64
    g = torch.Generator().manual_seed(3)
    q, k, v = torch.randn(T, H, d, generator=g) * 0.1, torch.randn(T, G, d, generator=g) * 0.1, torch.randn(T, G, d, generator=g)
    q[:, :, 0] += 1.0
    k[:, :, 1] += 1.0
    k[at, :, 0], k[at, :, 1] = 1.0, 0.0
    v[at] = 5.0
    wq, wk, sink = torch.ones(H * d), torch.ones(G * d), torch.tensor([0.0, 3.0, -5.0, 8.0])
    if form != "rows":
        q, k, v = b16(q), b16(k), b16(v)
    kw = dict(cap=8.0, sink=sink, temp=(0.2, 100))
    ref = _attend_ref(q, k, v, wq, wk, 0.25, **kw)
    assert 1.5 < ref[-1, 0] < 4.9 and ref[-1, d] < 4.9 and ref[-1, 3 * d] < 0.75 * ref[-1, 0]
    for cuts in ([T], [200, 2, 97, 1], [290] + [1] * 10):
        got = _attend_in_cuts(q, k, v, wq, wk, cuts, 0.25, form=form, **kw)
        _near(got, ref, 3e-5 if form == "rows" else 2e-2)


# ------------------------------------------------------------------------------------------ #
# mechanisms alone: the latent attention
# ------------------------------------------------------------------------------------------ #
def _latent_case(H, d, r, dv, rank, base, T, seed=0, W=48):
    cfg = {"heads": H, "dim": d, "rot_dim": r, "vdim": dv, "kv_rank": rank, "scale": 0.3, "rot": {"dims": r, "base": base}}
    full = _cfg(W, 9, [({"type": "latent_attention", "mixer": cfg}, None)])
    st = R.random_state(full, seed=seed)
    h = torch.randn(T, W, generator=torch.Generator().manual_seed(seed + 1))
    return full, st, b16(h).float()


def _latent_in_cuts(full, st, h, dtype, cuts, min_rows=None):
    """The product's latent attention of one layer, portion by portion, on shuffled NaN-filled pages."""
    from mi355_decode import hybrid_runner as HR
    from mi355_decode import ops, weights
    from mi355_decode.config import ModelConfig
    cfg = ModelConfig.from_dict(full)
    lw, A = weights.from_state_dict(cfg, st, dtype, "cuda").layers[0], cfg.hybrid.layers[0].lattn
    T = h.shape[0]
    n, spare = -(-T // 16), 3
    order = torch.randperm(n + spare, generator=torch.Generator().manual_seed(5))[:n]
    nan = float("nan")
    cache = torch.full((n + spare, 16, A.kv_rank + A.rot_dim), nan, dtype=dtype, device="cuda")
    cache_t = torch.full((n + spare, A.kv_rank, 16), nan, dtype=dtype, device="cuda") if ops.latent_tiles_ok(dtype, A.kv_rank, A.rot_dim) else None
    table = HR.rotary_table(A.rot_dims, A.rot_base, T + 16, "cuda", exact=True)
    r = SimpleNamespace(latent_cache=[(cache, cache_t)], rotary=lambda *a, **k: table, eps=cfg.rms_norm_eps, dtype=dtype,
                        linear=lambda x, w: torch.mm(x, w.t()))
    mixer = HR.LatentAttention(A, lw, r, 0, True)
    bt = order.to(torch.int32).view(1, n).cuda()
    slots = (order[torch.arange(T) // 16] * 16 + torch.arange(T) % 16).cuda()
    outs, at, expanded = [], 0, 0
    cuts = list(cuts) + ([T - sum(cuts)] if sum(cuts) < T else [])
    keep = HR.LatentPlan.EXPAND_MIN_ROWS
    try:
        if min_rows is not None:
            HR.LatentPlan.EXPAND_MIN_ROWS = min_rows
        for c in cuts:
            cu = np.array([0, c])
            plan = HR.LatentPlan(cu, [at + c], bt.cpu().numpy(), "cuda")
            expanded += int(mixer.expands and plan.fits and c > 1)
            b = HR.StepBatch(torch.zeros(c, dtype=torch.int64, device="cuda"), torch.arange(at, at + c, device="cuda"), slots[at:at + c], bt,
                             torch.tensor([0, c], dtype=torch.int32, device="cuda"), torch.zeros(c, dtype=torch.int32, device="cuda"), None,
                             long_chunks=c > 1, pair_tiles=lambda heads: torch.from_numpy(ops.pair_tiles(cu, heads)).cuda(),
                             latent_plan=lambda: plan)
            x = h[at:at + c].to(dtype).cuda()
            outs.append(mixer(torch.mm(x, lw.in_w.t()), b).float().cpu())
            at += c
    finally:
        HR.LatentPlan.EXPAND_MIN_ROWS = keep
    return torch.cat(outs), expanded


def _latent_ref(full, st, h):
    m = full["layers"][0]["mixer"]
    return R.latent_attention_mixer({k: v.double() for k, v in st.items()}, "l0.mix.", m, h.double(), full["norm"]["eps"])


@pytest.mark.parametrize("H,d,r,dv,rank,base", [(3, 16, 8, 24, 32, 500.0), (1, 8, 2, 8, 8, 50.0), (7, 13, 6, 9, 22, 77.0), (5, 24, 4, 8, 300, 1e4),
                                                (2, 40, 48, 20, 16, 1e4)])
def test_latent_attention_in_float32(H, d, r, dv, rank, base):
    full, st, h = _latent_case(H, d, r, dv, rank, base, 90)
    want = _latent_ref(full, st, h)
    for cuts in CUTS:
        _near(_latent_in_cuts(full, st, h, torch.float32, cuts)[0], want, 3e-5)


@pytest.mark.parametrize("H,d,r,dv,rank,base", [(3, 16, 8, 24, 32, 500.0), (8, 64, 16, 48, 64, 1e4), (5, 24, 8, 40, 272, 1e4), (7, 13, 6, 9, 22, 77.0),
                                                (17, 32, 32, 16, 112, 1e5), (3, 20, 4, 12, 48, 100.0), (17, 64, 64, 64, 512, 1e4), (5, 24, 8, 40, 192, 1e4),
                                                (2, 16, 8, 24, 128, 1e3), (33, 16, 64, 8, 256, 1e4), (3, 16, 128, 16, 512, 1e4)])
def test_latent_attention_on_the_latents_in_bfloat16(H, d, r, dv, rank, base):
    full, st, h = _latent_case(H, d, r, dv, rank, base, 90)
    want = _latent_ref(full, st, h)
    for cuts in CUTS:
        got, expanded = _latent_in_cuts(full, st, h, torch.bfloat16, cuts, min_rows=1 << 30)
        _near(got, want, 4e-2)
        assert expanded == 0


@pytest.mark.parametrize("H,d,r,dv,rank,base", [(4, 96, 32, 64, 128, 1e4), (3, 128, 64, 128, 256, 1e6), (1, 48, 16, 128, 40, 50.0), (2, 56, 8, 64, 72, 1e4),
                                                (5, 64, 128, 64, 512, 1e3)])
def test_latent_attention_with_expanded_keys_and_values(H, d, r, dv, rank, base):
    full, st, h = _latent_case(H, d, r, dv, rank, base, 150)
    want = _latent_ref(full, st, h)
    for cuts, least, n in (([150], 2, 1), ([2, 3, 1, 30, 2, 16, 96], 2, 6), ([49, 1, 1, 50, 2, 47], 20, 3), ([150], 48, 1), ([100, 40, 10], 48, 1)):
        got, expanded = _latent_in_cuts(full, st, h, torch.bfloat16, cuts, min_rows=least)
        assert expanded == n
        _near(got, want, 4e-2)


@pytest.mark.parametrize("dtype,least", [(torch.float32, None), (torch.bfloat16, 1 << 30), (torch.bfloat16, 2)])
@pytest.mark.parametrize("at", [0, 15, 16, 200])
def test_a_far_latent_among_hundreds(dtype, least, at):
    """One token's latent is matched by every later query; its value is loud.  The last queries, in prompts and decoded,
    hear it across hundreds of keys and many pages."""
    full, st, _ = _latent_case(4, 96, 32, 64, 128, 1e4, 1)
    T, W = 270, 48
    g = torch.Generator().manual_seed(1)
    h = torch.randn(T, W, generator=g) * 0.3
    h[:, 0], h[:, 1], h[:, 2] = 0.0, 1.0, 1.0
    h[at, 0], h[at, 1] = 1.0, 0.0
    h = b16(h).float()
    for n in ("q", "dkv", "uk", "uv"):
        st["l0.mix." + n] = st["l0.mix." + n] * 0.1
    st["l0.mix.dkv"][0, 0], st["l0.mix.dkv"][1, 1] = 8.0, 8.0     # latent 0 marks the one token, latent 1 the others
    st["l0.mix.q"].view(4, 128, W)[:, 0, 2] = 4.0                 # every query asks along unrotated coordinate 0
    st["l0.mix.uk"].view(4, 96, 128)[:, 0, 0] = 1.0               # which the marked latent lights
    st["l0.mix.uv"].view(4, 64, 128)[:, :, 0] = 1.0
    st = {k: b16(v).float() for k, v in st.items()}
    want = _latent_ref(full, st, h)
    quiet = h.clone()
    quiet[at] = h[at + 1]
    assert (want - _latent_ref(full, st, quiet))[-1].abs().max() > 0.5 * want[-1].abs().max()
    for cuts in ([T], [200, 2, 67, 1], [260] + [1] * 10):
        _near(_latent_in_cuts(full, st, h, dtype, cuts, min_rows=least)[0], want, 3e-5 if dtype == torch.float32 else 3e-2)


def test_rotation_of_neighbours():
    """Alone, in place and into the pages: coordinates 2i, 2i + 1 turn together; the half-split pairing is another result."""
    from mi355_decode import ops
    from mi355_decode.hybrid_runner import rotary_table
    T, H, hw, off, rot = 40, 3, 26, 10, 12
    g = torch.Generator().manual_seed(0)
    q = torch.randn(T, H * hw, generator=g)
    table = rotary_table(rot, 300.0, T, "cuda", exact=True)
    want = q.view(T, H, hw).clone()
    want[:, :, off: off + rot] = R.rotate_neighbours(want[:, :, off: off + rot], {"dims": rot, "base": 300.0})
    a, b = q.cuda(), q.cuda()
    ops.latent_q_rotate(a, H, hw, off, table, torch.arange(T).cuda(), interleaved=True)
    ops.latent_q_rotate(b, H, hw, off, table, torch.arange(T).cuda())
    _near(a.view(T, H, hw), want, 1e-6)
    assert not torch.allclose(a, b)
    qe = torch.full((T, H, 20 + rot), 7.0, device="cuda")
    ops.latent_q_pack(None, q.cuda(), hw, off, rot, table, torch.arange(T).cuda(), interleaved=True, out=qe)
    _near(qe[:, :, 20:], want[:, :, off: off + rot], 1e-6)
    assert (qe[:, :, :20] == 7.0).all()
    x = torch.randn(T, 20 + rot, generator=g)
    cache = torch.zeros(3, 16, 20 + rot, device="cuda")
    ops.latent_kv_write(x.cuda(), torch.ones(20, device="cuda"), table, torch.arange(T).cuda(), torch.arange(T).cuda(), cache, 20, rot, 1e-5,
                        interleaved=True)
    flat = cache.view(48, -1)[:T]
    _near(flat[:, 20:], R.rotate_neighbours(x[:, 20:], {"dims": rot, "base": 300.0}), 1e-6)
    _near(flat[:, :20], R.rms_norm(x[:, :20], torch.ones(20), 1e-5), 1e-6)


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
        R.forward(_weights(name), CONFIGS[name], toks, want)
    assert len(trace) == len(want)
    for i, (a, b) in enumerate(zip(trace, want)):
        assert np.abs(a - b.numpy()).max() <= 1e-4 * np.abs(b.numpy()).max(), f"layer run {i}"
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
    lens = {"a": 60, "b": 23, "c": 131, "d": 2, "e": 47, "f": 85}
    toks = {r: _tokens(name, n, ord(r)) for r, n in lens.items()}
    plan = {"a": [30, 1, 1, 2, 26], "b": [2, 1, 20], "c": [16, 57, 1, 1, 1, 55], "d": [1, 1], "e": [2, 45], "f": [64, 2, 19]}
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


@pytest.mark.parametrize("name", ["wide", "mix"])
def test_mixed_batches_in_bfloat16(name):
    """At the wide sizes steps hold chunks whose context is expanded beside single tokens that stay on the latents."""
    eng = _engine(name, dtype="bfloat16", pages=24)
    for toks, got in _run_mixed(eng, name).values():
        _tracks(got, _ref(name, toks), _ref(name, toks).std())


def test_pages_and_slots_are_reused_without_leaking():
    for name in ("plain", "mix"):
        eng = _engine(name, pages=8, max_model_len=128)         # one 100-token request nearly fills the pool
        for i in range(6):
            toks = _tokens(name, 100 - 7 * i, 50 + i)
            _close(_run_cuts(eng, f"r{i}", toks, [40, 3] + [1] * 10), _ref(name, toks))


@pytest.mark.parametrize("name", ["mix", "odd"])
def test_long_decoding_across_pages_and_temperature_steps(name):
    eng = _engine(name)
    toks = _tokens(name, 300, 9)
    _close(_run_cuts(eng, "long", toks, [10] + [1] * 290), _ref(name, toks), tol=6e-4)


@pytest.mark.parametrize("name", ["mix", "wide", "odd"])
def test_bfloat16_tracks_the_float32_restatement(name):
    """Whole prompts (library GEMMs, the staged attentions, expert tiles) and decode-sized steps (at width 512 the
    tiled weight stream) in bfloat16 against the restatement and against each other."""
    eng = _engine(name, dtype="bfloat16")
    if name == "wide":
        assert eng.runner._tiled_w, "no tiled weight copies at width 512"
    toks = _tokens(name, 140, 4)
    want = _ref(name, toks)
    whole = _run_cuts(eng, "h", toks, [140])
    for got in (whole, _run_cuts(eng, "h", toks, [60, 2] + [1] * 20 + [50, 2, 6])):
        for a, b in ((got, want), (got, whole)):
            _tracks(a, b, want.std())


@pytest.mark.parametrize("name,dtype", [("mix", "float32"), ("plain", "float32"), ("wide", "bfloat16")])
def test_greedy_generation_through_the_engine(name, dtype):
    """LLM.generate: scheduler admission, prefill, then decode steps replayed from HIP graphs with
    run-ahead.  A token may leave the restatement's only where its own margin is inside the error."""
    from mi355_decode.llm import LLM
    from mi355_decode.sampling_params import SamplingParams
    eng = _engine(name, dtype=dtype)
    prompts = [_tokens(name, n, 70 + n) for n in (5, 73, 18, 1, 26)]     # five requests on four slots: one waits
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


def _save_model(model_dir, cfg, w):
    import json
    from safetensors.torch import save_file
    model_dir.mkdir()
    json.dump(cfg, open(model_dir / "config.json", "w"))
    save_file({k: (v if v.dtype == torch.int32 else v.to(torch.bfloat16)).contiguous() for k, v in w.items()}, str(model_dir / "model.safetensors"))


def test_served_from_a_model_directory(tmp_path):
    """The OpenAI server started on a directory with config.json + model.safetensors of this design: the
    model class chosen by config.json, weights from the checkpoint names, greedy completions by token
    id against the restatement (margin rule), and a seeded sampled completion through the sampler."""
    import os
    import signal
    import socket
    import subprocess
    import sys
    import time
    from conftest import PKG, ROOT
    from mi355_decode.harness import BenchClient
    name = "mix"
    cfg, w = CONFIGS[name], _weights(name)
    model_dir = tmp_path / "model"
    _save_model(model_dir, cfg, w)
    with socket.socket() as s:
        s.bind(("127.0.0.1", 0))
        port = s.getsockname()[1]
    args = ["--model", str(model_dir), "--served-model-name", "tables", "--host", "127.0.0.1", "--port", str(port),
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
            assert time.time() - t0 < 100, "server did not become healthy"
            time.sleep(0.2)
        post = lambda **body: client.http.post(f"{url}/v1/completions", json={"model": "tables", **body})   # noqa: E731
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
    from conftest import ROOT
    name = "plain"
    cfg, w = CONFIGS[name], _weights(name)
    model_dir, out_dir = tmp_path / "model", tmp_path / "out"
    _save_model(model_dir, cfg, w)
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
