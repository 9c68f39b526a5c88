"""Plain, slow restatement of the Rigazen decoder in float32 (or float64) torch on the CPU, one
function per mechanism.  TEST INFRASTRUCTURE (see oracle/__init__.py): nothing here is imported by
the product and nothing of the product is imported here.

Notation.  W: model width; rms(x) = x / sqrt(mean(x^2) + eps); act(z) = gelu with the tanh formula.

    x     = embed[tok] * embedding.scale
    layer:  x += rms(mixer(x)) (1 + norm1);  x += rms(ff(x)) (1 + norm2)         (norms on the outputs only)
            e = side.embed[tok, i D : (i + 1) D];  x += rms(P (act(G x) e)) * side.norm        (D = token_side.dim)
    logits = embed (rms(x) (1 + final.norm))                                     (no scale on the tied table)

Mixer "mlstm", H heads of `dim` (queries, keys) and `vdim` (values): q = Q x / sqrt(dim), k = K x,
v = V x; per head a = cap tanh((I x + bi) / cap), b = log sigmoid(cap tanh((F x + bf) / cap)).  From
C = 0, n = 0, m = 0, token by token:
    m' = max(b + m, a);  r = exp(b + m - m'), w = exp(a - m');  C <- r C + w k v^T;  n <- r n + w k;  m <- m'
    o = C^T q / (max(|n . q|, exp(-m)) + 1e-6)
rms per head, all heads side by side times norm times sigmoid(G x), then O.

Mixer "parallel": left_scale * L(x) + right_scale * R(x).
  L: grouped-query softmax attention with biased q, k, v; rms of the whole query row and of the whole
     key row (all heads at once) times a weight each, then rotation of the first R = rot.dims
     coordinates of every head (pairs i, i + R/2; angle p base^(-2i/R)); score q . k * scale; position i
     sees j <= i with i - j < mask.size or j < mask.keep_first.
  R: q = silu(Q x), k = silu(K x), v = silu(V x); per head S <- decay S + k v^T, o = S^T q; rms over all
     heads at once times norm times sigmoid(G x), then O.

Feed-forward: D relu(U x)^2, or none.
"""
from __future__ import annotations

import math

import torch
import torch.nn.functional as F


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def lin(wt, name, x):
    return x @ wt[name].to(x.dtype).T


def embed_tokens(wt, cfg, tokens, dtype=torch.float32):
    tok = torch.as_tensor(tokens, dtype=torch.int64)
    return wt["embed"][tok].to(dtype) * float((cfg.get("embedding") or {}).get("scale", 1.0))


# ---- the matrix memory with exponential gates
def mlstm_gates(zi, zf, cap):
    """zi, zf: the projections plus biases.  Returns (log input gate, log forget gate)."""
    return cap * torch.tanh(zi / cap), F.logsigmoid(cap * torch.tanh(zf / cap))


def mlstm_memory(q, k, v, a, b, state=None):
    """q, k [T, H, d] (q scaled already), v [T, H, dv], a, b [T, H]: log input / forget gates.  Token by
    token from `state` = (C [H, d, dv], n [H, d], m [H]) or zeros.  Returns (o [T, H, dv], state)."""
    T, H, d = q.shape
    dv = v.shape[2]
    C, n, m = state if state is not None else (q.new_zeros(H, d, dv), q.new_zeros(H, d), q.new_zeros(H))
    out = []
    for t in range(T):
        m2 = torch.maximum(b[t] + m, a[t])
        r, w = torch.exp(b[t] + m - m2), torch.exp(a[t] - m2)
        C = r[:, None, None] * C + w[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = r[:, None] * n + w[:, None] * k[t]
        m = m2
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out.append(torch.einsum("hdv,hd->hv", C, q[t]) / den[:, None])
    return torch.stack(out), (C, n, m)


def head_norm_gate(o, w, gate, eps):
    """o [T, H, dv] -> rms per head, heads side by side, times w [H dv] times sigmoid(gate)."""
    return rms(o, eps).reshape(o.shape[0], -1) * w * torch.sigmoid(gate)


def mlstm(wt, pre, m, x, eps):
    T, H, d, dv, cap = x.shape[0], int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["gate_cap"])
    q = lin(wt, pre + "q", x).view(T, H, d) * d ** -0.5
    k, v = lin(wt, pre + "k", x).view(T, H, d), lin(wt, pre + "v", x).view(T, H, dv)
    a, b = mlstm_gates(lin(wt, pre + "i", x) + wt[pre + "i.b"].to(x.dtype), lin(wt, pre + "f", x) + wt[pre + "f.b"].to(x.dtype), cap)
    o, _ = mlstm_memory(q, k, v, a, b)
    return lin(wt, pre + "o", head_norm_gate(o, wt[pre + "norm"].to(x.dtype), lin(wt, pre + "g", x), eps))


# ---- linear attention with a constant decay per head
def decayed_memory(q, k, v, decay, state=None):
    """q, k [T, H, d], v [T, H, dv], decay [H]: S <- decay S + k v^T, o = S^T q.  Returns (o, S)."""
    S = state if state is not None else q.new_zeros(q.shape[1], q.shape[2], v.shape[2])
    dec = torch.as_tensor(decay, dtype=torch.float64).to(q.dtype)
    out = []
    for t in range(q.shape[0]):
        S = dec[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out), S


def all_norm_gate(o, w, gate, eps):
    """o [T, H, dv] -> rms over all heads at once, times w times sigmoid(gate)."""
    return rms(o.reshape(o.shape[0], -1), eps) * w * torch.sigmoid(gate)


def lightning(wt, pre, m, x, eps):
    T, H, d, dv = x.shape[0], int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k = F.silu(lin(wt, pre + "q", x)).view(T, H, d), F.silu(lin(wt, pre + "k", x)).view(T, H, d)
    o, _ = decayed_memory(q, k, F.silu(lin(wt, pre + "v", x)).view(T, H, dv), m["decay"])
    return lin(wt, pre + "o", all_norm_gate(o, wt[pre + "norm"].to(x.dtype), lin(wt, pre + "g", x), eps))


# ---- windowed attention with kept first tokens
def rotate(x, rot, first=0):
    """x [T, heads, dim] at positions first, first + 1, ..."""
    R = int((rot or {}).get("dims", 0))
    if R == 0:
        return x
    f = float(rot["base"]) ** (-2.0 * torch.arange(R // 2, dtype=torch.float64) / R)
    ang = torch.arange(first, first + x.shape[0], dtype=torch.float64)[:, None] * f[None, :]
    c, s = torch.cos(ang)[:, None, :].to(x.dtype), torch.sin(ang)[:, None, :].to(x.dtype)
    a, b, rest = x[..., : R // 2], x[..., R // 2: R], x[..., R:]
    return torch.cat([a * c - b * s, b * c + a * s, rest], dim=-1)


def window_mask(T, size, keep):
    """bool [T, T]: j <= i and (i - j < size or j < keep); size 0: no window."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    near = (i - j < size) | (j < keep) if size else torch.ones(T, T, dtype=torch.bool)
    return (j <= i) & near


def attend(q, k, v, scale, size, keep):
    """q [T, H, d], k [T, G, d], v [T, G, dv] as they enter the scores.  Returns [T, H dv]."""
    rep = q.shape[1] // k.shape[1]
    ke, ve = k.repeat_interleave(rep, dim=1), v.repeat_interleave(rep, dim=1)
    s = torch.einsum("ihd,jhd->hij", q, ke) * scale
    p = torch.softmax(s.masked_fill(~window_mask(q.shape[0], size, keep), float("-inf")), dim=-1)
    return torch.einsum("hij,jhc->ihc", p, ve).reshape(q.shape[0], -1)


def normed_projection(wt, name, x, eps):
    """Biased projection, rms over the whole row, times '<name>.norm'."""
    return rms(lin(wt, name, x) + wt[name + ".b"].to(x.dtype), eps) * wt[name + ".norm"].to(x.dtype)


def attention(wt, pre, m, x, eps):
    T, H, G, d, dv = x.shape[0], int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = rotate(normed_projection(wt, pre + "q", x, eps).view(T, H, d), m.get("rot"))
    k = rotate(normed_projection(wt, pre + "k", x, eps).view(T, G, d), m.get("rot"))
    v = (lin(wt, pre + "v", x) + wt[pre + "v.b"].to(x.dtype)).view(T, G, dv)
    mask = m.get("mask") or {}
    return lin(wt, pre + "o", attend(q, k, v, float(m["scale"]), int(mask.get("size") or 0), int(mask.get("keep_first") or 0)))


# ---- the layer
def mixer(wt, pre, L, x, eps):
    m = L["mixer"]
    if L["type"] == "mlstm":
        return mlstm(wt, pre, m, x, eps)
    return float(m["left_scale"]) * attention(wt, pre + "left.", m["left"], x, eps) \
        + float(m["right_scale"]) * lightning(wt, pre + "right.", m["right"], x, eps)


def relu2_ff(wt, pre, x):
    return lin(wt, pre + "down", torch.relu(lin(wt, pre + "up", x)) ** 2)


def token_side(wt, pre, i, dim, tokens, x, eps):
    e = wt["side.embed"][torch.as_tensor(tokens, dtype=torch.int64), i * dim: (i + 1) * dim].to(x.dtype)
    return rms(lin(wt, pre + "side.proj", gelu_tanh(lin(wt, pre + "side.gate", x)) * e), eps) * wt[pre + "side.norm"].to(x.dtype)


def forward(wt, cfg, tokens, dtype=torch.float32, layers_out=None):
    """Whole-sequence forward from position 0.  Returns logits [T, vocab]; layers_out (a list) receives the
    residual stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = embed_tokens(wt, cfg, tokens, dtype)
    side = int((cfg.get("token_side") or {}).get("dim", 0))
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + rms(mixer(wt, p + "mix.", L, x, eps), eps) * (1.0 + wt[p + "norm1"].to(dtype))
        if L.get("mlp") is not None:
            x = x + rms(relu2_ff(wt, p + "mlp.", x), eps) * (1.0 + wt[p + "norm2"].to(dtype))
        if side:
            x = x + token_side(wt, p, i, side, tokens, x, eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return (rms(x, eps) * (1.0 + wt["final.norm"].to(dtype))) @ wt["embed"].to(dtype).T


def random_state(cfg, seed=0, bf16_grid=True):
    """Seeded random tensors under the checkpoint names of `cfg` (a config dict), float32; with
    bf16_grid every value is representable in bfloat16."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def mat(*shape, s=1.0, mean=0.0):
        t = torch.randn(tuple(shape), generator=g) * s + mean
        return t.to(torch.bfloat16).float() if bf16_grid else t

    D = int((cfg.get("token_side") or {}).get("dim", 0))
    st = {"embed": mat(V, W, s=W ** -0.5), "final.norm": mat(W, s=0.2)}
    if D:
        st["side.embed"] = mat(V, len(cfg["layers"]) * D)
    for i, L in enumerate(cfg["layers"]):
        p, q, m = f"l{i}.", f"l{i}.mix.", L["mixer"]
        st[p + "norm1"] = mat(W, s=0.2)
        if L["type"] == "mlstm":
            H, d, dv = m["heads"], m["dim"], m["vdim"]
            for n, rows in (("q", H * d), ("k", H * d), ("v", H * dv), ("g", H * dv), ("i", H), ("f", H)):
                st[q + n] = mat(rows, W, s=W ** -0.5)
            st[q + "i.b"], st[q + "f.b"] = mat(H, s=1.0), mat(H, s=1.0, mean=3.0)
            st[q + "norm"], st[q + "o"] = mat(H * dv, s=0.1, mean=1.0), mat(W, H * dv, s=(H * dv) ** -0.5)
        else:
            a, b, r, l = m["left"], q + "left.", m["right"], q + "right."
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                st[b + n], st[b + n + ".b"] = mat(rows, W, s=W ** -0.5), mat(rows, s=0.3)
            st[b + "q.norm"], st[b + "k.norm"] = mat(H * d, s=0.2, mean=1.0), mat(G * d, s=0.2, mean=1.0)
            st[b + "o"] = mat(W, H * dv, s=(H * dv) ** -0.5)
            H, d, dv = r["heads"], r["dim"], r["vdim"]
            for n, rows in (("q", H * d), ("k", H * d), ("v", H * dv), ("g", H * dv)):
                st[l + n] = mat(rows, W, s=W ** -0.5)
            st[l + "norm"], st[l + "o"] = mat(H * dv, s=0.1, mean=1.0), mat(W, H * dv, s=(H * dv) ** -0.5)
        if L.get("mlp") is not None:
            ff = L["mlp"]["ff"]
            st[p + "norm2"] = mat(W, s=0.2)
            st[p + "mlp.up"], st[p + "mlp.down"] = mat(ff, W, s=W ** -0.5), mat(W, ff, s=ff ** -0.5)
        if D:
            st[p + "side.gate"], st[p + "side.proj"] = mat(D, W, s=W ** -0.5), mat(W, D, s=D ** -0.5)
            st[p + "side.norm"] = mat(W, s=0.1, mean=0.5)
    return st
