"""Plain, slow restatement of the Bapavik decoder in float32 (or float64) torch on the CPU, one
function per mechanism.  TEST INFRASTRUCTURE (see oracle/__init__.py): nothing here is imported by
the product and nothing of the product is imported here.

Notation.  W: model width; ln(x; g) = (x - m) / sqrt(mean((x - m)^2) + eps) * g, m = mean(x);
rms(x; g) = x / sqrt(mean(x^2) + eps) * g.

    x0[t]  = embed[tok_t] * embedding.scale
    layer:   x += mixer(ln(x; norm1));  x += ff(ln(x; norm2))   (a layer may have no ff)
    loop:    layers start .. stop - 1 run `times` times in a row with one set of weights, every pass
             attending to keys of its own
    logits = head ln(x; final.norm)

Mixers
  * "attention": H query heads on G key/value heads; q = rms(Q h; gq), k = rms(K h; gk), each norm over all
    heads of the row at once; no rotation; q is multiplied by a temperature that grows with the position,
    1 + coef ln(floor((p + 1) / every) + 1); s = cap tanh(q.k scale / cap); causal; the softmax denominator
    holds one more term exp(sink[head]) that carries no value and takes no part in scale and cap; O.
  * "latent_attention": c = rms(first kv_rank rows of D h), one rotated key part per token from the
    remaining rot_dim rows; per head key [UK c | rotated part], value UV c; query [unrotated | rotated] per
    head; rotation of neighbours (coordinates 2i, 2i + 1) by p base^(-2i / dims); causal softmax; O.

Feed-forward
  * dense: g = min(G h, limit), u = clamp(U h, -limit, limit); D (g sigmoid(1.702 g) (u + 1));
  * mixture without a router: row token id of a table names the token's experts, each of weight
    1 / top; an expert is D relu(U h)^2.
"""
from __future__ import annotations

import math

import torch


def layer_norm(x, g, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * g


def rms_norm(x, g, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * g


def query_temperature(T, q_temp, dtype=torch.float32):
    """[T] factor on the queries of positions 0 .. T - 1."""
    if not q_temp:
        return torch.ones(T, dtype=dtype)
    return torch.tensor([1.0 + q_temp["coef"] * math.log(math.floor((p + 1) / q_temp["every"]) + 1) for p in range(T)],
                        dtype=dtype)


def capped(s, cap):
    return cap * torch.tanh(s / cap) if cap else s


def causal_weights(s, sink=None):
    """s [T, T] (query, key) -> softmax weights over the keys up to the query; sink: one number, a term of the
    denominator without a value."""
    T = s.shape[0]
    hidden = torch.ones(T, T, dtype=torch.bool).triu(1)
    s = s.masked_fill(hidden, float("-inf"))
    top = s.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink.to(s.dtype).expand_as(top))
    e = torch.exp(s - top)
    den = e.sum(-1, keepdim=True)
    if sink is not None:
        den = den + torch.exp(sink - top)
    return e / den


def attention(q, k, v, scale, cap, sink):
    """q [T, H, d], k [T, G, d], v [T, G, dv], sink [H] or None -> [T, H * dv]."""
    H, G = q.shape[1], k.shape[1]
    out = []
    for h in range(H):
        g = h // (H // G)
        s = capped(q[:, h] @ k[:, g].T * scale, cap)
        out.append(causal_weights(s, None if sink is None else sink[h]) @ v[:, g])
    return torch.cat(out, dim=-1)


def attention_mixer(wt, p, m, h, eps):
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ wt[p + "q"].T, wt[p + "q.norm"], eps)
    k = rms_norm(h @ wt[p + "k"].T, wt[p + "k.norm"], eps)
    v = h @ wt[p + "v"].T
    q = q * query_temperature(T, m.get("q_temp"), h.dtype)[:, None]
    o = attention(q.view(T, H, d), k.view(T, G, d), v.view(T, G, dv), m["scale"], m.get("softcap"), wt.get(p + "sink"))
    return o @ wt[p + "o"].T


def rotate_neighbours(x, rot):
    """x [T, ..., n]: coordinates 2i and 2i + 1 of the first rot.dims turn together, row t by t base^(-2i / dims)."""
    T, R = x.shape[0], int(rot["dims"])
    i = torch.arange(R // 2, dtype=torch.float64)
    a = torch.arange(T, dtype=torch.float64)[:, None] * float(rot["base"]) ** (-2.0 * i / R)
    shape = [T] + [1] * (x.dim() - 2) + [R // 2]
    c, s = torch.cos(a).to(x.dtype).view(shape), torch.sin(a).to(x.dtype).view(shape)
    y = x.clone()
    u, v = x[..., 0:R:2], x[..., 1:R:2]
    y[..., 0:R:2], y[..., 1:R:2] = u * c - v * s, v * c + u * s
    return y


def latent_of(wt, p, m, h, eps):
    """(c [T, kv_rank], rotated shared key part [T, rot_dim])."""
    z, R = h @ wt[p + "dkv"].T, m["kv_rank"]
    return rms_norm(z[:, :R], wt[p + "dkv.norm"], eps), rotate_neighbours(z[:, R:], m["rot"])


def latent_attention_mixer(wt, p, m, h, eps):
    T, H, d, r, dv = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    q = (h @ wt[p + "q"].T).view(T, H, d + r)
    c, kr = latent_of(wt, p, m, h, eps)
    qr = rotate_neighbours(q[..., d:], m["rot"])
    kn, v = (c @ wt[p + "uk"].T).view(T, H, d), (c @ wt[p + "uv"].T).view(T, H, dv)
    out = []
    for i in range(H):
        s = (q[:, i, :d] @ kn[:, i].T + qr[:, i] @ kr.T) * m["scale"]
        out.append(causal_weights(s) @ v[:, i])
    return torch.cat(out, dim=-1) @ wt[p + "o"].T


def limited_act(g, u, limit):
    g = torch.clamp(g, max=limit)
    u = torch.clamp(u, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def dense_ff(wt, p, mlp, h):
    return limited_act(h @ wt[p + "gate"].T, h @ wt[p + "up"].T, mlp["limit"]) @ wt[p + "down"].T


def expert(wt, p, h):
    return torch.relu(h @ wt[p + "up"].T) ** 2 @ wt[p + "down"].T


def table_moe_ff(wt, p, mlp, h, tokens):
    top, out = mlp["router"]["top"], torch.zeros_like(h)
    table = wt[p + "table"]
    for t, tok in enumerate(tokens):
        for e in table[tok].tolist():
            out[t] += expert(wt, f"{p}e{int(e)}.", h[t:t + 1])[0] / top
    return out


def runs(cfg):
    """Layer numbers in the order they run."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return list(range(n))
    a, b = lp["start"], lp["stop"]
    return list(range(a)) + list(range(a, b)) * lp["times"] + list(range(b, n))


def forward(wt, cfg, tokens, trace=None):
    """Logits [T, vocab] of one whole sequence; wt: name -> tensor.  `trace`, a list, receives the
    residual stream after every layer run."""
    eps = cfg["norm"]["eps"]
    tokens = [int(t) for t in tokens]
    x = wt["embed"][torch.as_tensor(tokens)] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    for i in runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        mixer = {"attention": attention_mixer, "latent_attention": latent_attention_mixer}[L["type"]]
        x = x + mixer(wt, p + "mix.", L["mixer"], layer_norm(x, wt[p + "norm1"], eps), eps)
        mlp = L.get("mlp")
        if mlp is not None:
            h = layer_norm(x, wt[p + "norm2"], eps)
            x = x + (table_moe_ff(wt, p + "mlp.", mlp, h, tokens) if mlp["kind"] == "moe" else dense_ff(wt, p + "mlp.", mlp, h))
        if trace is not None:
            trace.append(x.clone())
    return layer_norm(x, wt["final.norm"], eps) @ wt["head"].T


def random_state(cfg, seed=0, bf16_grid=True):
    """Seeded random tensors under the checkpoint names of `cfg` (a config dict), float32 (tables int32);
    with bf16_grid every value is representable in bfloat16."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def mat(*shape, s=1.0, mean=0.0):
        t = torch.randn(tuple(shape), generator=g) * s + mean
        return t.to(torch.bfloat16).float() if bf16_grid else t

    st = {"embed": mat(V, W, s=1.0 / float((cfg.get("embedding") or {}).get("scale", 1.0))), "head": mat(V, W, s=W ** -0.5),
          "final.norm": mat(W, s=0.1, mean=1.0)}
    for i, L in enumerate(cfg["layers"]):
        p, q, m = f"l{i}.", f"l{i}.mix.", L["mixer"]
        st[p + "norm1"] = mat(W, s=0.1, mean=1.0)
        if L["type"] == "attention":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                st[q + n] = mat(rows, W, s=W ** -0.5)
            st[q + "q.norm"], st[q + "k.norm"] = mat(H * d, s=0.3, mean=1.5), mat(G * d, s=0.3, mean=1.5)
            st[q + "sink"] = mat(H, s=1.0, mean=1.0)
            st[q + "o"] = mat(W, H * dv, s=(H * dv) ** -0.5)
        else:
            H, d, r, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            st[q + "q"], st[q + "dkv"] = mat(H * (d + r), W, s=2.0 * W ** -0.5), mat(R + r, W, s=2.0 * W ** -0.5)
            st[q + "dkv.norm"] = mat(R, s=0.1, mean=1.0)
            st[q + "uk"], st[q + "uv"] = mat(H * d, R, s=R ** -0.5), mat(H * dv, R, s=R ** -0.5)
            st[q + "o"] = mat(W, H * dv, s=(H * dv) ** -0.5)
        mlp = L.get("mlp")
        if mlp is None:
            continue
        st[p + "norm2"] = mat(W, s=0.1, mean=1.0)
        f = p + "mlp."
        if mlp["kind"] == "moe":
            E, top, Fw = mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"]
            st[f + "table"] = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(V)]).to(torch.int32)
            for e in range(E):
                st[f"{f}e{e}.up"], st[f"{f}e{e}.down"] = mat(Fw, W, s=W ** -0.5), mat(W, Fw, s=Fw ** -0.5)
        else:
            for n, shape in (("gate", (mlp["ff"], W)), ("up", (mlp["ff"], W)), ("down", (W, mlp["ff"]))):
                st[f + n] = mat(*shape, s=shape[1] ** -0.5)
    return st


def greedy(wt, cfg, prompt, steps):
    """Greedy continuation of one prompt by full recomputation; returns (tokens, their logits rows)."""
    toks, rows = list(prompt), []
    for _ in range(steps):
        z = forward(wt, cfg, toks)[-1]
        rows.append(z)
        toks.append(int(torch.argmax(z)))
    return toks[len(prompt):], torch.stack(rows)
