"""The plain Falisun model: one function per mechanism, written from the design's equations, whole sequences at once,
no cache, no batching, float64 by default. It shares no code with the engine; the tests hold the engine to it.

Notation: x [n, W] the residual stream of a sequence of n tokens at positions 0 .. n - 1; `w` maps checkpoint tensor
names to tensors; `p` is a tensor name prefix; N(v) = v / sqrt(mean(v^2) + eps).

  layer             x <- x + ls1 * (N(mixer(N(x) g1)) g1b); x <- x + ls2 * (N(ffn(N(x) g2)) g2b)
  latent_attention  q = Wq a as [H, dim | rot]; Wdkv a = [c' | r']; c = N(c') gc; r = turn(r'); k_h = [Wuk,h c | r],
                    v_h = Wuv,h c; p = softmax over j <= i of scale [q_h, turned] . k_h; o = concat_h(p v_h) * sigmoid(Wg a);
                    Wo o. With `kv_from` = j, c and r are layer j's.
  turning           pair (i, i + dims / 2): (u, v) -> (u cos t - v sin t, v cos t + u sin t) (0.1 ln factor + 1), t = p f'_i,
                    f'_i the frequencies base^(-2i / dims) rescaled as YaRN does
  mamba2            Win a = [z | u | b]; [x B C] = silu(conv(u)), dt = softplus(b + dt_bias); per head h of group g:
                    S <- exp(-exp(A_log_h) dt) S + dt B_g x_h^T, y_h = S^T C_g + D_h x_h; y <- N over each of
                    `norm_groups` parts of (y silu(z)), times its weight; Wo y
  experts           s = softmax(Wr a); a group's score is its largest s; among the experts of the `keep` best groups the
                    `top` largest s are chosen, weights s / (sum of the chosen + 1e-20); + the shared expert
"""
from __future__ import annotations

import math

import torch


def unit(v, eps):
    return v / torch.sqrt(v.pow(2).mean(-1, keepdim=True) + eps)


def silu(z):
    return z / (1 + torch.exp(-z))


def frequencies(rot, dtype=torch.float64):
    """([dims / 2] frequencies, the factor of cos and sin)."""
    dims, base = rot["dims"], rot["base"]
    plain = [base ** (-2 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return torch.tensor(plain, dtype=dtype), 1.0

    def index_of(turns):
        return dims * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(index_of(s["fast"])), 0), min(math.ceil(index_of(s["slow"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * ramp + f * (1 - ramp))
    return torch.tensor(out, dtype=dtype), 0.1 * math.log(s["factor"]) + 1.0


def turn(u, rot):
    """u [n, ..., d]: dimension i paired with i + dims / 2."""
    f, gain = frequencies(rot, u.dtype)
    dims = rot["dims"]
    t = torch.arange(u.shape[0], dtype=u.dtype)[:, None] * f
    t = t.view((u.shape[0],) + (1,) * (u.dim() - 2) + (dims // 2,))
    a, b = u[..., : dims // 2], u[..., dims // 2: dims]
    return torch.cat(((a * t.cos() - b * t.sin()) * gain, (b * t.cos() + a * t.sin()) * gain, u[..., dims:]), dim=-1)


def hidden(n):
    return torch.arange(n)[None, :] > torch.arange(n)[:, None]


def latent(w, p, m, a, eps):
    """What a token leaves for later ones: (c [n, kv_rank], the turned key part [n, rot_dim])."""
    both = a @ w[p + "dkv"].T
    return unit(both[:, : m["kv_rank"]], eps) * w[p + "dkv.norm"], turn(both[:, m["kv_rank"]:], m["rot"])


def latent_attention(w, p, m, a, kept, gate=True):
    n, heads, dim, vdim = a.shape[0], m["heads"], m["dim"], m["vdim"]
    c, r = kept
    q = (a @ w[p + "q"].T).view(n, heads, dim + m["rot_dim"])
    turned = turn(q[..., dim:], m["rot"])
    uk, uv = w[p + "uk"].view(heads, dim, -1), w[p + "uv"].view(heads, vdim, -1)
    out = a.new_zeros(n, heads, vdim)
    for h in range(heads):
        s = (q[:, h, :dim] @ (c @ uk[h].T).T + turned[:, h] @ r.T) * m["scale"]
        out[:, h] = torch.softmax(s.masked_fill(hidden(n), -math.inf), dim=-1) @ (c @ uv[h].T)
    out = out.reshape(n, -1)
    if gate:
        out = out * torch.sigmoid(a @ w[p + "g"].T)
    return out @ w[p + "o"].T


def causal_filter(u, taps, bias):
    """u [n, C], taps [C, T], the last one for the current token; zeros before the start."""
    n, k = u.shape[0], taps.shape[1]
    padded = torch.cat((u.new_zeros(k - 1, u.shape[1]), u))
    return sum(taps[:, j] * padded[j: j + n] for j in range(k)) + bias


def softplus(v):
    return torch.log1p(torch.exp(-v.abs())) + v.clamp(min=0)


def ssd(x, B, C, dt, A_log, D):
    """x [n, H, V], B, C [n, G, N], dt [n, H] -> y [n, H, V], token by token."""
    n, heads, vdim = x.shape
    group = heads // B.shape[1]
    S = x.new_zeros(heads, B.shape[2], vdim)
    y = torch.empty_like(x)
    for t in range(n):
        for h in range(heads):
            b, c = B[t, h // group], C[t, h // group]
            S[h] = torch.exp(-torch.exp(A_log[h]) * dt[t, h]) * S[h] + dt[t, h] * torch.outer(b, x[t, h])
            y[t, h] = S[h].T @ c + D[h] * x[t, h]
    return y


def mamba2(w, p, m, a, eps):
    n, heads, vdim, groups, state = a.shape[0], m["heads"], m["vdim"], m["groups"], m["state"]
    inner, gn = heads * vdim, groups * state
    z, u, b = torch.split(a @ w[p + "in"].T, [inner, inner + 2 * gn, heads], dim=-1)
    u = silu(causal_filter(u, w[p + "conv"], w[p + "conv.b"]))
    x, B, C = torch.split(u, [inner, gn, gn], dim=-1)
    y = ssd(x.reshape(n, heads, vdim), B.reshape(n, groups, state), C.reshape(n, groups, state),
            softplus(b + w[p + "dt_bias"]), w[p + "A_log"], w[p + "D"])
    y = (y.reshape(n, inner) * silu(z)).view(n, m["norm_groups"], -1)
    return (unit(y, eps).reshape(n, inner) * w[p + "norm"]) @ w[p + "o"].T


def expert(w, p, a):
    return (silu(a @ w[p + "gate"].T) * (a @ w[p + "up"].T)) @ w[p + "down"].T


def route(z, router):
    """z [E] -> [(expert, weight)]."""
    s = torch.softmax(z, dim=0)
    experts, top = s.shape[0], router["top"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    size = experts // groups["count"]
    best = sorted(range(groups["count"]), key=lambda g: -float(s[g * size: (g + 1) * size].max()))[: groups["keep"]]
    allowed = [e for e in range(experts) if e // size in best]
    chosen = sorted(allowed, key=lambda e: -float(s[e]))[:top]
    total = sum(s[e] for e in chosen) + 1e-20
    return [(e, s[e] / total) for e in chosen]


def moe_ffn(w, p, mlp, a):
    z = a @ w[p + "router"].T
    out = torch.zeros_like(a)
    for t in range(a.shape[0]):
        for e, weight in route(z[t], mlp["router"]):
            out[t] += weight * expert(w, f"{p}e{e}.", a[t: t + 1])[0]
    if mlp.get("shared"):
        out = out + expert(w, p + "shared.", a)
    return out


def forward(config, tensors, ids, dtype=torch.float64, gate=True):
    """-> (logits [n, vocab], the residual stream after every layer [[n, W]]). `gate` False leaves the attention's
    output gate out (for tests that show what it does)."""
    w = {k: v.to(dtype) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.tensor(ids)]
    streams, kept = [], {}
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        a = unit(x, eps) * w[p + "norm1"]
        if layer["type"] == "mamba2":
            y = mamba2(w, p + "mix.", m, a, eps)
        else:
            src = m.get("kv_from")
            if src is None:
                src, kept[i] = i, latent(w, p + "mix.", m, a, eps)
            y = latent_attention(w, p + "mix.", m, a, kept[src], gate)
        x = x + unit(y, eps) * w[p + "norm1b"] * w[p + "ls1"]
        if layer.get("mlp"):
            y = moe_ffn(w, p + "mlp.", layer["mlp"], unit(x, eps) * w[p + "norm2"])
            x = x + unit(y, eps) * w[p + "norm2b"] * w[p + "ls2"]
        streams.append(x)
    return (unit(x, eps) * w["final.norm"]) @ w["embed"].T, streams
