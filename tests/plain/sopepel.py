"""The plain Sopepel model: one function per mechanism, written from the design's equations, whole sequences at once, no
cache, no batching, float64 by default. It shares no code with the engine; the tests hold the engine to it.

Notation: x [n, W] the residual stream of a sequence of n tokens at positions 0 .. n - 1; `w` maps checkpoint tensor
names to tensors; `p` is a tensor name prefix; N(v) = v / sqrt(mean(v^2) + eps).

  embedding    x_i = E[t_i] + B[(t_(i-1) mul_prev + t_i mul_cur) mod buckets], the first token: E[t_0] + B[buckets]
  layer        x <- x + N(mixer(x)) g1; x <- x + N(ffn(x)) g2
  mixer        left_scale attention(x) + right_scale linear_attention(x)
  attention    q, k, v = W x + b per head; q, k <- turn(N(q) gq), turn(N(k) gk); p = softmax over the keys j <= i of i's
               own chunk (j div size = i div size) of scale q . k; o_h = (p v)_h sigmoid((Wg x)_h); Wo o + bo
  turning      pair (i, i + dims / 2): (u, v) -> (u cos t - v sin t, v cos t + u sin t), t = p base^(-2i / dims)
  linear_attention  per head: alpha = sigmoid(Wa2 Wa1 x + ba2)^(1 / tau); S <- diag(alpha) S + k v^T;
               o = S^T q dim^(-1/2); o <- N(o) g; Wo (o silu(Wg x))
  dense        Wdown (gelu(Wgate x) * (Wup x)), gelu in its tanh form
  experts      s = sigmoid(Wr x); the `top` largest are chosen; sum of Wdown relu(Wup (s x))^2 over them, plus the shared
               one's Wdown relu(Wup x)^2 times sigmoid(Wsg x)
  head         E (N(x) g) logit_scale
"""
from __future__ import annotations

import math

import torch


def unit(v, eps):
    return v / torch.sqrt(v.pow(2).mean(-1, keepdim=True) + eps)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def bigram_rows(ids, bigram):
    """The row of the bigram table each token takes."""
    rows, prev = [], None
    for t in ids:
        rows.append(bigram["buckets"] if prev is None else (prev * bigram["mul_prev"] + t * bigram["mul_cur"]) % bigram["buckets"])
        prev = t
    return rows


def embedding(w, config, ids, with_bigram=True):
    x = w["embed"][torch.tensor(ids)]
    return x + w["bigram"][torch.tensor(bigram_rows(ids, config["embedding"]["bigram"]))] if with_bigram else x


def turn(u, rot):
    """u [n, ..., d]: dimension i paired with i + dims / 2, for i below dims / 2."""
    dims = rot["dims"]
    f = torch.tensor([rot["base"] ** (-2 * i / dims) for i in range(dims // 2)], dtype=u.dtype)
    t = torch.arange(u.shape[0], dtype=u.dtype)[:, None] * f
    t = t.view((u.shape[0],) + (1,) * (u.dim() - 2) + (dims // 2,))
    a, b = u[..., : dims // 2], u[..., dims // 2: dims]
    return torch.cat((a * t.cos() - b * t.sin(), b * t.cos() + a * t.sin(), u[..., dims:]), dim=-1)


def seen(n, size):
    """[n, n]: whether query i sees key j."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & (i // size == j // size)


def heads_of(w, p, x, name, heads, eps):
    """A projection as heads, each normed: [n, heads, dim]."""
    y = (x @ w[p + name].T + w[f"{p}{name}.b"]).view(x.shape[0], heads, -1)
    return unit(y, eps) * w[f"{p}{name}.norm"]


def attention(w, p, m, x, eps, gate=True):
    n, heads, groups = x.shape[0], m["heads"], m["kv_heads"]
    q, k = heads_of(w, p, x, "q", heads, eps), heads_of(w, p, x, "k", groups, eps)
    v = (x @ w[p + "v"].T + w[p + "v.b"]).view(n, groups, m["vdim"])
    if m.get("rot"):
        q, k = turn(q, m["rot"]), turn(k, m["rot"])
    gates = sigmoid(x @ w[p + "g"].T)
    visible = seen(n, m["mask"]["size"])
    out = x.new_zeros(n, heads, m["vdim"])
    for h in range(heads):
        g = h // (heads // groups)
        s = (q[:, h] @ k[:, g].T * m["scale"]).masked_fill(~visible, -math.inf)
        out[:, h] = torch.softmax(s, dim=-1) @ v[:, g] * (gates[:, h: h + 1] if gate else 1)
    return out.reshape(n, -1) @ w[p + "o"].T + w[p + "o.b"]


def decays(w, p, m, x):
    z = x @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "a2.b"]
    return (sigmoid(z) ** (1 / m["tau"])).view(x.shape[0], m["heads"], m["dim"])


def linear_attention_scan(q, k, v, alpha):
    """q, k, alpha [n, H, D], v [n, H, V] -> [n, H, V], token by token."""
    n, heads, dim = q.shape
    S = v.new_zeros(heads, dim, v.shape[2])
    out = torch.empty_like(v)
    for t in range(n):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def linear_attention(w, p, m, x, eps):
    n, heads, dim, vdim = x.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (x @ w[p + "q"].T).view(n, heads, dim) * dim ** -0.5
    k, v = (x @ w[p + "k"].T).view(n, heads, dim), (x @ w[p + "v"].T).view(n, heads, vdim)
    o = unit(linear_attention_scan(q, k, v, decays(w, p, m, x)), eps) * w[p + "norm"]
    z = x @ w[p + "g"].T
    return (o.reshape(n, -1) * z * sigmoid(z)) @ w[p + "o"].T


def mixer(w, p, m, x, eps, gate=True):
    return m["left_scale"] * attention(w, p + "left.", m["left"], x, eps, gate) + \
        m["right_scale"] * linear_attention(w, p + "right.", m["right"], x, eps)


def dense_ffn(w, p, x):
    return (gelu_tanh(x @ w[p + "gate"].T) * (x @ w[p + "up"].T)) @ w[p + "down"].T


def expert(w, p, x):
    return torch.relu(x @ w[p + "up"].T) ** 2 @ w[p + "down"].T


def route(z, top):
    """z [E] -> [(expert, weight)]."""
    s = sigmoid(z)
    return [(e, s[e]) for e in sorted(range(s.shape[0]), key=lambda e: -float(s[e]))[:top]]


def moe_ffn(w, p, mlp, x):
    z = x @ w[p + "router"].T
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for e, weight in route(z[t], mlp["router"]["top"]):
            out[t] += expert(w, f"{p}e{e}.", weight * x[t])
    if mlp.get("shared"):
        out = out + expert(w, p + "shared.", x) * sigmoid(x @ w[p + "shared.sg"].T)
    return out


def forward(config, tensors, ids, dtype=torch.float64, gate=True, with_bigram=True):
    """-> (logits [n, vocab], the residual stream after every layer [[n, W]]). `gate` and `with_bigram` False leave a
    mechanism out (for tests that show what it does)."""
    w = {k: v.to(dtype) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    x = embedding(w, config, ids, with_bigram)
    streams = []
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        x = x + unit(mixer(w, p + "mix.", layer["mixer"], x, eps, gate), eps) * w[p + "norm1"]
        mlp = layer.get("mlp")
        if mlp:
            y = dense_ffn(w, p + "mlp.", x) if mlp["kind"] == "dense" else moe_ffn(w, p + "mlp.", mlp, x)
            x = x + unit(y, eps) * w[p + "norm2"]
        streams.append(x)
    return (unit(x, eps) * w["final.norm"]) @ w["embed"].T * config["logit_scale"], streams
