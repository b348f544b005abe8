"""A plain, slow implementation of the Pitenex decoder in float64 on the CPU, one function per
mechanism, written from the design's equations.  It shares no code with the library: it reads
``config.json`` and the safetensors file by itself and works on whole sequences with dense
masks, a loop over experts and a token-by-token loop for the recurrence.

The design in this file's notation (t: a position from 0):

* embedding: ``x = E[t_n] + B[(t_{n-1} mul_prev + t_n mul_cur) mod buckets]``, the first token of a
  sequence with the last row of B;
* layer: ``h = LN(x); x <- x + m (mixer(h) + ff(h))``, one layer norm with weight and bias in front
  of both;
* mixer: ``left_scale A(h) + right_scale R(h)`` with A a rotary attention inside chunks of the
  positions whose softmax has a learned sink per head, and R the gated delta rule whose decay is a
  number per key channel;
* feed-forward: gated with the tanh form of gelu, or a routed mixture of clamped gated experts of
  which some hand their input on;
* logits: ``c E LN(x)``.
"""
import json
import math
import os

import torch

from plain_llama import read_safetensors

F = torch.float64


def load_folder(folder):
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    w = {}
    for k, v in read_safetensors(os.path.join(folder, "model.safetensors")).items():
        w[k] = v.to(F) if v.is_floating_point() else v.to(torch.int64)
    return cfg, w


# --------------------------------------------------------------------------- small pieces
def layer_norm(x, weight, bias, eps):
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * weight + bias


def over_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def embed(w, cfg, tokens):
    e = cfg["embedding"]["bigram"]
    rows = [e["buckets"]]
    for a, b in zip(tokens, tokens[1:]):
        rows.append((a * e["mul_prev"] + b * e["mul_cur"]) % e["buckets"])
    return w["embed"][torch.tensor(tokens)] + w["bigram"][torch.tensor(rows)]


# --------------------------------------------------------------------------- attention
def rotate_pairs(x, rot):
    """x [T, heads, d]: pairs (2i, 2i + 1) of the first ``dims`` elements, i < dims / 2, turned by
    t base^(-2i/dims)."""
    if not rot or not rot["dims"]:
        return x
    T, n = x.shape[0], rot["dims"]
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / n) for i in range(n // 2)], dtype=F)
    a = torch.arange(T, dtype=F)[:, None, None] * f
    out = x.clone()
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * torch.cos(a) - v * torch.sin(a)
    out[..., 1:n:2] = v * torch.cos(a) + u * torch.sin(a)
    return out


def chunk_mask(T, size):
    """[i, j]: j <= i within one chunk of ``size`` positions."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def softmax_with_sink(s, sink):
    """s [H, T, T] (masked entries -inf), sink [H]: exp(sink) joins the denominator."""
    m = torch.maximum(s.max(-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink[:, None, None] - m))


def chunked_attention(w, p, m, h):
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate_pairs((h @ w[p + "q"].T).view(T, H, d), m.get("rot"))
    k = rotate_pairs((h @ w[p + "k"].T).view(T, G, d), m.get("rot"))
    v = (h @ w[p + "v"].T).view(T, G, dv)
    of = [i // (H // G) for i in range(H)]
    s = torch.einsum("ihd,jhd->hij", q, k[:, of]) * m["scale"]
    s = s.masked_fill(~chunk_mask(T, m["mask"]["size"]), -math.inf)
    o = torch.einsum("hij,jhe->ihe", softmax_with_sink(s, w[p + "sink"]), v[:, of])
    return o.reshape(T, H * dv) @ w[p + "o"].T


# --------------------------------------------------------------------------- the recurrence
def short_convolution(x, taps):
    """x [T, C], taps [C, K]: y_t = sum_k taps[:, k] x_{t - (K - 1) + k}, zeros before the start."""
    T, K = x.shape[0], taps.shape[1]
    y = torch.zeros_like(x)
    for k in range(K):
        back = K - 1 - k
        if back < T:
            y[back:] += taps[:, k] * x[:T - back]
    return y


def channel_delta_rule(q, k, v, beta, g):
    """q, k, g [T, H, d], v [T, H, dv], beta [T, H] -> [T, H, dv], S [H, d, dv] from zero."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = []
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hde,hd->he", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append(torch.einsum("hde,hd->he", S, q[t]))
    return torch.stack(out)


def delta_mixer(w, p, m, eps, h):
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    of = [i // (H // G) for i in range(H)]
    conv = {n: silu(short_convolution(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv"}
    q = unit(conv["q"].view(T, G, d))[:, of] * d ** -0.5
    k = unit(conv["k"].view(T, G, d))[:, of]
    beta = torch.sigmoid(h @ w[p + "b"].T)
    z = (h @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "dt_bias"]).view(T, H, d)
    g = torch.exp(-torch.exp(w[p + "A_log"])[:, None] * softplus(z))
    o = channel_delta_rule(q, k, conv["v"].view(T, H, dv), beta, g)
    gate = torch.sigmoid(h @ w[p + "g1"].T @ w[p + "g2"].T).view(T, H, dv)
    return (over_rms(o, eps) * w[p + "norm"] * gate).reshape(T, H * dv) @ w[p + "o"].T


def mixer(w, p, m, eps, h):
    return (m["left_scale"] * chunked_attention(w, p + "left.", m["left"], h)
            + m["right_scale"] * delta_mixer(w, p + "right.", m["right"], eps, h))


# --------------------------------------------------------------------------- feed-forwards
def dense(w, p, h):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def clamped_expert(w, p, limit, h):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def route(z, correction, top):
    """z [T, E] -> (chosen [T, top], weights [T, top])."""
    s = torch.softmax(z, -1)
    chosen = torch.topk(s + correction, top, -1).indices
    picked = torch.gather(s, -1, chosen)
    return chosen, picked / (picked.sum(-1, keepdim=True) + 1e-20)


def mixture(w, p, mlp, h):
    r = mlp["router"]
    chosen, weights = route(h @ w[p + "router"].T, w[p + "correction"], r["top"])
    y = torch.zeros_like(h)
    for e in range(r["experts"] + r.get("identity", 0)):
        share = (weights * (chosen == e)).sum(-1, keepdim=True)
        y += share * (clamped_expert(w, f"{p}e{e}.", mlp["expert"]["limit"], h) if e < r["experts"] else h)
    if mlp.get("shared"):
        y += clamped_expert(w, p + "shared.", mlp["shared"]["limit"], h)
    return y


def feed_forward(w, p, mlp, h):
    return dense(w, p, h) if mlp["kind"] == "dense" else mixture(w, p, mlp, h)


# --------------------------------------------------------------------------- whole model
def forward(w, cfg, tokens, outs=None):
    """Logits [T, vocab] of one sequence; ``outs``: a list that gets the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = embed(w, cfg, tokens)
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps)
        y = mixer(w, p + "mix.", layer["mixer"], eps, h)
        if layer.get("mlp") is not None:
            y = y + feed_forward(w, p + "mlp.", layer["mlp"], h)
        x = x + cfg["residual_mult"] * y
        if outs is not None:
            outs.append(x)
    return layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["embed"].T * cfg["logit_scale"]


def greedy_generate(w, cfg, prompt, max_new_tokens):
    tokens = list(prompt)
    for _ in range(max_new_tokens):
        tokens.append(int(forward(w, cfg, tokens)[-1].argmax()))
    return tokens[len(prompt):]
