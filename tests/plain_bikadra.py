"""A plain, slow implementation of the Bikadra decoder in float64 on the CPU, one function per
mechanism, written from the design's equations.  It shares no code with the library: it reads
``config.json`` and the safetensors file by itself and works on whole sequences with dense
masks, expanded keys and values, and a token-by-token loop for the recurrence.

The design in this file's notation (h: what a sublayer reads, t: a position from 0):

* streams: ``X_1 = ... = X_S = c_embed E[token]``; a sublayer q of a layer reads
  ``rms(sum_s a_s X_s) w`` and gives y; all streams move at once,
  ``X_t <- sum_s M[s, t] X_s + b_t y``; the model's output reads ``sum_s X_s``.
* mixer "latent_attention": one latent per token in place of keys and values, a rotated key
  part shared by the heads, queries through a latent, a gate per head on the result.
* mixer "mamba2": a matrix state per head with a decay that depends on the token, behind a short
  causal convolution, gated before it is normed.
* feed-forward: two matrices with the tanh form of gelu between them.
* layers ``loop.start .. loop.stop - 1`` run ``loop.times`` times with the same weights.
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
def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return unit_rms(x, eps) * weight


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# --------------------------------------------------------------------------- streams
def stream_read(X, a):
    """X [S, T, D], a [S] -> sum_s a_s X_s."""
    return torch.einsum("s,std->td", a, X)


def stream_write(X, mix, out, y):
    """New streams: stream t is ``sum_s mix[s, t] X_s + out[t] y``; mix is [from, to]."""
    return torch.einsum("st,snd->tnd", mix, X) + out[:, None, None] * y[None]


# --------------------------------------------------------------------------- rotation
def rotary_frequencies(rot):
    """(frequencies [dims / 2], factor on cos and sin).  Plain ladder ``base^(-2i/dims)``; with
    ``scaling`` the slow end is divided by ``factor`` along a linear ramp between the places
    whose pairs make ``fast`` and ``slow`` full turns over ``original`` positions, and cos and sin
    grow by ``0.1 ln(factor) + 1``."""
    dims, base = int(rot["dims"]), float(rot["base"])
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=F)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    factor, original = float(sc["factor"]), float(sc["original"])

    def place(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(place(float(sc["fast"]))), 0)
    hi = min(math.ceil(place(float(sc["slow"]))), dims - 1)
    ramp = torch.tensor([min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(half)], dtype=F)
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rotate_half(x, positions, rot):
    """x [T, heads, d]: pairs (i, i + dims/2) of the first ``rot.dims`` elements turned by
    position times frequency: (u, v) -> (u cos - v sin, v cos + u sin)."""
    if not rot or not int(rot.get("dims", 0)):
        return x
    dims = int(rot["dims"])
    half = dims // 2
    f, grow = rotary_frequencies(rot)
    a = positions.to(F)[:, None] * f[None, :]
    cos, sin = (torch.cos(a) * grow)[:, None, :], (torch.sin(a) * grow)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    out = x.clone()
    out[..., :half] = u * cos - v * sin
    out[..., half:dims] = v * cos + u * sin
    return out


# --------------------------------------------------------------------------- mixers
def causal_attention(q, k, v, scale):
    """q, k [T, H, d], v [T, H, dv] -> [T, H, dv]; position i sees every j <= i."""
    T = q.shape[0]
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    s = s.masked_fill(torch.arange(T)[None, :] > torch.arange(T)[:, None], -math.inf)
    return torch.einsum("hij,jhd->ihd", torch.softmax(s, -1), v)


def latent_attention(w, p, m, eps, h):
    """Keys and values are written out in full here (every head's own)."""
    T, H, d, dr, dv, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    cq = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    q = (cq @ w[p + "uq"].T).view(T, H, d + dr)
    kv = h @ w[p + "dkv"].T
    c = rms_norm(kv[:, :R], w[p + "dkv.norm"], eps)
    kr = rotate_half(kv[:, None, R:], pos, m.get("rot"))                # one head, shared
    q = torch.cat([q[..., :d], rotate_half(q[..., d:], pos, m.get("rot"))], -1)
    k = torch.cat([(c @ w[p + "uk"].T).view(T, H, d), kr.expand(T, H, dr)], -1)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    o = causal_attention(q, k, v, m["scale"])
    o = o * torch.sigmoid(h @ w[p + "g"].T)[..., None]
    return o.reshape(T, H * dv) @ w[p + "o"].T


def short_convolution(x, taps, bias):
    """x [T, C], taps [C, K] (last column: the current token), zeros before the start."""
    K = taps.shape[1]
    padded = torch.cat([torch.zeros(K - 1, x.shape[1], dtype=x.dtype), x])
    return sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(K)) + bias


def state_space(x, B, C, dt, A_log, D):
    """x [T, H, dv], B, C [T, G, N], dt [T, H] (after softplus) -> y [T, H, dv], token by token:
    ``S <- exp(-exp(A_log) dt) S + dt B x^T; y = S^T C + D x``."""
    T, H, dv = x.shape
    G, N = B.shape[1:]
    S = torch.zeros(H, N, dv, dtype=x.dtype)
    group = torch.arange(H) // (H // G)
    out = []
    for t in range(T):
        decay = torch.exp(-torch.exp(A_log) * dt[t])
        S = decay[:, None, None] * S + dt[t][:, None, None] * B[t][group][:, :, None] * x[t][:, None, :]
        out.append(torch.einsum("hnd,hn->hd", S, C[t][group]) + D[:, None] * x[t])
    return torch.stack(out)


def gated_group_norm(y, z, weight, groups, eps):
    """The gate first, then every one of ``groups`` equal parts by its own root mean square."""
    T, W = y.shape
    u = (y * silu(z)).view(T, groups, W // groups)
    return unit_rms(u, eps).reshape(T, W) * weight


def mamba2(w, p, m, eps, h):
    T, H, dv, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * dv
    row = h @ w[p + "in"].T
    z, xbc, dt = row[:, :inner], row[:, inner:2 * inner + 2 * G * N], row[:, 2 * inner + 2 * G * N:]
    xbc = silu(short_convolution(xbc, w[p + "conv"], w[p + "conv.b"]))
    x = xbc[:, :inner].view(T, H, dv)
    B = xbc[:, inner:inner + G * N].view(T, G, N)
    C = xbc[:, inner + G * N:].view(T, G, N)
    y = state_space(x, B, C, softplus(dt + w[p + "dt_bias"]), w[p + "A_log"], w[p + "D"])
    return gated_group_norm(y.reshape(T, inner), z, w[p + "norm"], m["norm_groups"], eps) @ w[p + "o"].T


MIXERS = {"latent_attention": latent_attention, "mamba2": mamba2}


def dense_feed_forward(w, p, h):
    return gelu_tanh(h @ w[p + "up"].T) @ w[p + "down"].T


# --------------------------------------------------------------------------- whole model
def run_order(cfg):
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def forward(w, cfg, tokens, taps=None):
    """Logits [T, vocab] of one sequence; ``taps``: a list that gets the sum of the streams
    after every layer run."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    X = x[None].repeat(cfg.get("streams", 1), 1, 1)
    for i in run_order(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        subs = [lambda h: MIXERS[layer["type"]](w, p + "mix.", layer["mixer"], eps, h)]
        if layer.get("mlp") is not None:
            subs.append(lambda h: dense_feed_forward(w, p + "mlp.", h))
        for q, sub in enumerate(subs, 1):
            hc = f"{p}hc{q}."
            y = sub(rms_norm(stream_read(X, w[hc + "in"]), w[f"{p}norm{q}"], eps))
            X = stream_write(X, w[hc + "mix"], w[hc + "out"], y)
        if taps is not None:
            taps.append(X.sum(0))
    logits = rms_norm(X.sum(0), w["final.norm"], eps) @ w["embed"].T
    cap = cfg.get("logit_softcap")
    return logits if not cap else cap * torch.tanh(logits / cap)


def greedy_generate(w, cfg, prompt, max_new_tokens):
    tokens = list(prompt)
    for _ in range(max_new_tokens):
        tokens.append(int(forward(w, cfg, tokens)[-1].argmax()))
    return tokens[len(prompt):]
