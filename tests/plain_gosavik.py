"""The Gosavik decoder written out plainly: float64, whole sequences, one function per mechanism.

Nothing here is shared with the engine: no cache, no pages, no state slots, no kernels. A sequence goes in as a list of
token ids, logits for every position come out (and, if asked, the summed stream after every layer run). Tests compare
the engine with this.

The design: S streams X_1 .. X_S, all E[token] at the start. A sublayer reads u = sum_s a_s X_s through an RMS norm and
gives y; then X_t <- sum_s M[s, t] X_s + b_t y. What a mixer reads is moved towards the row before it, channel by channel.
A layer's mixer is attention over a low-rank latent inside a window (queries through a latent of their own, rotation with
slowed long waves, a learned sink per head, a gate per channel) or grouped-query attention (biases, a short convolution
on queries, keys and values, rotation of keys and of values, a learned sink); its feed-forward is Wd gelu(Wu h). A run of
layers may be passed several times. logits = head norm(sum_s X_s).
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms_norm(x, gain, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * gain


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ---- several streams instead of one -------------------------------------------------------------------------------------

def read_streams(X, weights):
    """X [S, T, width], weights [S]: the one row per position that a sublayer sees."""
    return torch.einsum("s,stw->tw", weights, X)


def write_streams(X, mix, out, y):
    """Every new stream from all the old ones: X_t <- sum_s mix[s, t] X_s + out[t] y."""
    return torch.einsum("st,slw->tlw", mix, X) + out.view(-1, 1, 1) * y


def token_shift(h, amount):
    """Row t becomes h_t + (h_(t-1) - h_t) * amount, with nothing (zeros) before the first row."""
    before = torch.cat((torch.zeros_like(h[:1]), h[:-1]))
    return h + (before - h) * amount


def run_order(n_layers, loop):
    """The layers' indices in the order they run."""
    if not loop:
        return list(range(n_layers))
    start, stop, times = loop["start"], loop["stop"], loop["times"]
    return list(range(start)) + list(range(start, stop)) * times + list(range(stop, n_layers))


# ---- rotation ---------------------------------------------------------------------------------------------------------

def frequencies(dims, base):
    return float(base) ** (-2.0 * torch.arange(dims // 2, dtype=F64) / dims)


def slowed(dims, base, scaling):
    """(frequencies, factor on cosine and sine) with long waves slowed: pair i turns at f_i up to pair `lo`, at f_i /
    factor from pair `hi` on, and is blended linearly between the two; lo and hi are the (whole) pairs that turn `fast`
    and `slow` times within `original` positions."""
    f = frequencies(dims, base)
    factor, orig = float(scaling["factor"]), float(scaling["original"])

    def pair_of(turns):
        return dims * math.log(orig / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_of(float(scaling["fast"]))), 0)
    hi = min(math.ceil(pair_of(float(scaling["slow"]))), dims - 1)
    out = f.clone()
    for i in range(f.numel()):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out[i] = f[i] / factor * r + f[i] * (1.0 - r)
    return out, 0.1 * math.log(factor) + 1.0


def rotate_half(x, positions, dims, freqs, factor=1.0):
    """x [T, heads, D]: channel i < dims/2 turns with channel i + dims/2; channels from dims on stay."""
    half = dims // 2
    ang = positions.to(F64).view(-1, 1, 1) * freqs
    c, s = torch.cos(ang) * factor, torch.sin(ang) * factor
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat((u * c - v * s, v * c + u * s, x[..., dims:]), dim=-1)


def rotate_pairs(x, positions, dims, freqs, factor=1.0):
    """x [T, heads, D]: channel 2i turns with channel 2i + 1 for 2i < dims; channels from dims on stay."""
    ang = positions.to(F64).view(-1, 1, 1) * freqs
    c, s = torch.cos(ang) * factor, torch.sin(ang) * factor
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    y = torch.stack((u * c - v * s, v * c + u * s), dim=-1).flatten(-2)
    return torch.cat((y, x[..., dims:]), dim=-1)


# ---- attention --------------------------------------------------------------------------------------------------------

def seen_mask(T, window):
    """[T, T] booleans: row i sees column j if 0 <= i - j, and i - j < window where there is one (0: none)."""
    d = torch.arange(T).view(-1, 1) - torch.arange(T).view(1, -1)
    return (d >= 0) & (d < window) if window else d >= 0


def sink_softmax(scores, sink):
    """scores [H, T, T] (-inf where not seen), sink [H]: exp(s_ij) / (exp(sink_h) + sum_j exp(s_ij))."""
    full = torch.cat((scores, sink.view(-1, 1, 1).expand(scores.shape[0], scores.shape[1], 1)), dim=-1)
    return torch.softmax(full, dim=-1)[..., :-1]


def causal_conv(x, taps):
    """x [T, C], taps [C, K]: y_t = sum_d taps[:, K-1-d] * x_(t-d), nothing before the first row."""
    T, K = x.shape[0], taps.shape[1]
    y = torch.zeros_like(x)
    for d in range(min(K, T)):
        y[d:] += x[:T - d] * taps[:, K - 1 - d]
    return y


def latent_attention(h, w, pre, m, eps, positions):
    T = h.shape[0]
    H, D, R, V, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = rms_norm(h @ w[pre + "dq"].t(), w[pre + "dq.norm"], eps)
    q = (cq @ w[pre + "uq"].t()).view(T, H, D + R)
    ckv = h @ w[pre + "dkv"].t()
    c = rms_norm(ckv[:, :C], w[pre + "dkv.norm"], eps)
    k_rot = ckv[:, C:].view(T, 1, R)
    q_plain, q_rot = q[..., :D], q[..., D:]
    rot = m.get("rot") or {}
    if rot.get("dims"):
        dims = rot["dims"]
        f, factor = slowed(dims, rot["base"], rot["scaling"]) if rot.get("scaling") else (frequencies(dims, rot["base"]), 1.0)
        q_rot, k_rot = rotate_half(q_rot, positions, dims, f, factor), rotate_half(k_rot, positions, dims, f, factor)
    k_plain = (c @ w[pre + "uk"].t()).view(T, H, D)
    v = (c @ w[pre + "uv"].t()).view(T, H, V)
    s = (torch.einsum("ihd,jhd->hij", q_plain, k_plain) + torch.einsum("ihr,jr->hij", q_rot, k_rot[:, 0])) * float(m["scale"])
    s = s.masked_fill(~seen_mask(T, int((m.get("mask") or {}).get("size", 0))), -math.inf)
    o = torch.einsum("hij,jhv->ihv", sink_softmax(s, w[pre + "sink"]), v).reshape(T, H * V)
    return (o * torch.sigmoid(h @ w[pre + "g"].t())) @ w[pre + "o"].t()


def attention(h, w, pre, m, positions):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (causal_conv(h @ w[pre + n].t() + w[pre + n + ".b"], w[pre + n + ".conv"]) for n in ("q", "k", "v"))
    q, k, v = q.view(T, H, D), k.view(T, G, D), v.view(T, G, V)
    rot = m.get("rot") or {}
    base = float(rot.get("base", 1.0))
    if rot.get("dims"):
        f = frequencies(rot["dims"], base)
        q, k = rotate_pairs(q, positions, rot["dims"], f), rotate_pairs(k, positions, rot["dims"], f)
    fv = frequencies(V, base)
    v = rotate_pairs(v, positions, V, fv)
    k, v = k.repeat_interleave(H // G, dim=1), v.repeat_interleave(H // G, dim=1)
    s = torch.einsum("ihd,jhd->hij", q, k) * float(m["scale"])
    s = s.masked_fill(~seen_mask(T, 0), -math.inf)
    o = torch.einsum("hij,jhv->ihv", sink_softmax(s, w[pre + "sink"]), v)
    o = rotate_pairs(o, -positions, V, fv).reshape(T, H * V)
    return o @ w[pre + "o"].t() + w[pre + "o.b"]


def dense_ff(h, w, pre):
    return gelu_tanh(h @ w[pre + "up"].t()) @ w[pre + "down"].t()


# ---- the model --------------------------------------------------------------------------------------------------------

def layer(X, w, i, entry, eps, positions):
    p = f"l{i}."
    h = rms_norm(read_streams(X, w[p + "hc1.in"]), w[p + "norm1"], eps)
    h = token_shift(h, w[p + "shift"])
    if entry["type"] == "latent_attention":
        y = latent_attention(h, w, p + "mix.", entry["mixer"], eps, positions)
    else:
        y = attention(h, w, p + "mix.", entry["mixer"], positions)
    X = write_streams(X, w[p + "hc1.mix"], w[p + "hc1.out"], y)
    if entry.get("mlp") is not None:
        h = rms_norm(read_streams(X, w[p + "hc2.in"]), w[p + "norm2"], eps)
        X = write_streams(X, w[p + "hc2.mix"], w[p + "hc2.out"], dense_ff(h, w, p + "mlp."))
    return X


def forward(cfg, w, ids, layers_out=None):
    """logits [T, vocab] in float64. w: {tensor name: float64 tensor}. layers_out: a list that receives the sum of the
    streams after every layer run."""
    eps = float(cfg["norm"]["eps"])
    positions = torch.arange(len(ids))
    X = w["embed"][torch.tensor(list(ids), dtype=torch.long)].expand(cfg["streams"], -1, -1)
    for i in run_order(len(cfg["layers"]), cfg.get("loop")):
        X = layer(X, w, i, cfg["layers"][i], eps, positions)
        if layers_out is not None:
            layers_out.append(X.sum(0))
    return rms_norm(X.sum(0), w["final.norm"], eps) @ w["head"].t()


def greedy_generate(cfg, w, prompt, n_new):
    """The n_new tokens that follow `prompt` when the largest logit is taken every time (the whole sequence is run again
    for every token: plain, not fast)."""
    ids = list(prompt)
    for _ in range(n_new):
        ids.append(int(torch.argmax(forward(cfg, w, ids)[-1])))
    return ids[len(prompt):]
