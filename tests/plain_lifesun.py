"""A plain, slow implementation of the Lifesun decoder, written from its equations: one function per mechanism,
whole sequences at a time, float64 unless told otherwise.  It shares no code with the engine: it reads config.json
and model.safetensors itself (with the safetensors package), masks a full score matrix and walks the recurrent layers
token by token.

    x0 = E[tok];  x = x0;  layers in order, a looped stretch several times in a row: in front of every pass
    x <- W [x; x0];  per layer  h = L(x);  x += mixer(h) + ff(h);  logits = scale * head L(x)
    L(v) = (v - mean) / sqrt(mean((v - mean)^2) + eps) * w + b;   rms(v) = sqrt(mean(v^2) + eps)

    both mixers: a * left(h) + b * right(h)
    mixer "parallel"
        left: q, k per head v / rms(v); softmax with one more 1 in the denominator over the keys of the query's chunk,
              every head's output times sigmoid(W_g h)_head, W_o
        right: y = gelu(W_y h + b_y);  u = conv(W_x h + b_x) + b_c;  per block  r = sigmoid(A u + a), i = sigmoid(B u + b)
               log a_t = -8 r softplus(lam);  S <- a S + sqrt(1 - a^2) i u;  W_o (S y)
    mixer "parallel_2"
        left: q, k over the whole projection v / rms(v) * w, the leading elements of every head turned (pairs i,
              i + dims/2);  score = cap tanh(q . k * scale / cap), softmax over a sliding window, W_o
        right: q, k turned the same way, k / sqrt(dim);  S <- decay S + k v^T;  o = S^T q;
               W_o (o / rms(o) * silu(W_g h))
    ff: W_d (gelu(W_g h) * (W_u h))
"""
import json
import math
import os

import torch
from safetensors import safe_open


# --------------------------------------------------------------------------------------------------- small pieces
def rms_divide(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def layer_norm(x, weight, bias, eps):
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * weight + bias


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(u, taps_weight, bias, before=None):
    """u [T, C]; taps_weight [C, K], the last column is the current token's.  ``before``: the K - 1 rows in front of
    the sequence (zeros if None)."""
    T, C = u.shape
    K = taps_weight.shape[1]
    if before is None:
        before = torch.zeros(K - 1, C, dtype=u.dtype)
    rows = torch.cat([before, u], dim=0)
    y = bias.expand(T, C).clone()
    for j in range(K):
        y = y + taps_weight[:, j] * rows[j: j + T]
    return y, rows[T:]


def turn(x, positions, rot):
    """x [T, heads, d]; element i of the leading rot['dims'] pairs up with element i + dims/2."""
    dims, half = rot["dims"], rot["dims"] // 2
    ang = torch.tensor([[p * rot["base"] ** (-2.0 * i / dims) for i in range(half)] for p in positions], dtype=x.dtype)
    cos, sin = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def same_chunk(i, j, size):
    return j <= i and (size is None or i // size == j // size)


def in_window(i, j, size):
    return j <= i and (size is None or i - j < size)


def visible(positions, rule, size):
    return torch.tensor([[rule(i, j, size) for j in positions] for i in positions])


def sink_softmax(scores, mask):
    """One more 1 in the denominator: a score of zero that has no value."""
    s = scores.masked_fill(~mask, float("-inf"))
    top = s.max(dim=-1, keepdim=True).values.clamp_min(0.0)
    e = torch.exp(s - top)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(-top))


# --------------------------------------------------------------------------------------------------- the four mixers
def gated_chunk_attention(h, w, p, m, eps, positions):
    T = h.shape[0]
    H, G = m["heads"], m["kv_heads"]
    q = rms_divide((h @ w[p + "q"].T).reshape(T, H, m["dim"]), eps)
    k = rms_divide((h @ w[p + "k"].T).reshape(T, G, m["dim"]), eps)
    v = (h @ w[p + "v"].T).reshape(T, G, m["vdim"])
    gate = torch.sigmoid(h @ w[p + "g"].T)  # [T, H]
    mask = visible(positions, same_chunk, m["mask"]["size"] if m.get("mask") else None)
    heads = []
    for hd in range(H):
        g = hd // (H // G)
        a = sink_softmax((q[:, hd] @ k[:, g].T) * m["scale"], mask)
        heads.append((a @ v[:, g]) * gate[:, hd: hd + 1])
    return torch.cat(heads, dim=-1) @ w[p + "o"].T


def capped_window_attention(h, w, p, m, eps, positions):
    T = h.shape[0]
    H, G, cap = m["heads"], m["kv_heads"], m["softcap"]
    q = (rms_divide(h @ w[p + "q"].T, eps) * w[p + "q.norm"]).reshape(T, H, m["dim"])
    k = (rms_divide(h @ w[p + "k"].T, eps) * w[p + "k.norm"]).reshape(T, G, m["dim"])
    v = (h @ w[p + "v"].T).reshape(T, G, m["vdim"])
    q, k = turn(q, positions, m["rot"]), turn(k, positions, m["rot"])
    mask = visible(positions, in_window, m["mask"]["size"] if m.get("mask") else None)
    heads = []
    for hd in range(H):
        g = hd // (H // G)
        s = cap * torch.tanh((q[:, hd] @ k[:, g].T) * m["scale"] / cap)
        heads.append(torch.softmax(s.masked_fill(~mask, float("-inf")), dim=-1) @ v[:, g])
    return torch.cat(heads, dim=-1) @ w[p + "o"].T


def gated_unit(h, w, p, m, state=None):
    """Token by token.  ``state``: None (a sequence's start) or (S [width], the convolution's rows before)."""
    T, blocks = h.shape[0], m["blocks"]
    W = m["width"]
    y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
    u, tail = causal_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"], w[p + "conv.b"],
                          None if state is None else state[1])
    ub = u.reshape(T, blocks, W // blocks)
    r = torch.stack([torch.sigmoid(ub[:, b] @ w[p + "ra"][b].T + w[p + "ra.b"][b]) for b in range(blocks)], 1).reshape(T, W)
    i = torch.stack([torch.sigmoid(ub[:, b] @ w[p + "ri"][b].T + w[p + "ri.b"][b]) for b in range(blocks)], 1).reshape(T, W)
    log_a = -8.0 * r * torch.nn.functional.softplus(w[p + "lam"])
    a = torch.exp(log_a)
    take = torch.sqrt(-torch.expm1(2.0 * log_a)) * i * u
    S = torch.zeros(W, dtype=h.dtype) if state is None else state[0].clone()
    out = torch.zeros_like(u)
    for t in range(T):
        S = a[t] * S + take[t]
        out[t] = S
    return (out * y) @ w[p + "o"].T, (S, tail)


def retention(h, w, p, m, eps, positions, state=None):
    """Token by token.  ``state``: None (a sequence's start) or S [heads, dim, vdim]."""
    T = h.shape[0]
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    q = turn((h @ w[p + "q"].T).reshape(T, H, dk), positions, m["rot"])
    k = turn((h @ w[p + "k"].T).reshape(T, H, dk), positions, m["rot"]) * dk ** -0.5
    v = (h @ w[p + "v"].T).reshape(T, H, dv)
    S = torch.zeros(H, dk, dv, dtype=h.dtype) if state is None else state.clone()
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for t in range(T):
        for hd in range(H):
            S[hd] = m["decay"][hd] * S[hd] + torch.outer(k[t, hd], v[t, hd])
            out[t, hd] = S[hd].T @ q[t, hd]
    o = rms_divide(out, eps).reshape(T, H * dv) * silu(h @ w[p + "g"].T)
    return o @ w[p + "o"].T, S


def mixer(kind, h, w, p, m, eps, positions):
    if kind == "parallel":
        left = gated_chunk_attention(h, w, p + "left.", m["left"], eps, positions)
        right, _ = gated_unit(h, w, p + "right.", m["right"])
    elif kind == "parallel_2":
        left = capped_window_attention(h, w, p + "left.", m["left"], eps, positions)
        right, _ = retention(h, w, p + "right.", m["right"], eps, positions)
    else:
        raise ValueError(kind)
    return m["left_scale"] * left + m["right_scale"] * right


def dense(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


# --------------------------------------------------------------------------------------------------- the model
def run_order(cfg):
    """(layer, begins a pass) in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if loop is None:
        return [(i, False) for i in range(n)]
    order = [(i, False) for i in range(loop["start"])]
    for _ in range(loop["times"]):
        order += [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return order + [(i, False) for i in range(loop["stop"], n)]


def forward(cfg, w, tokens, dtype=torch.float64, taps=None):
    """Logits [T, vocab] of one whole sequence.  ``taps``: a list that receives the stream behind every layer run."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    positions = list(range(len(tokens)))
    x0 = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    x = x0
    for i, begins in run_order(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        if begins:
            x = torch.cat([x, x0], dim=-1) @ w["loop.in"].T
        h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps)
        y = mixer(layer["type"], h, w, p + "mix.", layer["mixer"], eps, positions)
        if layer.get("mlp") is not None:
            y = y + dense(h, w, p + "mlp.")
        x = x + y
        if taps is not None:
            taps.append(x.clone())
    return layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["head"].T * cfg["logit_scale"]


def load(folder):
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    w = {}
    with safe_open(os.path.join(folder, "model.safetensors"), framework="pt") as f:
        for name in f.keys():
            w[name] = f.get_tensor(name)
    return cfg, w
