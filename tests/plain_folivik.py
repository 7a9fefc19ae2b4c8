"""A plain, slow implementation of the Folivik decoder, written from its equations: one function per mechanism,
whole sequences at a time, float64 unless told otherwise.  It shares no code with the engine: it reads config.json
and model.safetensors itself (with the safetensors package), masks a full score matrix and walks the recurrent layer
token by token.

    x = E[tok];  per layer:  x += mixer(N(x; g1));  x += ff(N(x; g2));   logits = head N(x; g_f)
    N(v; g) = g v / rms(v) with ONE number g;   U(v; w) = v / rms(v) * w;   rms(v) = sqrt(mean(v^2) + eps)

    mixer "latent_attention":
        q = W_uq U(W_dq h; w_q), head by head [unrotated | rotated];   W_dkv h = [c' | r];   c = U(c'; w_c)
        rotated parts turned (pairs 2i, 2i + 1, angle p * base^(-2i / dims));  k_h = [W_uk,h c | r], v_h = W_uv,h c
        softmax over j <= i of scale * q . k;   head h's output times sigmoid(W_g h)_h;   W_o
    mixer "attention":
        q, k per head U(.; w);  no rotation;  score = q . k * scale * temp_h - r1_h ln(1 + r2_h (i - j)),
        softmax over 0 <= i - j < size;  W_o
    mixer "mamba2":
        [z | x | B | C | dt] = W_in h;   x, B, C = silu(conv(.) + b);   dt = softplus(dt + dt_bias)
        per head (B, C of its group):  S <- exp(-exp(A_log) dt) S + dt B x^T;   y = S^T C + D x
        W_o (w * groupwise U(y * silu(z)))
    ff: s = softmax(W_r h) over experts and identity experts;  c = s + correction;  groups of neighbours scored by their
        largest c, the best `keep` stay;  the `top` largest c among them;  weights s / (sum of the chosen s + 1e-20) * scale;
        expert: W_down (silu(W_gate h) * W_up h);  identity expert: h;  plus the shared expert, unweighted
"""
import json
import os

import torch
from safetensors import safe_open

WEIGHT_FLOOR = 1e-20  # added to the sum the chosen scores are divided by


# --------------------------------------------------------------------------------------------------- small pieces
def rms_divide(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.logaddexp(z, torch.zeros_like(z))


def turn_pairs(x, positions, rot):
    """x [T, heads, d]: element 2i turns with element 2i + 1, i below rot['dims'] / 2."""
    dims, base = rot["dims"], float(rot["base"])
    ang = torch.tensor([[p * base ** (-2.0 * i / dims) for i in range(dims // 2)] for p in positions], dtype=x.dtype)
    cos, sin = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    out = x.clone()
    a, b = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = a * cos - b * sin
    out[..., 1:dims:2] = b * cos + a * sin
    return out


def causal_conv(u, taps_weight, bias, before=None):
    """u [T, C]; taps_weight [C, K], the last column is the current token's.  ``before``: the K - 1 rows in front of
    the sequence (zeros if None)."""
    T, C = u.shape
    K = taps_weight.shape[1]
    if before is None:
        before = torch.zeros(K - 1, C, dtype=u.dtype)
    rows = torch.cat([before, u], dim=0)
    y = torch.zeros_like(u) + bias
    for j in range(K):
        y = y + taps_weight[:, j] * rows[j: j + T]
    return y


def masked_softmax(scores, positions, size=None):
    """scores [T, T] of one head; row i over 0 <= i - j (and i - j < size)."""
    p = torch.tensor(positions)
    d = p[:, None] - p[None, :]
    mask = (d >= 0) if size is None else (d >= 0) & (d < size)
    return torch.softmax(scores.masked_fill(~mask, float("-inf")), dim=-1)


# --------------------------------------------------------------------------------------------------- mixers
def latent_attention(h, w, p, m, eps, positions):
    T = h.shape[0]
    H, dn, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = rms_divide(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].T).reshape(T, H, dn + dr)
    q_n, q_r = q[..., :dn], turn_pairs(q[..., dn:], positions, m["rot"])
    down = h @ w[p + "dkv"].T
    c = rms_divide(down[:, :r], eps) * w[p + "dkv.norm"]
    k_r = turn_pairs(down[:, None, r:], positions, m["rot"])[:, 0]
    k_n = (c @ w[p + "uk"].T).reshape(T, H, dn)
    v = (c @ w[p + "uv"].T).reshape(T, H, dv)
    gate = torch.sigmoid(h @ w[p + "g"].T)  # [T, H]
    heads = []
    for hd in range(H):
        sc = (q_n[:, hd] @ k_n[:, hd].T + q_r[:, hd] @ k_r.T) * m["scale"]
        heads.append((masked_softmax(sc, positions) @ v[:, hd]) * gate[:, hd: hd + 1])
    return torch.cat(heads, dim=-1) @ w[p + "o"].T


def distance_penalty(distance, r1, r2):
    return r1 * torch.log(1.0 + r2 * distance)


def window_attention(h, w, p, m, eps, positions):
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_divide((h @ w[p + "q"].T).reshape(T, H, dk), eps) * w[p + "q.norm"]
    k = rms_divide((h @ w[p + "k"].T).reshape(T, G, dk), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T).reshape(T, G, dv)
    pos = torch.tensor(positions, dtype=h.dtype)
    distance = (pos[:, None] - pos[None, :]).clamp(min=0.0)
    heads = []
    for hd in range(H):
        g = hd // (H // G)
        sc = (q[:, hd] @ k[:, g].T) * m["scale"] * w[p + "temp"][hd]
        sc = sc - distance_penalty(distance, w[p + "r1"][hd], w[p + "r2"][hd])
        heads.append(masked_softmax(sc, positions, m["mask"]["size"]) @ v[:, g])
    return torch.cat(heads, dim=-1) @ w[p + "o"].T


def mamba2(h, w, p, m, eps, state=None):
    """Token by token.  ``state``: None (a sequence's start) or (S [H, N, P], the convolution's rows before).
    Returns the output and the state behind the last token."""
    T = h.shape[0]
    H, P, N, G, K = m["heads"], m["vdim"], m["state"], m["groups"], m["conv"]
    inner = H * P
    rows = h @ w[p + "in"].T
    z, u, dt = rows[:, :inner], rows[:, inner: 2 * inner + 2 * G * N], rows[:, 2 * inner + 2 * G * N:]
    before = torch.zeros(K - 1, u.shape[1], dtype=h.dtype) if state is None else state[1]
    y = silu(causal_conv(u, w[p + "conv"], w[p + "conv.b"], before))
    x = y[:, :inner].reshape(T, H, P)
    B = y[:, inner: inner + G * N].reshape(T, G, N)
    C = y[:, inner + G * N:].reshape(T, G, N)
    dt = softplus(dt + w[p + "dt_bias"])
    decay = torch.exp(-torch.exp(w[p + "A_log"]) * dt)
    S = torch.zeros(H, N, P, dtype=h.dtype) if state is None else state[0].clone()
    group = torch.tensor([hd // (H // G) for hd in range(H)])
    out = torch.zeros(T, H, P, dtype=h.dtype)
    for t in range(T):
        S = decay[t][:, None, None] * S + (dt[t][:, None] * B[t, group])[:, :, None] * x[t][:, None, :]
        out[t] = torch.einsum("hnp,hn->hp", S, C[t, group]) + w[p + "D"][:, None] * x[t]
    y = out.reshape(T, inner) * silu(z)
    parts = m["norm_groups"]
    y = rms_divide(y.reshape(T, parts, inner // parts), eps).reshape(T, inner) * w[p + "norm"]
    tail = torch.cat([before, u])[u.shape[0]:]
    return y @ w[p + "o"].T, (S, tail)


# --------------------------------------------------------------------------------------------------- feed-forward
def choose_experts(z, correction, router):
    """z [E + identity] logits of one token -> (chosen expert ids, their weights)."""
    E, top = z.shape[0], router["top"]
    s = torch.softmax(z, dim=-1)
    c = s + correction
    groups = router.get("groups")
    allowed = [True] * E
    if groups is not None:
        n, per = groups["count"], E // groups["count"]
        score = [max(float(c[e]) for e in range(gi * per, (gi + 1) * per)) for gi in range(n)]
        kept = sorted(range(n), key=lambda gi: (-score[gi], gi))[: groups["keep"]]
        allowed = [(e // per) in kept for e in range(E)]
    order = sorted((e for e in range(E) if allowed[e]), key=lambda e: (-float(c[e]), e))[:top]
    return order, weigh(s, order, router)


def weigh(s, chosen, router):
    total = sum(s[e] for e in chosen) + WEIGHT_FLOOR
    return [s[e] / total * router.get("scale", 1.0) for e in chosen]


def gated_expert(h, w, p):
    return w[p + "down"] @ (silu(w[p + "gate"] @ h) * (w[p + "up"] @ h))


def routed_experts(h, w, p, mlp, choices=None):
    T = h.shape[0]
    router = mlp["router"]
    z = h @ w[p + "router"].T
    out = torch.zeros_like(h)
    picked = []
    for t in range(T):
        ids, weights = choose_experts(z[t], w[p + "correction"], router)
        if choices is not None:  # (the caller's choice; the weights are still this token's own scores)
            ids = [int(e) for e in choices[t]]
            weights = weigh(torch.softmax(z[t], dim=-1), ids, router)
        picked.append(ids)
        for e, g in zip(ids, weights):
            out[t] = out[t] + g * (gated_expert(h[t], w, p + f"e{e}.") if e < router["experts"] else h[t])
        if mlp.get("shared") is not None:
            out[t] = out[t] + gated_expert(h[t], w, p + "shared.")
    return out, picked


# --------------------------------------------------------------------------------------------------- the model
def mix(h, w, p, layer, eps, positions):
    m = layer["mixer"]
    if layer["type"] == "latent_attention":
        return latent_attention(h, w, p, m, eps, positions)
    if layer["type"] == "attention":
        return window_attention(h, w, p, m, eps, positions)
    if layer["type"] == "mamba2":
        return mamba2(h, w, p, m, eps)[0]
    raise ValueError(layer["type"])


def forward(cfg, w, tokens, dtype=torch.float64, taps=None, choices=None):
    """Logits [T, vocab] of one whole sequence.  ``taps``: a list that receives the stream behind every layer.
    ``choices``: per layer a [T, top] table of expert ids to use instead of the model's own choice."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    positions = list(range(len(tokens)))
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    chosen = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + mix(rms_divide(x, eps) * w[p + "norm1"], w, p + "mix.", layer, eps, positions)
        ids = None
        if layer.get("mlp") is not None:
            y, ids = routed_experts(rms_divide(x, eps) * w[p + "norm2"], w, p + "mlp.", layer["mlp"],
                                    None if choices is None else choices[i])
            x = x + y
        chosen.append(ids)
        if taps is not None:
            taps.append(x.clone())
    return (rms_divide(x, eps) * w["final.norm"]) @ w["head"].T, chosen


def load(folder):
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    w = {}
    with safe_open(os.path.join(folder, "model.safetensors"), framework="pt") as f:
        for name in f.keys():
            w[name] = f.get_tensor(name)
    return cfg, w
