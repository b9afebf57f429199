"""A plain, slow statement of the Pinirax decoder: whole sequences, no cache, one function per mechanism.

Written from the design's equations and sharing no code with the product package: model folders are read with the
`safetensors` package, every tensor stays on the CPU, and every call recomputes the whole sequence in float64.

The design, in this file's notation.  x is the residual stream [T, W]; rms(z) = z / sqrt(mean(z^2) + eps).
  embedding   x_t = c * E[id_t] + P(t), P(t)[2i] = sin(t f_i), P(t)[2i+1] = cos(t f_i), f_i = 10000^(-2i/W)
  norm_g      rms(z) * (1 + g): gains are stored around zero
  layer       x <- x + norm_b1(mixer(norm_1(x)));  x <- x + norm_b2(ff(norm_2(x)))   (ff may be absent)
  parallel    left_scale * left(h) + right_scale * right(h)
    left      q = Wq h + bq, k = Wk h + bk, v = Wv h + bv; every head of q and of k: rms over its coordinates times a gain
              that the heads share; s_ij = cap * tanh(scale * q_i . k_j / cap); token i sees the tokens j with
              0 <= i - j < size; plain softmax; head h's sum times sigmoid(Wg h)_h; then Wo
    right     q, k, v = silu(conv(W h)), causal over time per channel; q and k unit vectors per head (x / sqrt(sum x^2 + 1e-6)),
              q times dim^-1/2; b = sigmoid(Wb h); a = exp(-exp(A) softplus(Wa h + dt)); per head, with S [dim, vdim]:
              S <- a S; u = b (v - S^T k); S <- S + k u^T; o = S^T q; then rms over vdim times a gain that the heads share,
              times silu(Wg h); then Wo
  mamba2      [z | x | B | C | d] = Win h; x, B, C through silu(conv + bias); d = softplus(d + dt); per head (its group's B, C):
              S <- exp(-exp(A) d) S + d B x^T; y = S^T C + D x; y silu(z), rms in equal parts of the row, times a gain; Wo
  ff          s = softmax(Wr h); the `top` largest s + correction are chosen; y = sum over the chosen of s_e expert_e(h);
              expert(h) = Wdown (silu(Wgate h) * (Wup h)), and the last `identity` experts give h itself
  output      logits = Whead norm_f(x)
"""
import json
import math
import os

import torch

F64 = torch.float64
UNIT_EPS = 1e-6
WAVE_BASE = 10000.0


def read_config(folder):
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)


def read_weights(folder, dtype=F64):
    from safetensors import safe_open
    tensors = {}
    with safe_open(os.path.join(folder, "model.safetensors"), framework="pt") as f:
        for name in f.keys():
            tensors[name] = f.get_tensor(name).to(dtype)
    return tensors


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def centered_norm(x, g, eps):
    return rms(x, eps) * (1.0 + g)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp(min=0.0)


def position_vectors(T, width, dtype=F64):
    out = torch.zeros((T, width), dtype=dtype)
    for t in range(T):
        for c in range(width):
            # the frequency is a 32-bit number, as the design computes angles in 32-bit
            f = float(torch.tensor(WAVE_BASE ** (-2.0 * (c // 2) / width), dtype=torch.float32))
            out[t, c] = math.sin(t * f) if c % 2 == 0 else math.cos(t * f)
    return out


def embed(cfg, w, ids):
    x = w["embed"][torch.tensor(ids, dtype=torch.long)]
    return x * cfg["embedding"]["scale"] + position_vectors(len(ids), x.shape[1], x.dtype)


def causal_convolution(x, taps_w, bias=None):
    """x [T, C], taps_w [C, taps] (the last column is the current token's), bias [C] or None."""
    T, taps = x.shape[0], taps_w.shape[1]
    out = torch.zeros_like(x)
    if bias is not None:
        out = out + bias
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            out[back:] += taps_w[:, j] * x[:T - back]
    return out


def capped_window_attention(q, k, v, scale, cap, window, positions=None):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]; window None: every earlier token; cap None: no cap."""
    T, H, _ = q.shape
    G = k.shape[1]
    pos = torch.arange(T) if positions is None else torch.as_tensor(positions, dtype=torch.long)
    back = pos[:, None] - pos[None, :]
    seen = back >= 0
    if window is not None:
        seen = seen & (back < window)
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        if cap is not None:
            s = cap * torch.tanh(s / cap)
        out[:, h] = torch.softmax(s.masked_fill(~seen, float("-inf")), dim=1) @ v[:, g]
    return out


def left_mixer(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, D)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, D)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(T, G, V)
    q = rms(q, eps) * w[p + "q.norm"]
    k = rms(k, eps) * w[p + "k.norm"]
    mask = m.get("mask")
    o = capped_window_attention(q, k, v, m["scale"], m.get("softcap"), mask["size"] if mask else None)
    o = o * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * V) @ w[p + "o"].T


def unit(x):
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + UNIT_EPS)


def gated_delta_rule(q, k, v, a, b, state=None):
    """q, k [T, H, D], v [T, H, V], a, b [T, H] -> (o [T, H, V], the state behind the last token)."""
    T, H, D = q.shape
    S = torch.zeros((H, D, v.shape[2]), dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros_like(v)
    for t in range(T):
        S = a[t][:, None, None] * S
        u = b[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(dim=1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(dim=1)
    return out, S


def right_mixer(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(causal_convolution(h @ w[p + "q"].T, w[p + "q.conv"])).reshape(T, G, D)
    k = silu(causal_convolution(h @ w[p + "k"].T, w[p + "k.conv"])).reshape(T, G, D)
    v = silu(causal_convolution(h @ w[p + "v"].T, w[p + "v.conv"])).reshape(T, H, V)
    of_head = [i // (H // G) for i in range(H)]
    q, k = (unit(q) * D ** -0.5)[:, of_head], unit(k)[:, of_head]
    b = torch.sigmoid(h @ w[p + "b"].T)
    a = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o, _ = gated_delta_rule(q, k, v, a, b)
    o = rms(o, eps) * w[p + "norm"] * silu(h @ w[p + "g"].T).reshape(T, H, V)
    return o.reshape(T, H * V) @ w[p + "o"].T


def parallel_mixer(h, w, p, m, eps):
    return (m["left_scale"] * left_mixer(h, w, p + "left.", m["left"], eps)
            + m["right_scale"] * right_mixer(h, w, p + "right.", m["right"], eps))


def state_space(x, B, C, d, a, D, state=None):
    """x [T, H, V], B, C [T, H, N] (each head's group's), d, a [T, H], D [H] -> (y [T, H, V], the last state [H, N, V])."""
    T, H, V = x.shape
    S = torch.zeros((H, B.shape[2], V), dtype=x.dtype) if state is None else state.clone()
    out = torch.zeros_like(x)
    for t in range(T):
        S = a[t][:, None, None] * S + (d[t][:, None] * B[t])[:, :, None] * x[t][:, None, :]
        out[t] = (S * C[t][:, :, None]).sum(dim=1) + D[:, None] * x[t]
    return out, S


def parts_norm(y, parts, g, eps):
    T, n = y.shape
    return rms(y.reshape(T, parts, n // parts), eps).reshape(T, n) * g


def mamba2_mixer(h, w, p, m, eps):
    T = h.shape[0]
    H, V, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * V
    u = h @ w[p + "in"].T
    z, xbc, d = u[:, :inner], u[:, inner:2 * inner + 2 * G * N], u[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_convolution(xbc, w[p + "conv"], w[p + "conv.b"]))
    of_head = [i // (H // G) for i in range(H)]
    x = xbc[:, :inner].reshape(T, H, V)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)[:, of_head]
    C = xbc[:, inner + G * N:].reshape(T, G, N)[:, of_head]
    d = softplus(d + w[p + "dt_bias"])
    y, _ = state_space(x, B, C, d, torch.exp(-torch.exp(w[p + "A_log"]) * d), w[p + "D"])
    y = parts_norm(y.reshape(T, inner) * silu(z), m["norm_groups"], w[p + "norm"], eps)
    return y @ w[p + "o"].T


def route(h, w, p, router):
    """-> (ids [T][top], weights [T][top])."""
    total = router["experts"] + router.get("identity", 0)
    s = torch.softmax(h @ w[p + "router"].T, dim=-1)
    assert s.shape[1] == total
    c = s + w[p + "correction"]
    ids = [sorted(range(total), key=lambda e: (-float(c[t, e]), e))[:router["top"]] for t in range(h.shape[0])]
    return ids, [[s[t, e] for e in chosen] for t, chosen in enumerate(ids)]


def expert(h, w, q):
    return w[q + "down"] @ (silu(w[q + "gate"] @ h) * (w[q + "up"] @ h))


def routed_feed_forward(h, w, p, mlp):
    ids, weights = route(h, w, p, mlp["router"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(ids[t], weights[t]):
            out[t] += s * (h[t] if e >= mlp["router"]["experts"] else expert(h[t], w, p + "e%d." % e))
    return out


def forward(cfg, w, ids, stream_after_layers=None):
    """Logits [T, vocab] of one whole sequence.  stream_after_layers: a list that receives the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = embed(cfg, w, ids)
    for i, layer in enumerate(cfg["layers"]):
        p, m = "l%d." % i, layer["mixer"]
        h = centered_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "parallel":
            y = parallel_mixer(h, w, p + "mix.", m, eps)
        elif layer["type"] == "mamba2":
            y = mamba2_mixer(h, w, p + "mix.", m, eps)
        else:
            raise ValueError("unknown mixer %r" % layer["type"])
        x = x + centered_norm(y, w[p + "norm1b"], eps)
        if layer.get("mlp") is not None:
            y = routed_feed_forward(centered_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"])
            x = x + centered_norm(y, w[p + "norm2b"], eps)
        if stream_after_layers is not None:
            stream_after_layers.append(x)
    return centered_norm(x, w["final.norm"], eps) @ w["head"].T
