"""A plain, slow implementation of the Rasodra decoder, one function per mechanism.

Whole sequences, float32 (or a low dtype for products and their activations), no cache, no batching, every recurrence a
Python loop over the tokens.  It shares no code with the library; the GPU tests compare the library with it.

Notation: T tokens, D the model's width.

    x        = E[t]
    sublayer:  x' = x + N_b(part(N_a(x))) with two norms of its own, around the mixer and then around the feed-forward
               (which may be absent)
    N(u)     = (u - mean u) / sqrt(mean (u - mean u)^2 + eps) w
    a layer may name an earlier layer whose tensors it uses; what it remembers of a sequence is its own
    logits   = H N_final(x)

Mixers:

    matrix memory   q = W_q h / sqrt(d), k = W_k h, v = W_v h per head; logarithms of the gates, per head and token,
               a = c tanh((w_i h + b_i) / c) and f = log sigmoid(c tanh((w_f h + b_f) / c)); a running maximum
               m_t = max(f_t + m_(t-1), a_t) from m = 0;
               S_t = e^(f_t + m_(t-1) - m_t) S_(t-1) + e^(a_t - m_t) k_t v_t^T,   n_t the same with k_t alone;
               o_t = S_t^T q_t / (max(|n_t . q_t|, e^(-m_t)) + 1e-6);
               o is divided per head by its root mean square, times a weight over all heads' elements, times sigmoid(W_g h), W_o
    latent attention   per head q = (q_c, q_r) from W_q h; W_d h = (c', r): c = c' / rms(c') w the latent, r one rotated key part
               for all heads; score = (q_c . W_uk c + turn(q_r) . turn(r)) s over all earlier positions; the softmax's denominator
               also holds exp(sink_h); the value is W_uv c; the heads' outputs are multiplied by sigmoid(W_g h) element by element, W_o
    chunked attention   q = W_q h + b_q, k = W_k h + b_k, v = k; q and k heads are divided by their root mean square and
               multiplied by a weight, then turned; position i sees the positions j <= i with floor(j / C) = floor(i / C)

Turning is by neighbouring pairs: (e_2i, e_2i+1) by p base^(-2i/r) over the first r elements.  The feed-forward is
W_down max(W_up h, 0)^2.

A weight dict maps the checkpoint's tensor names to float32 tensors (the bfloat16 values exactly).  `low` names the dtype
the products are rounded to (float32: nothing is).
"""
import math

import torch

F32 = torch.float32


def rnd(x, low):
    return x if low == F32 else x.to(low).to(x.dtype)


def product(x, w, low):
    return rnd(rnd(x, low) @ w.to(x.dtype).T, low)


def layer_norm(u, w, eps):
    d = u - u.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def unit_norm(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def angles(positions, base, dims):
    """[T, dims / 2]: position * base^(-2i/dims)"""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / dims)
    return positions.to(torch.float64)[:, None] * f[None, :]


def turn_pairs(v, ang):
    """v [T, heads, d]; elements 2i and 2i + 1 of each head, i < ang.shape[1], are turned by ang [T, n]."""
    n = ang.shape[1]
    if n == 0:
        return v
    c, s = torch.cos(ang).to(v.dtype)[:, None, :], torch.sin(ang).to(v.dtype)[:, None, :]
    out = v.clone()
    a, b = v[..., 0:2 * n:2], v[..., 1:2 * n:2]
    out[..., 0:2 * n:2] = a * c - b * s
    out[..., 1:2 * n:2] = b * c + a * s
    return out


def softmax_of(scores, sink=None):
    """scores [keys], sink a number or None -> the keys' weights (the sink's is left out)."""
    top = scores.max() if sink is None else torch.maximum(scores.max(), sink)
    e = torch.exp(scores - top)
    return e / (e.sum() + (0.0 if sink is None else torch.exp(sink - top)))


# ---- matrix memory ------------------------------------------------------------------------------------
def gate_logarithms(zi, zf, cap):
    """the logarithms of the input gate and of the forget gate from their products (biases added)"""
    capped = lambda z: cap * torch.tanh(z / cap)
    return capped(zi), torch.nn.functional.logsigmoid(capped(zf))


def matrix_memory(q, k, v, a, f, S=None, n=None, m=None):
    """q, k [T, H, d], v [T, H, dv], a, f [T, H] -> ([T, H, dv], the state after the last token)."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype) if S is None else S
    n = torch.zeros(H, d, dtype=q.dtype) if n is None else n
    m = torch.zeros(H, dtype=q.dtype) if m is None else m
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        m_new = torch.maximum(f[t] + m, a[t])
        keep, take = torch.exp(f[t] + m - m_new), torch.exp(a[t] - m_new)
        S = keep[:, None, None] * S + take[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + take[:, None] * k[t]
        m = m_new
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = (S * q[t][:, :, None]).sum(1) / den[:, None]
    return out, (S, n, m)


def mlstm(h, w, p, mix, eps, positions, low):
    T = h.shape[0]
    H, d, dv = mix["heads"], mix["dim"], mix["vdim"]
    q = product(h, w[p + "q"], low).view(T, H, d) * d ** -0.5
    k = product(h, w[p + "k"], low).view(T, H, d)
    v = product(h, w[p + "v"], low).view(T, H, dv)
    hl = rnd(h, low)
    a, f = gate_logarithms(hl @ w[p + "i"].to(h.dtype).T + w[p + "i.b"], hl @ w[p + "f"].to(h.dtype).T + w[p + "f.b"], mix["gate_cap"])
    o, _ = matrix_memory(q, k, v, a, f)
    o = unit_norm(o, eps).reshape(T, H * dv) * w[p + "norm"] * torch.sigmoid(product(h, w[p + "g"], low))
    return product(o, w[p + "o"], low)


# ---- latent attention -----------------------------------------------------------------------------------
def latent_attention(h, w, p, mix, eps, positions, low):
    T = h.shape[0]
    H, dn, dr, dv, rk = mix["heads"], mix["dim"], mix["rot_dim"], mix["vdim"], mix["kv_rank"]
    q = product(h, w[p + "q"], low).view(T, H, dn + dr)
    down = product(h, w[p + "dkv"], low)
    c = rnd(unit_norm(down[:, :rk], eps) * w[p + "dkv.norm"], low)
    ang = angles(positions, mix["rot"]["base"], mix["rot"]["dims"])
    r = rnd(turn_pairs(down[:, None, rk:], ang)[:, 0], low)
    qr = turn_pairs(q[:, :, dn:], ang)
    k = product(c, w[p + "uk"], low).view(T, H, dn)
    v = product(c, w[p + "uv"], low).view(T, H, dv)
    o = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(T):
        for g in range(H):
            s = (k[:i + 1, g] @ q[i, g, :dn] + r[:i + 1] @ qr[i, g]) * mix["scale"]
            o[i, g] = softmax_of(s, w[p + "sink"][g]) @ v[:i + 1, g]
    o = o.reshape(T, H * dv) * torch.sigmoid(product(h, w[p + "g"], low))
    return product(o, w[p + "o"], low)


# ---- chunked attention -------------------------------------------------------------------------------------
def visible(i, size):
    """the first position that position i sees when positions fall into chunks of `size`"""
    return i // size * size


def chunked_attention(h, w, p, mix, eps, positions, low):
    T = h.shape[0]
    H, G, d = mix["heads"], mix["kv_heads"], mix["dim"]
    q = (product(h, w[p + "q"], low) + w[p + "q.b"]).view(T, H, d)
    k = (product(h, w[p + "k"], low) + w[p + "k.b"]).view(T, G, d)
    v = rnd(k, low)
    ang = angles(positions, mix["rot"]["base"], mix["rot"]["dims"])
    q = rnd(turn_pairs(unit_norm(q, eps) * w[p + "q.norm"], ang), low)
    k = rnd(turn_pairs(unit_norm(k, eps) * w[p + "k.norm"], ang), low)
    o = torch.zeros(T, H, d, dtype=h.dtype)
    for i in range(T):
        lo = visible(i, mix["mask"]["size"])
        for g in range(H):
            kv = g // (H // G)
            o[i, g] = softmax_of((k[lo:i + 1, kv] @ q[i, g]) * mix["scale"]) @ v[lo:i + 1, kv]
    return product(o.reshape(T, H * d), w[p + "o"], low)


MIXERS = {"mlstm": mlstm, "latent_attention": latent_attention, "attention": chunked_attention}


# ---- feed-forward and the whole -------------------------------------------------------------------------------
def feed_forward(h, w, p, low):
    return product(rnd(torch.clamp(product(h, w[p + "up"], low), min=0.0) ** 2, low), w[p + "down"], low)


def source_of(layers, i):
    """the layer whose tensors layer i uses"""
    while layers[i].get("weights_of") is not None:
        i = layers[i]["weights_of"]
    return i


def forward(cfg, w, tokens, low=F32, every_layer=None):
    """Logits [T, vocab] of one sequence.  every_layer: a list that gets the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)]
    positions = torch.arange(len(tokens))
    for i, layer in enumerate(cfg["layers"]):
        p = "l%d." % source_of(cfg["layers"], i)
        y = MIXERS[layer["type"]](layer_norm(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps, positions, low)
        x = x + layer_norm(y, w[p + "norm1b"], eps)
        if layer["mlp"] is not None:
            y = feed_forward(layer_norm(x, w[p + "norm2"], eps), w, p + "mlp.", low)
            x = x + layer_norm(y, w[p + "norm2b"], eps)
        if every_layer is not None:
            every_layer.append(x.clone())
    return product(layer_norm(x, w["final.norm"], eps), w["head"], F32)


def greedy(cfg, w, prompt, n, low=F32):
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(torch.argmax(forward(cfg, w, tokens, low)[-1])))
    return tokens[len(prompt):]
