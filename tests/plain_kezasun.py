"""A plain, slow implementation of the Kezasun decoder, one function per mechanism.

Whole sequences, float32 (or a low dtype for products and their activations), no cache, no batching, every recurrence a
Python loop over the tokens.  It shares no code with the library; the GPU tests compare the library with it.

Notation: T tokens, D the model's width, m the layer's share of what it computes.

    x        = E[t]
    layer:     x' = x + m (mixer(h) + ff(h)),  h = N(x): one norm, read by both (there may be no feed-forward)
    N(u)     = u / sqrt(mean u^2 + eps) (1 + w)
    logits   = H N_final(x)

Mixers:

    time mixing   h^-_t = h_(t-1) (0 where there is none); the input of r is h + (h^- - h) mu_r, and so for k, v, g and w.
               r = W_r ., k = W_k ., v = W_v . per head; a_t = exp(-exp(A_2 tanh(A_1 .) + b)) per head and key channel;
               o_t = S_(t-1)^T r_t + (sum_i u_i k_i r_i) v_t,  S_t = diag(a_t) S_(t-1) + k_t v_t^T from S = 0;
               o is divided per head by its root mean square, times a weight over all heads' elements, times silu(W_g .), W_o
    attention  q = W_q h + b_q, k = W_k h + b_k, v = W_v h + b_v; all of q at once, and all of k at once, are divided by their root mean
               square and multiplied by a weight; then the heads are turned.  Position i sees positions i - M < j <= i; the softmax's
               denominator has one more 1; o_n <- o_n sigmoid(W_g h)_n for head n, then W_o.  A layer may read the keys and
               values of an earlier layer instead of its own.

Turning is in halves: (e_i, e_(i+r/2)) by p f_i with f_i = base^(-2i/r), and f scaled by its wavelength l = 2 pi / f: kept where
l < L / high, divided by F where l > L / low, between the two blended by s = (L / l - low) / (high - low).

Experts: z = R h over the experts with weights and, after them, those that give back their input; s = softmax z; chosen are the `top` with
the largest s + c among the groups kept, a group's rank being its largest s + c; weights are the chosen s over their sum.

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


def silu(z):
    return z * torch.sigmoid(z)


def unit_norm(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x, w, eps):
    return unit_norm(x, eps) * (1.0 + w)


# ---- time mixing ------------------------------------------------------------------------------------------
def shifted(h):
    """row t holds row t - 1, the first row zeros"""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]])


def mixed(h, before, mu):
    return h + (before - h) * mu


def decay(z):
    return torch.exp(-torch.exp(z))


def time_mixing(r, k, v, a, u, S=None):
    """r, k, a [T, H, d], v [T, H, dv], u [H, d] -> ([T, H, dv], the state after the last token)."""
    T, H, d = r.shape
    S = torch.zeros(H, d, v.shape[2], dtype=r.dtype) if S is None else S
    out = torch.zeros(T, H, v.shape[2], dtype=r.dtype)
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = ((S + u[:, :, None] * kv) * r[t][:, :, None]).sum(1)
        S = a[t][:, :, None] * S + kv
    return out, S


def wkv(h, w, p, mix, eps, low):
    T = h.shape[0]
    H, d = mix["heads"], mix["dim"]
    h = rnd(h, low)
    before = shifted(h)
    m = {s: mixed(h, before, w[p + "mu." + s]) for s in "rkvgw"}
    r, k, v = (product(m[s], w[p + s], low).view(T, H, d) for s in "rkv")
    z = torch.tanh(rnd(m["w"], low) @ w[p + "w1"].to(h.dtype).T) @ w[p + "w2"].to(h.dtype).T + w[p + "w0"]
    o, _ = time_mixing(r, k, v, decay(z).view(T, H, d), w[p + "u"])
    o = unit_norm(o, eps).reshape(T, H * d) * w[p + "norm"] * silu(product(m["g"], w[p + "g"], low))
    return product(o, w[p + "o"], low)


# ---- attention --------------------------------------------------------------------------------------------
def frequencies(rot):
    i = torch.arange(rot["dims"] // 2, dtype=torch.float64)
    f = torch.pow(torch.tensor(float(rot["base"]), dtype=torch.float64), -2.0 * i / max(rot["dims"], 1))
    sc = rot.get("scaling")
    if not sc:
        return f
    out = []
    for v in f.tolist():
        length = 2 * math.pi / v
        if length < sc["original"] / sc["high"]:
            out.append(v)
        elif length > sc["original"] / sc["low"]:
            out.append(v / sc["factor"])
        else:
            s = (sc["original"] / length - sc["low"]) / (sc["high"] - sc["low"])
            out.append((1 - s) * v / sc["factor"] + s * v)
    return torch.tensor(out, dtype=torch.float64)


def turn_halves(v, ang):
    """v [T, heads, d]; elements i and i + n of each head, i < n = ang.shape[1], are turned by ang [T, n]."""
    n = ang.shape[1]
    c, s = torch.cos(ang).to(v.dtype)[:, None, :], torch.sin(ang).to(v.dtype)[:, None, :]
    a, b = v[..., :n], v[..., n:2 * n]
    return torch.cat([a * c - b * s, b * c + a * s, v[..., 2 * n:]], -1)


def first_visible(i, size):
    """the first position that position i sees through a window of `size` positions, itself included"""
    return max(0, i - size + 1)


def softmax_with_one(scores):
    """exp(s_j) / (1 + sum exp(s_j))"""
    top = torch.clamp(scores.max(), min=0.0)
    e = torch.exp(scores - top)
    return e / (e.sum() + torch.exp(-top))


def attention(h, w, p, mix, eps, low, lent=None):
    """-> (output, (keys, values)); lent: the keys and values of the layer this one reads."""
    T = h.shape[0]
    H, G, d, dv = mix["heads"], mix["kv_heads"], mix["dim"], mix["vdim"]
    ang = torch.arange(T, dtype=torch.float64)[:, None] * frequencies(mix["rot"])[None, :]
    q = unit_norm(product(h, w[p + "q"], low) + w[p + "q.b"], eps) * w[p + "q.norm"]
    q = rnd(turn_halves(q.view(T, H, d), ang), low)
    if lent is None:
        k = unit_norm(product(h, w[p + "k"], low) + w[p + "k.b"], eps) * w[p + "k.norm"]
        k = rnd(turn_halves(k.view(T, G, d), ang), low)
        v = rnd(product(h, w[p + "v"], low) + w[p + "v.b"], low).view(T, G, dv)
    else:
        k, v = lent
    o = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(T):
        lo = first_visible(i, mix["mask"]["size"])
        for n in range(H):
            kv = n // (H // G)
            o[i, n] = softmax_with_one((k[lo:i + 1, kv] @ q[i, n]) * mix["scale"]) @ v[lo:i + 1, kv]
    o = o * torch.sigmoid(product(h, w[p + "g"], low))[:, :, None]
    return product(o.reshape(T, H * dv), w[p + "o"], low), (k, v)


# ---- feed-forward -----------------------------------------------------------------------------------------
def route(z, correction, router):
    """z [experts + identity], one token -> (chosen, weights)"""
    s = torch.softmax(z, -1)
    choice = s + correction
    groups = router.get("groups")
    if groups:
        per = len(z) // groups["count"]
        best = choice.view(groups["count"], per).max(-1).values
        kept = torch.topk(best, groups["keep"]).indices.tolist()
        open_ = torch.tensor([e // per in kept for e in range(len(z))])
        choice = torch.where(open_, choice, torch.full_like(choice, -math.inf))
    chosen = torch.topk(choice, router["top"]).indices
    return chosen, s[chosen] / (s[chosen].sum() + 1e-20)


def expert(h, w, p, low):
    return product(rnd(silu(product(h, w[p + "gate"], low)) * product(h, w[p + "up"], low), low), w[p + "down"], low)


def experts(h, w, p, mlp, low):
    router = mlp["router"]
    hl = rnd(h, low)
    z = hl @ w[p + "router"].to(h.dtype).T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        chosen, weight = route(z[t], w[p + "correction"], router)
        for e, a in zip(chosen.tolist(), weight):
            y = hl[t] if e >= router["experts"] else expert(h[t:t + 1], w, p + "e%d." % e, low)[0]
            out[t] += a * y
    return out


# ---- the whole --------------------------------------------------------------------------------------------
def forward(cfg, w, tokens, low=F32, every_layer=None):
    """Logits [T, vocab] of one sequence.  every_layer: a list that gets the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)]
    kv = {}
    for i, layer in enumerate(cfg["layers"]):
        p = "l%d." % i
        h = offset_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "wkv":
            y = wkv(h, w, p + "mix.", layer["mixer"], eps, low)
        else:
            source = layer["mixer"].get("kv_from")
            y, kv[i] = attention(h, w, p + "mix.", layer["mixer"], eps, low, None if source is None else kv[source])
        if layer["mlp"] is not None:
            y = y + experts(h, w, p + "mlp.", layer["mlp"], low)
        x = x + cfg["residual_mult"] * y
        if every_layer is not None:
            every_layer.append(x.clone())
    return product(offset_norm(x, w["final.norm"], eps), w["head"], F32)


def greedy(cfg, w, prompt, n, low=F32):
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(torch.argmax(forward(cfg, w, tokens, low)[-1])))
    return tokens[len(prompt):]
