"""Teberax written plainly: one function per mechanism, a whole sequence at a time, token by token where a state is
carried.  It shares nothing with the package: tensors come as a dict of checkpoint names, the configuration as the
parsed config.json.  `bf16=True` rounds to bfloat16 at the places where an engine that stores bfloat16 numbers must
(the products' inputs and outputs, what a cache holds); how far that moves the plain model's own logits is the
yardstick of the bfloat16 tests.

    x = n_e(E[token]);  per layer  x <- x + n1b(mixer(n1(x))),  x <- x + n2b(ff(n2(x)));  logits = cap tanh(H n_f(x) / cap)

with n(x) = x / sqrt(mean(x^2) + eps) * g, g one number.
"""

import math

import torch

F = torch.float64


def rnd(t, bf16):
    return t.to(torch.bfloat16).to(t.dtype) if bf16 else t


def linear(w, x, bf16, bias=None):
    """W x (+ b) for every row of x, the product rounded as a bfloat16 product would be."""
    y = rnd(rnd(x, bf16) @ w.to(x.dtype).t(), bf16)
    return y if bias is None else y + bias.to(x.dtype)


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def one_number_norm(x, g, eps):
    return rms(x, eps) * g.to(x.dtype)


def softcap(z, cap):
    return cap * torch.tanh(z / cap) if cap else z


# ---- attention: masks, the softmax with and without a sink, rotations ------------------------------------------------
def visible(T, mask):
    """[T, T] bool: whether position i (row) sees position j (column).  mask None: every j <= i."""
    i, j = torch.arange(T).view(-1, 1), torch.arange(T).view(1, -1)
    seen = j <= i
    if mask and mask.get("size"):
        seen = seen & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))
    return seen


def softmax_weights(s, sink):
    """The softmax over a row's scores; with a sink one more score of 0 in the denominator, which has no value."""
    if sink:
        s = torch.cat([s, torch.zeros_like(s[..., :1])], dim=-1)
        return torch.softmax(s, dim=-1)[..., :-1]
    return torch.softmax(s, dim=-1)


def attention(q, k, v, scale, mask=None, cap=0.0, sink=False):
    """q [T, H, D], k [T, G, D], v [T, G, E]: head h reads kv head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    seen = visible(T, mask)
    for h in range(H):
        g = h // (H // G)
        s = softcap((q[:, h] @ k[:, g].t()) * scale, cap).masked_fill(~seen, -math.inf)
        out[:, h] = softmax_weights(s, sink) @ v[:, g]
    return out


def rotate_neighbours(x, positions, rot):
    """x [T, heads, D]: of every head's first rot.dims coordinates the pair (2i, 2i + 1) turns by position * f_i, f_i =
    base^(-2i / dims), divided by scaling.factor where rot names one."""
    R = rot["dims"]
    f = float(rot["base"]) ** (-2.0 * torch.arange(R // 2, dtype=F) / R)
    if rot.get("scaling"):
        f = f / float(rot["scaling"]["factor"])
    ang = positions.to(F).unsqueeze(1) * f.unsqueeze(0)
    cos, sin = torch.cos(ang).to(x.dtype).unsqueeze(1), torch.sin(ang).to(x.dtype).unsqueeze(1)
    a, b = x[..., 0:R:2], x[..., 1:R:2]
    out = x.clone()
    out[..., 0:R:2] = a * cos - b * sin
    out[..., 1:R:2] = b * cos + a * sin
    return out


# ---- differential attention -------------------------------------------------------------------------------------------
def differential_lambda(W, p, diff, dtype=F):
    def dot(a, b):
        return (W[p + a].to(dtype) * W[p + b].to(dtype)).sum()

    return torch.exp(dot("lq1", "lk1")) - torch.exp(dot("lq2", "lk2")) + diff


def differential_combine(a1, a2, lam, diff, eps):
    """Two maps' heads [T, H, E] -> the difference over its root mean square, times (1 - diff)."""
    return rms(a1 - lam * a2, eps) * (1.0 - diff)


def differential_attention(h, W, p, m, eps, bf16, kept, index):
    """kept: layer -> (k1, k2, v) of the layers that have projections of their own, for those that read them."""
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = linear(W[p + "q"], h, bf16).view(T, H, 2, D)
    if m.get("kv_from") is None:
        k = linear(W[p + "k"], h, bf16).view(T, G, 2, D)
        kept[index] = (k[:, :, 0], k[:, :, 1], linear(W[p + "v"], h, bf16).view(T, G, E))
        k1, k2, v = kept[index]
    else:
        k1, k2, v = kept[m["kv_from"]]
    a1 = attention(q[:, :, 0], k1, v, m["scale"], m.get("mask"))
    a2 = attention(q[:, :, 1], k2, v, m["scale"], m.get("mask"))
    lam = differential_lambda(W, p, m["diff"], h.dtype)
    o = differential_combine(a1, a2, lam, m["diff"], eps)
    return linear(W[p + "o"], o.reshape(T, H * E), bf16)


# ---- an attention beside a gated linear attention ----------------------------------------------------------------------
def sink_attention(h, W, p, m, positions, bf16):
    """Biased projections, neighbours turned, capped scores, a softmax with a sink."""
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = linear(W[p + "q"], h, bf16, W[p + "q.b"]).view(T, H, D)
    k = linear(W[p + "k"], h, bf16, W[p + "k.b"]).view(T, G, D)
    v = rnd(linear(W[p + "v"], h, bf16, W[p + "v.b"]), bf16).view(T, G, E)
    if m.get("rot"):
        q, k = rotate_neighbours(q, positions, m["rot"]), rotate_neighbours(k, positions, m["rot"])
    o = attention(rnd(q, bf16), rnd(k, bf16), v, m["scale"], m.get("mask"), m.get("softcap", 0.0), sink=True)
    return linear(W[p + "o"], o.reshape(T, H * E), bf16, W[p + "o.b"])


def channel_decay_scan(q, k, v, alpha):
    """Per head: S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t.  q, k, alpha [T, H, D], v [T, H, E]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    out = []
    for t in range(T):
        S = alpha[t].unsqueeze(2) * S + k[t].unsqueeze(2) * v[t].unsqueeze(1)
        out.append(torch.einsum("hde,hd->he", S, q[t]))
    return torch.stack(out)


def channel_decays(z, tau):
    return torch.exp(torch.nn.functional.logsigmoid(z) / tau)


def gated_linear_attention(h, W, p, m, eps, bf16):
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    q = linear(W[p + "q"], h, bf16).view(T, H, D) * D**-0.5
    k = linear(W[p + "k"], h, bf16).view(T, H, D)
    v = linear(W[p + "v"], h, bf16).view(T, H, E)
    z = linear(W[p + "a2"], linear(W[p + "a1"], h, bf16), bf16, W[p + "a2.b"])
    alpha = channel_decays(z, float(m["tau"])).view(T, H, D)
    o = rms(channel_decay_scan(q, k, v, alpha), eps) * W[p + "norm"].to(h.dtype)
    o = o.reshape(T, H * E) * torch.nn.functional.silu(linear(W[p + "g"], h, bf16))
    return linear(W[p + "o"], o, bf16)


def normed_mean(left, right, g_left, g_right, eps):
    return 0.5 * (rms(left, eps) * g_left.to(left.dtype) + rms(right, eps) * g_right.to(right.dtype))


def parallel_mixer(h, W, p, m, positions, eps, bf16):
    left = sink_attention(h, W, p + "left.", m["left"], positions, bf16)
    right = gated_linear_attention(h, W, p + "right.", m["right"], eps, bf16)
    return normed_mean(left, right, W[p + "left.out"], W[p + "right.out"], eps)


# ---- attention through a latent ------------------------------------------------------------------------------------------
def latent_attention(h, W, p, m, positions, eps, bf16):
    T = h.shape[0]
    H, D, R, E, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = linear(W[p + "q"], h, bf16).view(T, H, D + R)
    down = linear(W[p + "dkv"], h, bf16)
    c = rnd(rms(down[:, :C], eps) * W[p + "dkv.norm"].to(h.dtype), bf16)
    k_plain = linear(W[p + "uk"], c, bf16).view(T, H, D)
    v = linear(W[p + "uv"], c, bf16).view(T, H, E)
    k, qq = k_plain, q[..., :D]
    if R:
        k_turned = rnd(rotate_neighbours(down[:, C:].view(T, 1, R), positions, m["rot"]), bf16).expand(T, H, R)
        q_turned = rnd(rotate_neighbours(q[..., D:], positions, m["rot"]), bf16)
        qq, k = torch.cat([qq, q_turned], dim=-1), torch.cat([k, k_turned], dim=-1)
    o = attention(qq, k, v, m["scale"], m.get("mask"))
    return linear(W[p + "o"], o.reshape(T, H * E), bf16)


# ---- feed-forwards -----------------------------------------------------------------------------------------------------------
def poly_norm(z, act, eps):
    a, b, c, e = act.to(z.dtype)
    return a * rms(z, eps) + b * rms(z * z, eps) + c * rms(z * z * z, eps) + e


def poly_mlp(h, W, p, eps, bf16):
    return linear(W[p + "down"], poly_norm(linear(W[p + "up"], h, bf16), W[p + "act"], eps), bf16)


def corrected_choice(s, correction, top):
    """The `top` largest s + correction of every row; of equal ones the lower number first."""
    return torch.sort(s + correction.to(s.dtype), dim=-1, descending=True, stable=True).indices[:, :top]


def experts(h, W, p, f, bf16):
    """Experts chosen by corrected softmax scores; those numbered `experts` and up are the input itself."""
    r = f["router"]
    n, same, top = r["experts"], r.get("identity", 0), r["top"]
    s = torch.softmax(rnd(h, bf16) @ W[p + "router"].to(h.dtype).t(), dim=-1)
    chosen = corrected_choice(s, W[p + "correction"], top)
    silu = torch.nn.functional.silu
    out = torch.zeros_like(h)
    for e in range(n + same):
        rows = (chosen == e).any(dim=-1).nonzero().flatten()
        if not rows.numel():
            continue
        x = y = rnd(h[rows], bf16)
        if e < n:
            a = silu(linear(W[f"{p}e{e}.gate"], x, bf16)) * linear(W[f"{p}e{e}.up"], x, bf16)
            y = linear(W[f"{p}e{e}.down"], a, bf16)
        out[rows] += s[rows, e].unsqueeze(1) * y
    return out


# ---- the model ------------------------------------------------------------------------------------------------------------
def forward(raw, W, tokens, bf16=False, dtype=F, layers_out=None):
    """Logits [T, vocab] of one sequence from position 0.  layers_out: a list that receives the stream after every layer."""
    W = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in W.items()}
    eps = raw["norm"]["eps"]
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(tokens.shape[0])
    x = one_number_norm(W["embed"][tokens], W["embed.norm"], eps)
    kept = {}
    for i, layer in enumerate(raw["layers"]):
        p, mix, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        h = one_number_norm(x, W[p + "norm1"], eps)
        if layer["type"] == "attention":
            y = differential_attention(h, W, p + "mix.", mix, eps, bf16, kept, i)
        elif layer["type"] == "parallel":
            y = parallel_mixer(h, W, p + "mix.", mix, positions, eps, bf16)
        elif layer["type"] == "latent_attention":
            y = latent_attention(h, W, p + "mix.", mix, positions, eps, bf16)
        else:
            raise ValueError(layer["type"])
        x = x + one_number_norm(y, W[p + "norm1b"], eps)
        if f is not None:
            h = one_number_norm(x, W[p + "norm2"], eps)
            y = poly_mlp(h, W, p + "mlp.", eps, bf16) if f["kind"] == "dense" else experts(h, W, p + "mlp.", f, bf16)
            x = x + one_number_norm(rnd(y, bf16), W[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x)
    x = one_number_norm(x, W["final.norm"], eps)
    return softcap(rnd(x, bf16) @ W["head"].t(), raw.get("logit_softcap", 0.0))


def logits(raw, W, ids, rounded=False):
    """Logits [T, vocab] in float32: exact (float64 inside), or with bfloat16 activations."""
    return forward(raw, W, ids, bf16=rounded).float()
