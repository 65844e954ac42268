"""Tokuvik written plainly: one function per mechanism, a whole sequence at a time, token by token where a state is
carried.  It shares nothing with the package: tensors come as a dict of checkpoint names, the configuration as the
parsed config.json.  `bf16=True` rounds to bfloat16 at the places where an engine that stores bfloat16 numbers must
(the products' inputs and outputs, what a cache holds); how far that moves the plain model's own logits is the
yardstick of the bfloat16 tests.

    x = E[token];  per layer  x <- x + n1b(mixer(n1(x))),  x <- x + n2b(ff(n2(x))),  x <- x + r(P (gelu(G x) * e));
    logits = E n_f(x)

with n(x) = (x - mean) / sqrt(var + eps) * w, r(y) = y / sqrt(mean(y^2) + eps) * w, and e the layer's share of the row that
a second table holds for the token.
"""

import math

import torch

F = torch.float64


def rnd(t, bf16):
    return t.to(torch.bfloat16).to(t.dtype) if bf16 else t


def linear(w, x, bf16):
    """W x for every row of x, the product rounded as a bfloat16 product would be."""
    return rnd(rnd(x, bf16) @ w.to(x.dtype).t(), bf16)


# ---- norms ---------------------------------------------------------------------------------------------------------
def layer_norm(x, w, eps):
    centred = x - x.mean(dim=-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(dim=-1, keepdim=True) + eps) * w.to(x.dtype)


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w.to(x.dtype)


def grouped_rms_norm(x, w, eps, groups):
    """Every one of `groups` equal parts of the row over its own root mean square."""
    parts = x.view(*x.shape[:-1], groups, -1)
    return (parts / torch.sqrt((parts * parts).mean(dim=-1, keepdim=True) + eps)).reshape(x.shape) * w.to(x.dtype)


# ---- what a position sees, and the softmax -----------------------------------------------------------------------------
def visible(T, chunk=0):
    """[T, T] bool: whether position i (row) sees position j (column): j <= i, and both in the same chunk (0: no chunks)."""
    i, j = torch.arange(T).view(-1, 1), torch.arange(T).view(1, -1)
    seen = j <= i
    return seen & (i // chunk == j // chunk) if chunk else seen


def softmax_weights(s, sink=None):
    """The softmax over a row's scores; `sink`: one more score in the denominator, which has no value."""
    if sink is None:
        return torch.softmax(s, dim=-1)
    s = torch.cat([s, sink.to(s.dtype).expand(*s.shape[:-1], 1)], dim=-1)
    return torch.softmax(s, dim=-1)[..., :-1]


def attention(q, k, v, scale, chunk=0, sinks=None):
    """q [T, H, D], k [T, G, D], v [T, G, E]: head h reads kv head h // (H / G); sinks [H] or None."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    seen = visible(T, chunk)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].t()) * scale).masked_fill(~seen, -math.inf)
        out[:, h] = softmax_weights(s, None if sinks is None else sinks[h]) @ v[:, g]
    return out


# ---- attention over chunks, with a gate per head -----------------------------------------------------------------------
def head_gates(g, heads):
    """heads [T, H, E] times one number a head, sigmoid(g) [T, H]."""
    return heads * torch.sigmoid(g).unsqueeze(-1)


def chunked_attention(h, W, p, m, eps, bf16, kept, index):
    """kept: layer -> (k, v) of the layers that have projections of their own, for those that read them."""
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rnd(rms_norm(linear(W[p + "q"], h, bf16), W[p + "q.norm"], eps), bf16).view(T, H, D)
    if m.get("kv_from") is None:
        k = rnd(rms_norm(linear(W[p + "k"], h, bf16), W[p + "k.norm"], eps), bf16).view(T, G, D)
        kept[index] = (k, linear(W[p + "v"], h, bf16).view(T, G, E))
        k, v = kept[index]
    else:
        k, v = kept[m["kv_from"]]
    o = attention(q, k, v, m["scale"], (m.get("mask") or {}).get("size", 0))
    o = head_gates(linear(W[p + "g"], h, bf16), rnd(o, bf16))
    return linear(W[p + "o"], o.reshape(T, H * E), bf16)


# ---- attention through a latent, with a sink per head ----------------------------------------------------------------------
def latent_attention(h, W, p, m, eps, bf16):
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    cq = rnd(rms_norm(linear(W[p + "dq"], h, bf16), W[p + "dq.norm"], eps), bf16)
    q = linear(W[p + "uq"], cq, bf16).view(T, H, D)
    c = rnd(rms_norm(linear(W[p + "dkv"], h, bf16), W[p + "dkv.norm"], eps), bf16)
    k = linear(W[p + "uk"], c, bf16).view(T, H, D)
    v = linear(W[p + "uv"], c, bf16).view(T, H, E)
    o = rnd(attention(q, k, v, m["scale"], sinks=W[p + "sink"]), bf16).reshape(T, H * E)
    return linear(W[p + "o"], o * torch.sigmoid(linear(W[p + "g"], h, bf16)), bf16)


# ---- a state space per head ----------------------------------------------------------------------------------------------------
def causal_conv(x, w, bias):
    """x [T, C], w [C, taps]: out[t] = sum_i w[:, i] x[t - (taps - 1) + i] + bias, zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, x.shape[1], dtype=x.dtype), x])
    return sum(padded[i : i + T] * w[:, i].to(x.dtype) for i in range(taps)) + bias.to(x.dtype)


def state_space_scan(x, B, C, dt, log_rate, skip):
    """x [T, H, E], B and C [T, G, N], dt [T, H]: per head, with the group's B and C,
    S_t = exp(-exp(log_rate) dt) S_(t-1) + dt B_t x_t^T,  y_t = S_t^T C_t + skip x_t."""
    T, H, E = x.shape
    G, N = B.shape[1], B.shape[2]
    of = torch.arange(H) // (H // G)
    S = torch.zeros(H, N, E, dtype=x.dtype)
    out = []
    for t in range(T):
        a = torch.exp(-torch.exp(log_rate.to(x.dtype)) * dt[t])
        S = a.view(H, 1, 1) * S + dt[t].view(H, 1, 1) * B[t][of].unsqueeze(2) * x[t].unsqueeze(1)
        out.append((S * C[t][of].unsqueeze(2)).sum(dim=1) + skip.to(x.dtype).unsqueeze(1) * x[t])
    return torch.stack(out)


def softplus(z):
    return torch.logaddexp(z, torch.zeros_like(z))


def state_space(h, W, p, m, eps, bf16):
    T = h.shape[0]
    H, E, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * E
    z, xbc, dt = torch.split(linear(W[p + "in"], h, bf16), [inner, inner + 2 * G * N, H], dim=-1)
    xbc = causal_conv(xbc, W[p + "conv"], W[p + "conv.b"])
    x, B, C = torch.split(xbc * torch.sigmoid(xbc), [inner, G * N, G * N], dim=-1)
    dt = softplus(dt + W[p + "dt_bias"].to(h.dtype))
    y = state_space_scan(x.reshape(T, H, E), B.reshape(T, G, N), C.reshape(T, G, N), dt, W[p + "A_log"], W[p + "D"])
    y = y.reshape(T, inner) * (z * torch.sigmoid(z))
    return linear(W[p + "o"], grouped_rms_norm(y, W[p + "norm"], eps, m["norm_groups"]), bf16)


# ---- feed-forward and the token's own input --------------------------------------------------------------------------------
def gated_mlp(h, W, p, bf16):
    g = linear(W[p + "gate"], h, bf16)
    return linear(W[p + "down"], g * torch.sigmoid(g) * linear(W[p + "up"], h, bf16), bf16)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z**3)))


def token_input(x, W, p, e, eps, bf16):
    """What a layer adds for the tokens themselves: e [T, dim] gated by the stream, projected and normed."""
    y = linear(W[p + "side.proj"], gelu_tanh(linear(W[p + "side.gate"], x, bf16)) * e, bf16)
    return rms_norm(y, W[p + "side.norm"], eps)


# ---- the model ------------------------------------------------------------------------------------------------------------
def forward(raw, W, tokens, bf16=False, dtype=F, layers_out=None):
    """Logits [T, vocab] of one sequence from position 0.  layers_out: a list that receives the stream after every layer."""
    W = {k: v.to(dtype) for k, v in W.items()}
    eps = raw["norm"]["eps"]
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    x = W["embed"][tokens]
    kept = {}
    for i, layer in enumerate(raw["layers"]):
        p, mix, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        h = layer_norm(x, W[p + "norm1"], eps)
        if layer["type"] == "attention":
            y = chunked_attention(h, W, p + "mix.", mix, eps, bf16, kept, i)
        elif layer["type"] == "latent_attention":
            y = latent_attention(h, W, p + "mix.", mix, eps, bf16)
        elif layer["type"] == "mamba2":
            y = state_space(h, W, p + "mix.", mix, eps, bf16)
        else:
            raise ValueError(layer["type"])
        x = x + layer_norm(y, W[p + "norm1b"], eps)
        if f is not None:
            y = gated_mlp(layer_norm(x, W[p + "norm2"], eps), W, p + "mlp.", bf16)
            x = x + layer_norm(y, W[p + "norm2b"], eps)
        if raw.get("token_side"):
            dim = raw["token_side"]["dim"]
            x = x + token_input(x, W, p, W["side.embed"][tokens, i * dim : (i + 1) * dim], eps, bf16)
        if layers_out is not None:
            layers_out.append(x)
    return rnd(layer_norm(x, W["final.norm"], eps), bf16) @ W["embed"].t()


def logits(raw, W, ids, rounded=False):
    """Logits [T, vocab] in float32: exact (float64 inside), or with bfloat16 activations."""
    return forward(raw, W, ids, bf16=rounded).float()
