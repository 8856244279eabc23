"""Tesopel, plainly: whole sequences, no cache, no batch, one function a mechanism.

A decoder whose layers put an RMS norm behind each sublayer and none before it,

    x += rms(mixer(x)) w1;   x += rms(ff(x)) w2        (ff may be absent)

The mixer is, layer by layer,

  "latent_attention": softmax attention inside a sliding window whose keys and values are expanded from one
      normed, compressed vector a token; no positions.  A layer may have no compressed vectors of its own and
      expand those of an earlier layer with its own matrices;
  "mlstm": a matrix memory a head with capped exponential gates, a running maximum and a normaliser;
  "retention": a matrix memory a head with a fixed decay, rotated queries and keys, a unit norm a head and a
      silu gate.

The feed-forward is gated by a swish of slope 1.702 whose two inputs are held under a limit, the second one
raised by one.  The head is the embedding table behind the model's norm, and the logits are multiplied by a
factor.

Every function takes and returns tensors of one dtype (float64 in the tests' reference runs); `rounding` is a
function applied wherever a bfloat16 model would hold a tensor in bfloat16, and the identity otherwise.  Nothing
here is shared with the engine.
"""
from __future__ import annotations

import torch


def same(x):
    return x


def rms_norm(x, weight, eps):
    """x / sqrt(mean(x^2) + eps) * weight over the last axis; weight None: no weight."""
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def window_mask(length, size):
    """[T, T] True where query i may see key j: itself and the size - 1 positions before it."""
    behind = torch.arange(length)[:, None] - torch.arange(length)[None, :]
    return (behind >= 0) & (behind < size)


def masked_softmax(scores, mask):
    scores = scores.masked_fill(~mask, float("-inf"))
    e = torch.exp(scores - scores.max(dim=-1, keepdim=True).values)
    return e / e.sum(dim=-1, keepdim=True)


def compressed(h, w, p, eps, rounding=same):
    """The vector a token leaves in the cache: c = rms(W_dkv h) w."""
    return rounding(rms_norm(rounding(h @ w[p + "dkv"].T), w[p + "dkv.norm"], eps))


def latent_attention(h, latent, w, p, c, rounding=same):
    """h [T, width]; latent [T, rank], this layer's compressed vectors or an earlier layer's."""
    T = h.shape[0]
    H, d, dv = c["heads"], c["dim"], c["vdim"]
    q = rounding(h @ w[p + "q"].T).view(T, H, d)
    k = rounding(latent @ w[p + "uk"].T).view(T, H, d)
    v = rounding(latent @ w[p + "uv"].T).view(T, H, dv)
    mask = window_mask(T, c["mask"]["size"])
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for head in range(H):
        scores = q[:, head] @ k[:, head].T * c["scale"]
        out[:, head] = masked_softmax(scores, mask) @ v[:, head]
    return rounding(rounding(out.reshape(T, H * dv)) @ w[p + "o"].T)


def capped(z, cap):
    return cap * torch.tanh(z / cap)


def mlstm(h, w, p, c, eps, rounding=same):
    """Token by token: m = max(f + m, i); S = e^(f + m' - m) S + e^(i - m) k v^T, n likewise; S^T q over
    max(|n . q|, e^-m) + 1e-6."""
    T = h.shape[0]
    H, d, dv, cap = c["heads"], c["dim"], c["vdim"], c["gate_cap"]
    q = rounding(h @ w[p + "q"].T).view(T, H, d) * d ** -0.5
    k = rounding(h @ w[p + "k"].T).view(T, H, d)
    v = rounding(h @ w[p + "v"].T).view(T, H, dv)
    log_i = capped(rounding(h @ w[p + "i"].T) + w[p + "i.b"], cap)
    log_f = torch.nn.functional.logsigmoid(capped(rounding(h @ w[p + "f"].T) + w[p + "f.b"], cap))
    S = torch.zeros(H, d, dv, dtype=h.dtype)
    n = torch.zeros(H, d, dtype=h.dtype)
    m = torch.zeros(H, dtype=h.dtype)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for t in range(T):
        m_new = torch.maximum(log_f[t] + m, log_i[t])
        keep, take = torch.exp(log_f[t] + m - m_new), torch.exp(log_i[t] - m_new)
        S = keep[:, None, None] * S + take[:, None, None] * (k[t][:, :, None] * v[t][:, None, :])
        n = keep[:, None] * n + take[:, None] * k[t]
        m = m_new
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = (S * q[t][:, :, None]).sum(1) / den[:, None]
    o = rms_norm(out, None, eps).reshape(T, H * dv) * w[p + "norm"]
    return rounding(rounding(o * torch.sigmoid(rounding(h @ w[p + "g"].T))) @ w[p + "o"].T)


def rotate_half_split(x, dims, base):
    """x [T, heads, d]: element i of the first `dims` turns with element i + dims/2 by t * base^(-2i/dims)."""
    half = dims // 2
    i = torch.arange(half, dtype=torch.float64)
    freq = (float(base) ** (-2.0 * i / dims)).to(x.dtype)
    angle = torch.arange(x.shape[0]).to(x.dtype)[:, None, None] * freq
    cos, sin = torch.cos(angle), torch.sin(angle)
    u, v, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, rest], dim=-1)


def retention(h, w, p, c, eps, rounding=same):
    T = h.shape[0]
    H, d, dv, rot = c["heads"], c["dim"], c["vdim"], c["rot"]
    q = rotate_half_split(rounding(h @ w[p + "q"].T).view(T, H, d), rot["dims"], rot["base"])
    k = rotate_half_split(rounding(h @ w[p + "k"].T).view(T, H, d), rot["dims"], rot["base"]) * d ** -0.5
    v = rounding(h @ w[p + "v"].T).view(T, H, dv)
    decay = torch.tensor(c["decay"], dtype=h.dtype)
    S = torch.zeros(H, d, dv, dtype=h.dtype)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    g = rounding(h @ w[p + "g"].T)
    o = rms_norm(out, None, eps).reshape(T, H * dv)
    return rounding(rounding(o * (g * torch.sigmoid(g))) @ w[p + "o"].T)


def clamped_swish_gate(g, u, limit):
    """g under the limit, u between the limits; g sigmoid(1.702 g) (u + 1)."""
    g = torch.clamp(g, max=limit)
    u = torch.clamp(u, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def feed_forward(h, w, p, c, rounding=same):
    act = clamped_swish_gate(rounding(h @ w[p + "gate"].T), rounding(h @ w[p + "up"].T), c["limit"])
    return rounding(rounding(act) @ w[p + "down"].T)


def forward(tokens, w, cfg, rounding=same, keep_layers=False):
    """tokens: a list of ids; w: {name: tensor}; cfg: config.json as a dict.  Returns logits [T, vocab] (and the
    stream after every layer)."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)]
    latents, after = {}, []
    for i, layer in enumerate(cfg["layers"]):
        p, c, h = f"l{i}.mix.", layer["mixer"], rounding(x)
        if layer["type"] == "latent_attention":
            if c.get("kv_from") is None:
                latents[i] = compressed(h, w, p, eps, rounding)
            source = i if c.get("kv_from") is None else c["kv_from"]
            y = latent_attention(h, latents[source], w, p, c, rounding)
        else:
            y = {"mlstm": mlstm, "retention": retention}[layer["type"]](h, w, p, c, eps, rounding)
        x = x + rms_norm(y, w[f"l{i}.norm1"], eps)
        if layer.get("mlp") is not None:
            x = x + rms_norm(feed_forward(rounding(x), w, f"l{i}.mlp.", layer["mlp"], rounding), w[f"l{i}.norm2"], eps)
        after.append(x)
    logits = rounding(rms_norm(x, w["final.norm"], eps)) @ w["embed"].T * cfg["logit_scale"]
    return (logits, torch.stack(after)) if keep_layers else logits
