"""Plain reference of the Duguzen design: latent attention, dynamic-tanh norms, squared-relu and group-limited mixture feed-forwards, layers
that borrow another layer's weights.  One function per mechanism, written from the equations, in float64 by default, one sequence at a time,
no cache: the logits of position i are a function of tokens[0..i] alone.  Shares no code with aria_amd (TEST INFRASTRUCTURE ONLY).

``cast`` (default: nothing) is applied where a 16-bit implementation may round a tensor -- inputs and results of the projections, latents, keys,
values, activations -- so that the error of rounding alone can be measured beside an implementation's.

``cfg`` is the parsed config.json, ``w`` a dict of tensors under the checkpoint's names."""
import math

import torch


def exact(x):
    return x


def to_bf16(x):
    return x.to(torch.bfloat16).to(x.dtype)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def relu_squared(z):
    return torch.where(z > 0, z, torch.zeros_like(z)) ** 2


def dynamic_tanh(x, alpha, weight, bias):
    return torch.tanh(alpha * x) * weight + bias


def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def rotate_half(x, pos, base, dims):
    """x [..., n], pos broadcastable over x's leading dimensions: the first ``dims`` components turn, pairs (i, i + dims / 2)."""
    half = dims // 2
    out = x.clone()
    for i in range(half):
        a = pos * base ** (-2.0 * i / dims)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., i + half] = v * torch.cos(a) + u * torch.sin(a)
    return out


def causal_softmax_attention(q, k, v, scale):
    """q [T, dq], k [T, dq], v [T, dv] of one head."""
    T = q.shape[0]
    s = (q @ k.T) * scale
    s = s.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), -math.inf)
    s = s - s.max(-1, keepdim=True).values
    p = torch.exp(s)
    return (p / p.sum(-1, keepdim=True)) @ v


def latent_attention(h, w, pre, m, eps, cast=exact):
    """h [T, D] -> [T, D].  m: the layer's mixer sizes; pre: name prefix ('l3.mix')."""
    T = h.shape[0]
    H, dn, dr, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T, dtype=h.dtype)
    q = cast(h @ w[pre + ".q"].T).view(T, H, dn + dr)
    down = cast(h @ w[pre + ".dkv"].T)
    c = cast(rms_norm(down[:, :R], w[pre + ".dkv.norm"], eps))
    rot = m["rot"]
    kr = cast(rotate_half(down[:, R:], pos, rot["base"], rot["dims"]))
    gate = torch.sigmoid(h @ w[pre + ".g"].T)
    heads = []
    for i in range(H):
        kn = cast(c @ w[pre + ".uk"][i * dn:(i + 1) * dn].T)
        v = cast(c @ w[pre + ".uv"][i * dv:(i + 1) * dv].T)
        qr = cast(rotate_half(q[:, i, dn:], pos, rot["base"], rot["dims"]))
        qi, ki = torch.cat([q[:, i, :dn], qr], -1), torch.cat([kn, kr], -1)
        heads.append(causal_softmax_attention(qi, ki, v, m["scale"]) * gate[:, i:i + 1])
    return cast(cast(torch.cat(heads, -1)) @ w[pre + ".o"].T)


def choose_experts(choice, groups, keep, top):
    """choice [E] of one token -> the ``top`` best experts of the ``keep`` best groups (a group counts by its two best experts)."""
    E = choice.numel()
    size = E // groups
    rank = [sum(sorted((float(x) for x in choice[g * size:(g + 1) * size]), reverse=True)[:2]) for g in range(groups)]
    kept = sorted(range(groups), key=lambda g: -rank[g])[:keep]
    allowed = [e for g in kept for e in range(g * size, (g + 1) * size)]
    return sorted(allowed, key=lambda e: -float(choice[e]))[:top]


def routing_margin(choice, groups, keep, top):
    """how far one token's choice is from another one: the smallest gap between a group kept and one left out, an expert taken and one left"""
    size = choice.numel() // groups
    rank = sorted((sum(sorted((float(x) for x in choice[g * size:(g + 1) * size]), reverse=True)[:2]) for g in range(groups)), reverse=True)
    taken = choose_experts(choice, groups, keep, choice.numel())
    gaps = [rank[keep - 1] - rank[keep]] if keep < groups else []
    if top < len(taken):
        gaps.append(float(choice[taken[top - 1]]) - float(choice[taken[top]]))
    return min(gaps) if gaps else math.inf


def mixture(h, w, pre, mlp, margins=None, cast=exact):
    r = mlp["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    s = torch.sigmoid(h @ w[pre + ".router"].T)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        if margins is not None:
            margins[t] = min(margins[t], routing_margin(s[t] + w[pre + ".correction"], g["count"], g["keep"], r["top"]))
        for e in choose_experts(s[t] + w[pre + ".correction"], g["count"], g["keep"], r["top"]):
            up = cast(silu(cast(w[f"{pre}.e{e}.gate"] @ h[t])) * cast(w[f"{pre}.e{e}.up"] @ h[t]))
            out[t] += s[t, e] * cast(w[f"{pre}.e{e}.down"] @ up)
    return out


def dense_ff(h, w, pre, cast=exact):
    return cast(cast(relu_squared(cast(h @ w[pre + ".up"].T))) @ w[pre + ".down"].T)


def forward(cfg, weights, tokens, dtype=torch.float64, want_layers=False, margins=None, cast=exact):
    """tokens: list of ints -> logits [T, vocab] (and the residual stream after every layer).  margins: list [T], lowered to each position's
    smallest routing margin."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]

    def norm(x, name):
        return dynamic_tanh(x, w[name + ".alpha"], w[name], w[name + ".b"])

    x = w["embed"][torch.as_tensor(tokens)]
    trace = []
    for i, layer in enumerate(cfg["layers"]):
        src = f"l{layer.get('weights_of', i)}"
        x = x + norm(latent_attention(cast(norm(x, src + ".norm1")), w, src + ".mix", layer["mixer"], eps, cast), src + ".norm1b")
        mlp = layer.get("mlp")
        if mlp is not None:
            h = cast(norm(x, src + ".norm2"))
            f = dense_ff(h, w, src + ".mlp", cast) if mlp["kind"] == "dense" else mixture(h, w, src + ".mlp", mlp, margins, cast)
            x = x + norm(f, src + ".norm2b")
        trace.append(x)
    logits = cast(norm(x, "final.norm")) @ w["head"].T
    return (logits, torch.stack(trace)) if want_layers else logits
