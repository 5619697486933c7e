"""Plain reference of the Kozipel design: chunk-local softmax attention beside gated linear attention, lightning attention, gated relu feed-forwards,
a span of layers that runs several times.  One function per mechanism, written from the equations, in float64 by default, one sequence at a time, no
cache, token after token where there is a recurrence: the logits of position i are a function of tokens[0..i] alone.  Shares no code with aria_amd
(TEST INFRASTRUCTURE ONLY).

``cast`` (default: nothing) is applied where a 16-bit implementation may round a tensor -- inputs and results of the projections, keys, values,
activations -- so that the error of rounding alone can be measured beside an implementation's.

``cfg`` is the parsed config.json, ``w`` a dict of tensors under the checkpoint's names."""
import torch


def exact(x):
    return x


def to_bf16(x):
    return x.to(torch.bfloat16).to(x.dtype)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rms(x, eps):
    """x over its root mean square, last dimension"""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def chunk_attention(q, k, v, scale, size):
    """q, k [T, d], v [T, dv] of one head: position i sees the positions j <= i of its own chunk of ``size``."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=q.dtype)
    for i in range(q.shape[0]):
        first = i // size * size
        s = (k[first:i + 1] @ q[i]) * scale
        p = torch.exp(s - s.max())
        out[i] = (p / p.sum()) @ v[first:i + 1]
    return out


def linear_recurrence(q, k, v, decay, state=None):
    """q, k [T, d], v [T, dv], decay [T, d] (of the state's rows) of one head -> outputs [T, dv], last state [d, dv]."""
    s = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros_like(v)
    for t in range(q.shape[0]):
        s = decay[t][:, None] * s + torch.outer(k[t], v[t])
        out[t] = s.T @ q[t]
    return out, s


def chunked_mixer(h, w, pre, m, cast=exact):
    """Grouped-query softmax attention inside chunks; h [T, D] -> [T, D]."""
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = cast(h @ w[pre + ".q"].T).view(T, H, d)
    k = cast(h @ w[pre + ".k"].T).view(T, G, d)
    v = cast(h @ w[pre + ".v"].T).view(T, G, dv)
    heads = [chunk_attention(q[:, i], k[:, i // (H // G)], v[:, i // (H // G)], m["scale"], m["mask"]["size"]) for i in range(H)]
    return cast(cast(torch.cat(heads, -1)) @ w[pre + ".o"].T)


def gated_linear_mixer(h, w, pre, m, eps, cast=exact):
    """Linear attention with a decay per token and key channel, sigmoid(z)^(1 / tau); h [T, D] -> [T, D]."""
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (cast(h @ w[pre + ".q"].T) * d ** -0.5).view(T, H, d)
    k = cast(h @ w[pre + ".k"].T).view(T, H, d)
    v = cast(h @ w[pre + ".v"].T).view(T, H, dv)
    z = (cast(h @ w[pre + ".a1"].T) @ w[pre + ".a2"].T + w[pre + ".a2.b"]).view(T, H, d)
    decay = sigmoid(z) ** (1.0 / m["tau"])
    heads = [rms(linear_recurrence(q[:, i], k[:, i], v[:, i], decay[:, i])[0], eps) * w[pre + ".norm"] for i in range(H)]
    o = torch.cat(heads, -1) * silu(cast(h @ w[pre + ".g"].T))
    return cast(cast(o) @ w[pre + ".o"].T)


def lightning_mixer(h, w, pre, m, eps, cast=exact):
    """Linear attention with one constant decay per head, silu on queries, keys and values; h [T, D] -> [T, D]."""
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = cast(silu(cast(h @ w[pre + ".q"].T))).view(T, H, d)
    k = cast(silu(cast(h @ w[pre + ".k"].T))).view(T, H, d)
    v = cast(silu(cast(h @ w[pre + ".v"].T))).view(T, H, dv)
    heads = [linear_recurrence(q[:, i], k[:, i], v[:, i], torch.full((T, d), m["decay"][i], dtype=h.dtype))[0] for i in range(H)]
    o = rms(torch.cat(heads, -1), eps) * w[pre + ".norm"] * sigmoid(cast(h @ w[pre + ".g"].T))
    return cast(cast(o) @ w[pre + ".o"].T)


def parallel_mixer(h, w, pre, m, eps, cast=exact):
    left = rms(chunked_mixer(h, w, pre + ".left", m["left"], cast), eps) * w[pre + ".left.out"]
    right = rms(gated_linear_mixer(h, w, pre + ".right", m["right"], eps, cast), eps) * w[pre + ".right.out"]
    return 0.5 * (left + right)


def relu_glu(h, w, pre, cast=exact):
    gate, up = cast(h @ w[pre + ".gate"].T), cast(h @ w[pre + ".up"].T)
    return cast(cast(torch.where(gate > 0, gate, torch.zeros_like(gate)) * up) @ w[pre + ".down"].T)


def layer_runs(cfg):
    """[(layer, starts a pass after the first)] in the order they run"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    runs = [(i, False) for i in range(loop["start"])]
    for p in range(loop["times"]):
        runs += [(i, p > 0 and i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, False) for i in range(loop["stop"], n)]


def forward(cfg, weights, tokens, dtype=torch.float64, want_layers=False, cast=exact):
    """tokens: list of ints -> logits [T, vocab] (and the residual stream after every layer run)."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps, mult, cap = cfg["norm"]["eps"], cfg["residual_mult"], cfg["logit_softcap"]

    def norm(x, name):
        return cast(rms(x, eps) * (1 + w[name]))

    first = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    x, trace = first, []
    for i, again in layer_runs(cfg):
        if again:
            x = x + first
        layer, p = cfg["layers"][i], f"l{i}"
        mixer = {"lightning": lightning_mixer, "parallel": parallel_mixer}[layer["type"]]
        x = x + mult * mixer(norm(x, p + ".norm1"), w, p + ".mix", layer["mixer"], eps, cast)
        if layer.get("mlp") is not None:
            x = x + mult * relu_glu(norm(x, p + ".norm2"), w, p + ".mlp", cast)
        trace.append(x)
    logits = norm(x, "final.norm") @ w["head"].T
    logits = cap * torch.tanh(logits / cap)
    return (logits, torch.stack(trace)) if want_layers else logits
