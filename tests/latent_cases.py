"""Cases of the latent-attention family (kernels, layers, Duguzen end to end), shared by the emulator tests (tests/test_emu_latent.py, CPU) and the
hardware tests (tests/test_gpu_latent.py).  Everything is compared with oracle/latent_oracle.py in float64 on configurations and weights made here."""
import math

import torch

from oracle import latent_oracle as O

bf16, f32 = torch.bfloat16, torch.float32


def gen(seed):
    return torch.Generator().manual_seed(seed)


def rnd(*shape, seed=0, scale=1.0, dtype=bf16):
    return (torch.randn(*shape, generator=gen(seed)) * scale).to(dtype)


def rel(got, want):
    got, want = got.detach().cpu().double(), want.double()
    assert got.shape == want.shape, (got.shape, want.shape)
    return float((got - want).norm() / want.norm().clamp_min(1e-30))


TOL = {f32: 2e-5, bf16: 1.5e-2}


# ------------------------------------------------------------------------------------------ configurations and weights made up here
def mixer(heads=3, dim=24, rot_dim=8, vdim=40, kv_rank=48, base=10000.0, scale=None):
    return dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale or (dim + rot_dim) ** -0.5,
                rot=dict(base=base, dims=rot_dim))


def dense(ff=56):
    return dict(kind="dense", ff=ff)


def moe(ff=24, experts=12, top=3, count=4, keep=2):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top, groups=dict(count=count, keep=keep)))


def config(layers, width=48, vocab=90, eps=1e-5):
    out = []
    for e in layers:
        mix, mlp, *of = e
        out.append(dict(type="latent_attention", mixer=mix, mlp=mlp, **({"weights_of": of[0]} if of else {})))
    return dict(architecture="Duguzen", width=width, vocab=vocab, norm=dict(eps=eps), layers=out)


def checkpoint(cfg, seed=0):
    """Random weights under the checkpoint's names: unit-ish activations throughout, peaky routing and gates that are far from one half."""
    g = gen(seed)
    D, w = cfg["width"], {}

    def t(name, *shape, scale=1.0):
        w[name] = (torch.randn(*shape, generator=g) * scale).to(bf16)

    def norm(name):
        w[name] = (1 + 0.3 * torch.randn(D, generator=g)).to(bf16)
        t(name + ".b", D, scale=0.2)
        w[name + ".alpha"] = torch.tensor(0.5 + torch.rand((), generator=g).item()).to(bf16)

    t("embed", cfg["vocab"], D)
    t("head", cfg["vocab"], D, scale=D ** -0.5)
    norm("final.norm")
    for i, L in enumerate(cfg["layers"]):
        if "weights_of" in L:
            continue
        m, p = L["mixer"], f"l{i}."
        H, qd = m["heads"], m["dim"] + m["rot_dim"]
        norm(p + "norm1"), norm(p + "norm1b")
        t(p + "mix.q", H * qd, D, scale=2 * D ** -0.5)
        t(p + "mix.dkv", m["kv_rank"] + m["rot_dim"], D, scale=2 * D ** -0.5)
        w[p + "mix.dkv.norm"] = (1 + 0.3 * torch.randn(m["kv_rank"], generator=g)).to(bf16)
        t(p + "mix.uk", H * m["dim"], m["kv_rank"], scale=m["kv_rank"] ** -0.5)
        t(p + "mix.uv", H * m["vdim"], m["kv_rank"], scale=m["kv_rank"] ** -0.5)
        t(p + "mix.g", H, D, scale=3 * D ** -0.5)
        t(p + "mix.o", D, H * m["vdim"], scale=2 * (H * m["vdim"]) ** -0.5)
        if L["mlp"] is None:
            continue
        norm(p + "norm2"), norm(p + "norm2b")
        if L["mlp"]["kind"] == "dense":
            ff = L["mlp"]["ff"]
            t(p + "mlp.up", ff, D, scale=D ** -0.5)
            t(p + "mlp.down", D, ff, scale=ff ** -0.5)
            continue
        ff, E = L["mlp"]["expert"]["ff"], L["mlp"]["router"]["experts"]
        for e in range(E):
            t(f"{p}mlp.e{e}.gate", ff, D, scale=2 * D ** -0.5)
            t(f"{p}mlp.e{e}.up", ff, D, scale=2 * D ** -0.5)
            t(f"{p}mlp.e{e}.down", D, ff, scale=ff ** -0.5)
        t(p + "mlp.router", E, D, scale=2 * D ** -0.5)
        t(p + "mlp.correction", E, scale=0.3)
    return w


CONFIGS = {
    # unequal, odd sizes; a borrowed layer between; one layer without feed-forward
    "mixed": config([(mixer(), dense()), (mixer(heads=5, dim=16, rot_dim=16, vdim=8, kv_rank=64, base=500.0), moe()), (mixer(), dense(), 0),
                     (mixer(heads=1, dim=8, rot_dim=2, vdim=24, kv_rank=20), None), (mixer(heads=5, dim=16, rot_dim=16, vdim=8, kv_rank=64, base=500.0), moe(), 1)]),
    # sizes that are no multiple of 8, everything that can be 1 is 1
    "odd": config([(mixer(heads=2, dim=13, rot_dim=6, vdim=11, kv_rank=21), moe(ff=13, experts=6, top=1, count=1, keep=1)),
                   (mixer(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=9), dense(ff=9)), (mixer(heads=2, dim=13, rot_dim=6, vdim=11, kv_rank=21),
                                                                                        moe(ff=13, experts=6, top=1, count=1, keep=1), 0)],
                  width=37, vocab=51, eps=1e-3),
    # equal sizes everywhere, groups of one expert, every group kept
    "equal": config([(mixer(heads=4, dim=16, rot_dim=16, vdim=32, kv_rank=32), moe(ff=32, experts=4, top=4, count=4, keep=4))] * 2, width=32, vocab=32),
    # sharp scores: a softmax that is close to one-hot
    "sharp": config([(mixer(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=32, scale=0.7), dense(ff=40))] * 2, width=40, vocab=64),
    # a head of more than 16384 rows (the 32-row form of the batched decode projections), and a reduction of several rounds of its waves
    "vocabulary": config([(mixer(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=32), dense(ff=24))], width=24, vocab=16411),
    "broad": config([(mixer(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=32), dense(ff=24))], width=2061, vocab=45),
    # wider than the 64-expert sort, more heads than one group of 16, fused expert launch shapes (ff % 128 == 0, width % 64 == 0)
    "wide": config([(mixer(heads=18, dim=40, rot_dim=24, vdim=64, kv_rank=160), moe(ff=128, experts=72, top=6, count=8, keep=3))], width=64, vocab=80),
}


def build(cfg, w, dev, dtype):
    from aria_amd.duguzen import DuguzenForCausalLM

    return DuguzenForCausalLM.from_tensors(cfg, w, dev, dtype)


def tokens(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=gen(seed + 77)).tolist()


def clear_tokens(cfg, w, n, seed=0, margin=0.02):
    """Random tokens at none of which the routing of any layer is a close call (a bf16 router logit may round either way there)."""
    if not any(L["mlp"] and L["mlp"]["kind"] == "moe" for L in cfg["layers"]):
        return tokens(cfg, n, seed)
    g, out = gen(seed + 99), []
    while len(out) < n:
        tries = torch.randint(0, cfg["vocab"], (40, n - len(out)), generator=g).tolist()
        for tail in tries:                         # keep the longest clear beginning of a random continuation
            gaps = [math.inf] * n
            O.forward(cfg, w, out + tail, margins=gaps)
            bad = next((i for i in range(len(out), n) if gaps[i] < margin), n)
            if bad > len(out):
                out += tail[:bad - len(out)]
                break
        else:
            raise AssertionError("no clear token")
    return out


def logit_err(got, want):
    """worst row: rms of the difference over rms of the row"""
    d = got.detach().cpu().double() - want
    return float((d.pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt()).max())


def model_tol(cfg, w, toks, dtype):
    """float32: a fixed bound.  bf16: three times the worst row of the oracle with 16-bit tensors between its exact operations."""
    if dtype == f32:
        return 5e-5
    return 3 * max(logit_err(O.forward(cfg, w, t, cast=O.to_bf16), O.forward(cfg, w, t)) for t in toks)


# ------------------------------------------------------------------------------------------ mechanisms
def case_dyt_stream(dev, dtype, T=7, D=40):
    from aria_amd import ops
    from aria_amd.layers import DynamicTanh

    mk = lambda s: DynamicTanh(torch.tensor(0.3 + 0.4 * s), rnd(D, seed=10 + s), rnd(D, seed=20 + s), D).to(dev)  # noqa: E731
    post, nxt = mk(1), mk(2)

    def want(n, x):
        return O.dynamic_tanh(x, n.alpha, n.weight.cpu().double(), n.bias.cpu().double())

    table, ids = rnd(11, D, seed=1, dtype=dtype).to(dev), torch.tensor([3, 0, 10, 3, 7, 1, 9][:T], dtype=torch.int32)
    x = torch.empty(T, D, device=dev)
    h = ops.dyt_stream(x, None, nxt.params(), ids=ids.to(dev), table=table)
    x0 = table.cpu().double()[ids.long()]
    assert torch.equal(x.cpu().double(), x0)
    assert rel(h, want(nxt, x0)) < (2e-6 if dtype == f32 else 3e-3)
    y = rnd(T, D, seed=5, scale=3, dtype=dtype)
    h = ops.dyt_stream(x, post.params(), nxt.params(), y=y.to(dev))
    x1 = x0 + want(post, y.double())
    assert rel(x, x1) < 2e-6                                   # the stream itself stays 32-bit in both forms
    assert rel(h, want(nxt, x1)) < (2e-6 if dtype == f32 else 3e-3)
    k = 3
    eo, wts = rnd(T * k, D, seed=6, dtype=dtype), torch.rand(T, k, generator=gen(8))
    inv = torch.randperm(T * k, generator=gen(9)).to(torch.int32)
    h = ops.dyt_stream(x, post.params(), None, y=eo.to(dev), inv=inv.to(dev), weights=wts.to(dev))
    mix = (eo.double()[inv.long()].view(T, k, D) * wts.double()[..., None]).sum(1)
    assert h is None and rel(x, x1 + want(post, mix)) < 2e-6
    # saturation: large arguments give +-w + b, not NaN
    ops.dyt_stream(x, post.params(), nxt.params(), y=torch.full((T, D), 3e4, dtype=dtype, device=dev))
    assert bool(torch.isfinite(x).all())


def case_activations(dev, dtype):
    from aria_amd import ops

    u, g = rnd(5, 24, seed=1, scale=2, dtype=dtype), rnd(5, 24, seed=2, scale=2, dtype=dtype)
    tol = 2e-6 if dtype == f32 else 3e-3
    assert rel(ops.act_rows(u.to(dev)), O.relu_squared(u.double())) < tol
    assert rel(ops.act_rows(u.to(dev), gate=g.to(dev)), O.silu(g.double()) * u.double()) < tol


def case_gemm_relu_squared(dev, M, N, K):
    """The activation in the GEMM epilogue equals the GEMM followed by the elementwise pass, bit for bit."""
    from aria_amd import ops

    a, w = rnd(M, K, seed=3).to(dev), rnd(N, K, seed=4, scale=0.3).to(dev)
    got = ops.linear_any(a, w, relu_squared=True)
    assert torch.equal(got, ops.act_rows(ops.gemm(a, w)))
    assert rel(got, O.relu_squared(a.cpu().double() @ w.cpu().double().T)) < 1e-2


def case_gemm_f32(dev, M, N, K):
    from aria_amd import ops

    a, w = rnd(M, K, seed=1, dtype=f32), rnd(N, K, seed=2, dtype=f32)
    assert rel(ops.linear_any(a.to(dev), w.to(dev)), a.double() @ w.double().T) < 2e-6
    counts = [M // 3, 0, M - M // 3]
    we = rnd(3, N, K, seed=3, dtype=f32)
    off = torch.tensor([0, counts[0], counts[0], M], dtype=torch.int32, device=dev)
    want = torch.cat([a.double()[:counts[0]] @ we.double()[0].T, a.double()[counts[0]:] @ we.double()[2].T])
    assert rel(ops.grouped_linear_any(a.to(dev), we.to(dev), off), want) < 2e-6


def case_route_groups(dev, T, E, groups, keep, k):
    from aria_amd import ops

    ldl = (E + 7) // 8 * 8
    logits = torch.randn(T, ldl, generator=gen(E + k))
    # negative choice scores (a large negative correction) must still beat experts outside the kept groups
    corr = torch.randn(E, generator=gen(3)) * 0.4 - 1.0
    w, idx, counts = ops.moe_route_groups(logits.to(dev), corr.to(dev), groups, keep, k)
    s = torch.sigmoid(logits[:, :E].double())
    hist = torch.zeros(E, dtype=torch.int64)
    for t in range(T):
        want = O.choose_experts(s[t] + corr.double(), groups, keep, k)
        assert idx[t].tolist() == want, (t, idx[t].tolist(), want)
        assert rel(w[t], s[t][want]) < 1e-6
        hist[want] += 1
    assert torch.equal(counts.cpu().long(), hist)


def case_sort_wide(dev, T=40, E=100, k=3):
    from aria_amd import ops

    idx = torch.stack([torch.randperm(E, generator=gen(t))[:k] for t in range(T)]).to(torch.int32)
    counts = torch.bincount(idx.flatten().long(), minlength=E).to(torch.int32)
    off, src, inv = (x.cpu() for x in ops.moe_sort(idx.to(dev), counts.to(dev)))
    want = torch.sort(idx.flatten().long(), stable=True).indices
    assert torch.equal(src.long(), want) and torch.equal(off[1:].long(), counts.long().cumsum(0)) and off[0] == 0
    assert torch.equal(inv.long()[want], torch.arange(T * k))


def _attn(m, dev, dtype, D=32, seed=0, w=None):
    from aria_amd.layers import LatentAttention

    H, qd, R = m["heads"], m["dim"] + m["rot_dim"], m["kv_rank"]
    w = w or {"q": rnd(H * qd, D, seed=seed, scale=2 * D ** -0.5), "dkv": rnd(R + m["rot_dim"], D, seed=seed + 1, scale=2 * D ** -0.5),
              "dkv.norm": (1 + 0.3 * rnd(R, seed=seed + 2).float()).to(bf16), "uk": rnd(H * m["dim"], R, seed=seed + 3, scale=R ** -0.5),
              "uv": rnd(H * m["vdim"], R, seed=seed + 4, scale=R ** -0.5), "g": rnd(H, D, seed=seed + 5, scale=2 * D ** -0.5),
              "o": rnd(D, H * m["vdim"], seed=seed + 6, scale=(H * m["vdim"]) ** -0.5)}
    mod = LatentAttention(w, heads=H, dim=m["dim"], rot_dim=m["rot_dim"], vdim=m["vdim"], kv_rank=R, scale=m["scale"], rot_dims=m["rot"]["dims"],
                          rot_base=m["rot"]["base"], eps=1e-5, width=D, dtype=dtype).to(dev)
    return mod, {"m." + k: v for k, v in w.items()}


def case_latent_attention(dev, dtype, m, lens, tail=3, D=32):
    """The mixer alone: packed prompts of unequal lengths, then single tokens, against the oracle of each sequence by itself."""
    from aria_amd.layers import rotation_table
    from aria_amd.serving import StepBatch

    mod, w = _attn(m, dev, dtype, D)
    B, cap = len(lens), max(lens) + tail + 5
    cache = mod.new_cache(B + 1, cap, dev)
    cache.rows.fill_(float("nan"))                       # rows no sequence has written are never read
    rope = rotation_table(cap, m["rot"]["dims"], m["rot"]["base"], dev)
    hs = [rnd(n + tail, D, seed=40 + i) for i, n in enumerate(lens)]
    want = [O.latent_attention(h.double(), {k: v.double() for k, v in w.items()}, "m", m, 1e-5) for h in hs]
    slots = list(range(B, 0, -1))
    tol = TOL[dtype] if dtype == f32 else 2e-2
    b = StepBatch.build([[0] * n for n in lens], slots, [0] * B, None, dev)
    got = mod(torch.cat([h[:n] for h, n in zip(hs, lens)]).to(dtype).to(dev), b, cache, rope)
    assert rel(got, torch.cat([x[:n] for x, n in zip(want, lens)])) < tol
    for s in range(tail):
        b = StepBatch.build([[0]] * B, slots, [n + s for n in lens], None, dev)
        got = mod(torch.stack([h[n + s] for h, n in zip(hs, lens)]).to(dtype).to(dev), b, cache, rope)
        assert rel(got, torch.stack([x[n + s] for x, n in zip(want, lens)])) < tol, s


def case_one_key_stands_out(dev, dtype, positions, n):
    """Every query is pointed at ONE earlier row (its latent is scaled to dominate the scores): the output is that row's value alone, wherever the
    row lies -- far away, on either side of the 64-row tiles, the first rows, the query's own row -- in prompts and in decoding."""
    from aria_amd.layers import rotation_table
    from aria_amd.serving import StepBatch

    R, D = 64, 64
    m = dict(heads=1, dim=R, rot_dim=2, vdim=R, kv_rank=R, scale=3.0, rot=dict(base=100.0, dims=2))
    eye = torch.eye(R).to(bf16)
    z = lambda *s: torch.zeros(*s, dtype=bf16)  # noqa: E731
    # input row = [latent direction (32) | query direction (32)]
    q, dkv = z(R + 2, D), z(R + 2, D)
    q[:32, 32:] = torch.eye(32).to(bf16)
    dkv[:32, :32] = torch.eye(32).to(bf16)
    w = {"q": q, "dkv": dkv, "dkv.norm": torch.ones(R, dtype=bf16), "uk": eye, "uv": eye, "g": torch.cat([z(1, D - 1), z(1, 1) + 4], 1), "o": eye.clone()}
    mod, wo = _attn(m, dev, dtype, D, w=w)
    cap = n + 8
    rope = rotation_table(cap, 2, 100.0, dev)
    for far in positions:
        h = rnd(n, D, seed=far + 1, scale=0.3)
        h[:, 31] = 0
        h[far, :32] = 0
        h[far, 31] = 1                                   # the only row with this latent direction ...
        h[:, 32:] = 0
        h[:, 63] = 1                                     # ... and every query asks for it
        want = O.latent_attention(h.double(), {k: v.double() for k, v in wo.items()}, "m", m, 1e-5)
        assert far + 1 >= n or float(want[far + 1:, 31].min()) > 0.9 * float(want[far, 31])   # the case does what it says
        cache = mod.new_cache(1, cap, dev)
        cut = max(1, n - 4)
        b = StepBatch.build([[0] * cut], [0], [0], None, dev)
        got = [mod(h[:cut].to(dtype).to(dev), b, cache, rope)]
        for p in range(cut, n):
            b = StepBatch.build([[0]], [0], [p], None, dev)
            got.append(mod(h[p:p + 1].to(dtype).to(dev), b, cache, rope))
        got = torch.cat(got).cpu().double()
        err = (got - want).abs().amax(-1)
        assert float(err.max()) < (1e-3 if dtype == f32 else 0.12), (far, int(err.argmax()), float(err.max()))


def case_splits_agree(dev, T=3, n=300):
    """The matrix-pipe decode kernel over any number of splits (more splits than tiles included) against the any-size kernel."""
    import ctypes

    from aria_amd import hip, ops

    for H, R, dr in ((3, 48, 8), (20, 200, 24), (16, 512, 64)):
        cw = (R + dr + 63) // 64 * 64
        s = hip.LatentShape(H=H, dn=8, dr=dr, dv=8, R=R, rot=dr, dq=8 + dr, dvp=8, cw=cw, rp=(R + 7) // 8 * 8, ldp=H * (8 + dr) + R + dr + 64, kv_off=H * (8 + dr),
                            g_off=H * (8 + dr) + R + dr, S_cap=n + 20, scale=0.7 * (R + dr) ** -0.5, eps=1e-5)
        s.ldp = (s.g_off + H + 7) // 8 * 8
        qa = rnd(T, H, cw, seed=1)
        qa[..., R + dr:] = 0
        cache = rnd(2, n + 20, cw, seed=2)
        cache[..., R + dr:] = 0
        pos = torch.tensor([n - 1, 0, 64][:T], dtype=torch.int32)
        slot = torch.tensor([1, 0, 1][:T], dtype=torch.int32)
        outs = []
        for splits in (1, 2, 5, 7):
            po, ml = torch.full((T, splits, H, R), float("nan"), device=dev), torch.empty(T, splits, H, 2, device=dev)
            dv = [t.to(dev).contiguous() for t in (qa, cache, slot, pos)]
            hip.get_lib().call("aria_latent_attn", *(t.data_ptr() for t in dv[:2]), ctypes.byref(s), dv[2].data_ptr(), dv[3].data_ptr(), po.data_ptr(),
                               ml.data_ptr(), T, splits, 0, ops._stream(po))
            m, l = ml[..., 0].cpu().double(), ml[..., 1].cpu().double()
            f = torch.where(l > 0, torch.exp2(m - m.amax(1, keepdim=True)), torch.zeros_like(l))
            o = torch.where((l > 0)[..., None], po.cpu().double(), torch.zeros(1, dtype=torch.float64))
            outs.append((o * f[..., None]).sum(1) / (l * f).sum(1)[..., None])
        for t in range(T):
            k = cache[int(slot[t]), :int(pos[t]) + 1].double()
            p = torch.softmax(qa[t].double() @ k.T * s.scale, -1)
            for o in outs:
                assert rel(o[t], p @ k[:, :R]) < 6e-3


# ------------------------------------------------------------------------------------------ the model
def case_model(dev, dtype, name, lens=(9, 1, 17), tail=4):
    """A batch of unequal requests -- prompt, then tokens one by one, one request ending early -- against the oracle of each request alone; the slots
    are then used again by another batch."""
    from aria_amd.serving import Scheduler

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=len(name))
    m = build(cfg, w, dev, dtype)
    sched = Scheduler(m, max(lens) + tail + 3)
    for round_ in range(2):
        toks = [clear_tokens(cfg, w, n + tail, seed=i + 10 * round_) for i, n in enumerate(lens)]
        want = [O.forward(cfg, w, t) for t in toks]
        ids = [f"r{round_}{i}" for i in range(len(lens))]
        got = sched.step(ids, [t[:n] for t, n in zip(toks, lens)], [list(range(n)) for n in lens])
        worst = logit_err(got, torch.cat([x[:n] for x, n in zip(want, lens)]))
        live = list(range(len(lens)))
        for s in range(tail):
            got = sched.step([ids[i] for i in live], [[toks[i][lens[i] + s]] for i in live])
            worst = max(worst, logit_err(got, torch.stack([want[i][lens[i] + s] for i in live])))
            if s == 1:
                sched.finish(ids[live.pop(1)])
        assert worst < model_tol(cfg, w, toks, dtype), worst
        for i in live:
            sched.finish(ids[i])
        assert not sched.live and sorted(sched.free) == list(range(len(lens)))


def case_portions(dev, dtype, name="mixed", n=19):
    """One prompt whole, token by token, and in portions of several sizes down to two tokens: the same logits at every position."""
    from aria_amd.serving import Scheduler

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=3)
    m, toks = build(cfg, w, dev, dtype), clear_tokens(cfg, w, n, seed=5)
    want = O.forward(cfg, w, toks)
    for sizes in ([n], [1] * n, [2] * (n // 2) + [n % 2], [7, 2, 5, n - 14], [n - 3, 2, 1], [1, n - 1]):
        sched, at, got = Scheduler(m, n + 2), 0, []
        for k in [s for s in sizes if s]:
            got.append(sched.step(["a"], [toks[at:at + k]], [list(range(k))]).cpu())
            at += k
        assert logit_err(torch.cat(got), want) < model_tol(cfg, w, [toks], dtype), sizes


def case_continuation_beside_decode(dev, dtype, name="equal"):
    """A step that carries a portion of one request and single tokens of others."""
    from aria_amd.serving import Scheduler

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=4)
    m = build(cfg, w, dev, dtype)
    a, b = clear_tokens(cfg, w, 14, seed=1), clear_tokens(cfg, w, 6, seed=2)
    sched = Scheduler(m, 20)
    sched.step(["a", "b"], [a[:5], b[:4]], [[], []])
    g1 = sched.step(["b", "a"], [[b[4]], a[5:13]], [[0], list(range(8))])
    g2 = sched.step(["a", "b"], [[a[13]], [b[5]]])
    wa, wb = O.forward(cfg, w, a), O.forward(cfg, w, b)
    tol = model_tol(cfg, w, [a, b], dtype)
    assert logit_err(g1, torch.cat([wb[4:5], wa[5:13]])) < tol
    assert logit_err(g2, torch.stack([wa[13], wb[5]])) < tol


def case_rows_do_not_depend_on_company(dev, dtype, name="mixed", n=11):
    """Logits of one request alone, in a batch of 5 and in a batch past the one-call decode limit, on different slots."""
    from aria_amd import duguzen
    from aria_amd.serving import Scheduler

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=6)
    m = build(cfg, w, dev, dtype)
    toks = clear_tokens(cfg, w, n, seed=1)
    res = []
    for company in (0, 4, duguzen.DECODE_ROWS + 1):
        sched = Scheduler(m, n + 1)
        ids = [f"x{i}" for i in range(company)] + ["a"]
        ps = [tokens(cfg, 1 + i % 7, seed=20 + i) for i in range(company)]
        got = [sched.step(ids, ps + [toks[:n - 2]])[-1]]
        for s in (n - 2, n - 1):
            got.append(sched.step(ids, [[1 + i] for i in range(company)] + [[toks[s]]])[-1])
        res.append(torch.stack(got).cpu().double())
    for r in res[1:]:
        assert logit_err(r, res[0]) < model_tol(cfg, w, [toks], dtype) * (0.1 if dtype == f32 else 1)


def case_borrowed_layers_keep_their_own_cache(dev, dtype):
    """Two runs of one layer's weights cache different rows; and the borrowed stack equals one with the tensors copied out."""
    from aria_amd.serving import Scheduler

    mix, ff = mixer(heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=16), dense(ff=16)
    shared, plain = config([(mix, ff), (mix, ff, 0)], width=24, vocab=40), config([(mix, ff), (mix, ff)], width=24, vocab=40)
    w = checkpoint(shared, seed=2)
    w2 = dict(w, **{"l1." + k[3:]: v for k, v in w.items() if k.startswith("l0.")})
    toks, out = tokens(shared, 9), []
    for cfg, ww in ((shared, w), (plain, w2)):
        m = build(cfg, ww, dev, dtype)
        s = Scheduler(m, 12)
        s.step(["a"], [toks[:6]], [[]])
        out.append(torch.cat([s.step(["a"], [[t]]) for t in toks[6:]]))
        assert not torch.equal(m.caches[0].rows, m.caches[1].rows)
    assert torch.equal(out[0], out[1])


def case_stream_after_every_layer(dev, dtype, name="mixed", n=6):
    from aria_amd.serving import StepBatch

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=9)
    m, toks = build(cfg, w, dev, dtype), clear_tokens(cfg, w, n)
    want = O.forward(cfg, w, toks, want_layers=True)[1]
    m.setup_caches(1, n)
    trace = []
    m.step(StepBatch.build([toks], [0], [0], None, dev), trace)
    assert len(trace) == len(cfg["layers"])
    for got, x in zip(trace, want):
        assert got.dtype == f32 and rel(got[:, :cfg["width"]], x) < (1e-5 if dtype == f32 else 3e-2)


def case_greedy_generation(dev, dtype, name="sharp", n_new=6, tmp=None):
    """Greedy tokens through serving.generate (registry, loader, scheduler, sampling) equal the oracle's argmax chain wherever that is not a tie."""
    import json

    from safetensors.torch import save_file

    from aria_amd import registry, serving

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=12)
    (tmp / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp / "model.safetensors"))
    m = registry.load_model(str(tmp), dev, dtype)
    prompts = [tokens(cfg, n, seed=n) for n in (5, 1, 8)]
    got = serving.generate(m, prompts, n_new, temperature=0, max_batch=2)
    close = 1e-3 if dtype == f32 else 0.15
    for p, g in zip(prompts, got):
        assert len(g) == n_new
        logits = O.forward(cfg, w, p + g)
        for i, t in enumerate(g):
            row = logits[len(p) + i - 1]
            assert float(row.max() - row[t]) <= close * float(row.std()), (i, t, int(row.argmax()))
    stop = got[0][2]
    again = serving.generate(m, prompts, n_new, temperature=0, stop_token=stop)
    for g, a in zip(got, again):
        cut = g.index(stop) + 1 if stop in g else n_new
        assert len(a) == cut and (dtype != f32 or a == g[:cut])
    sampled = serving.generate(m, prompts[:2], 4, temperature=1.0, top_k=5)
    assert all(0 <= t < cfg["vocab"] for s in sampled for t in s) and [len(s) for s in sampled] == [4, 4]


def case_long_decode(dev, dtype, prompt=3, steps=150, name="sharp"):
    """Many single tokens after a short prompt: positions well past several cache tiles, against the oracle at every step."""
    from aria_amd.serving import Scheduler

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=13)
    m, toks = build(cfg, w, dev, dtype), tokens(cfg, prompt + steps, seed=3)
    want = O.forward(cfg, w, toks)
    s = Scheduler(m, prompt + steps)
    got = [s.step(["a"], [toks[:prompt]], [[prompt - 1]])]
    for t in toks[prompt:]:
        got.append(s.step(["a"], [[t]]))
    assert logit_err(torch.cat(got), want[prompt - 1:]) < model_tol(cfg, w, [toks], dtype)


def case_graph_replay(dev, name="mixed", n=70, steps=3):
    """The one-call decode step captured into a HIP graph: every replay, with eager work between, equals the eager step bit for bit."""
    from aria_amd.serving import Scheduler, StepBatch

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=6)
    m = build(cfg, w, dev, bf16)
    toks = clear_tokens(cfg, w, n, seed=1)
    s = Scheduler(m, n + 8)
    s.step(["a"], [toks[:n - steps]])
    eager = [s.step(["a"], [[t]]).clone() for t in toks[n - steps:]]
    b = StepBatch.build([[toks[n - steps]]], [0], [n - 1], None, dev)   # (max_len fixes the launch shapes for every replay)
    ids, pos = b.ids.clone(), torch.tensor([n - steps], dtype=torch.int32, device=dev)
    b.ids, b.pos = ids, pos
    side = torch.cuda.Stream()
    side.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(side):
        m.step(b)
    torch.cuda.current_stream().wait_stream(side)
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        out = m.step(b)
    for r in range(2):
        for j in range(steps):
            ids.fill_(toks[n - steps + j])
            pos.fill_(n - steps + j)
            g.replay()
            torch.cuda.synchronize()
            assert logit_err(out, eager[j].cpu().double()) < 1e-2, (r, j)
            torch.randn(1 << 16, device=dev).sum().item()


def case_bad_inputs(dev):
    import pytest

    from aria_amd.duguzen import DuguzenConfig
    from aria_amd.serving import Scheduler

    cfg = CONFIGS["equal"]
    m = build(cfg, checkpoint(cfg), dev, f32)
    s = Scheduler(m, 8)
    with pytest.raises(ValueError):
        s.step(["a"], [list(range(9))])
    with pytest.raises(ValueError):
        s.step(["a"], [[]])
    s.step(["a"], [[1, 2]])
    with pytest.raises(RuntimeError):
        s.step(["b"], [[1]])
    for bad in (dict(cfg, layers=[dict(cfg["layers"][0], type="other")]), dict(cfg, layers=[dict(cfg["layers"][0], weights_of=3)]),
                dict(cfg, layers=[cfg["layers"][0], dict(cfg["layers"][0], weights_of=0, mlp=None)])):
        with pytest.raises(ValueError):
            DuguzenConfig.from_dict(bad)
    assert math.isclose(DuguzenConfig.from_dict(cfg).eps, cfg["norm"]["eps"])
    one = cfg["layers"][0]
    chain = DuguzenConfig.from_dict(dict(cfg, layers=[dict(one, weights_of=2), dict(one, weights_of=0), one]))
    assert [l.source for l in chain.layers] == [2, 2, 2]
    with pytest.raises(ValueError):
        DuguzenConfig.from_dict(dict(cfg, layers=[dict(one, weights_of=1), dict(one, weights_of=0)]))
