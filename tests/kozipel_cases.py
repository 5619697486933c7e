"""Cases of chunk-local attention, linear attention, the RMS-normed stream and Kozipel end to end, shared by the emulator tests
(tests/test_emu_kozipel.py, CPU) and the hardware tests (tests/test_gpu_kozipel.py).  Everything is compared with oracle/kozipel_oracle.py in float64 on
configurations and weights made here."""
import json

import torch

from oracle import kozipel_oracle as O
from tests.latent_cases import gen, logit_err, rel, rnd, tokens

bf16, f32 = torch.bfloat16, torch.float32
EPS = 1e-5


# ------------------------------------------------------------------------------------------ configurations and weights made up here
def left(heads=4, kv_heads=2, dim=24, vdim=40, size=13, scale=None):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=size), scale=scale or dim ** -0.5)


def right(heads=2, dim=16, vdim=24, tau=8.0):
    return dict(heads=heads, dim=dim, vdim=vdim, tau=tau)


def parallel(lf=None, rt=None, ff=56):
    return dict(type="parallel", mixer=dict(left=lf or left(), right=rt or right()), mlp=dict(kind="dense", ff=ff) if ff else None)


def lightning(heads=3, dim=16, vdim=8, decay=(0.5, 0.9, 0.995), ff=40):
    return dict(type="lightning", mixer=dict(heads=heads, dim=dim, vdim=vdim, decay=list(decay)), mlp=dict(kind="dense", ff=ff) if ff else None)


def config(layers, width=48, vocab=90, eps=EPS, loop=None, scale=2.0, mult=0.5, cap=12.0):
    return dict(architecture="Kozipel", width=width, vocab=vocab, norm=dict(eps=eps), embedding=dict(scale=scale), residual_mult=mult, logit_softcap=cap,
                layers=layers, **({"loop": loop} if loop else {}))


def left_weights(t, p, m, D, sharp=2.0):
    t(p + "q", m["heads"] * m["dim"], D, scale=sharp * D ** -0.5)
    t(p + "k", m["kv_heads"] * m["dim"], D, scale=sharp * D ** -0.5)
    t(p + "v", m["kv_heads"] * m["vdim"], D, scale=D ** -0.5)
    t(p + "o", D, m["heads"] * m["vdim"], scale=(m["heads"] * m["vdim"]) ** -0.5)


def linear_weights(t, w, g, p, m, D, rank=5):
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    for n, r in (("q", d), ("k", d), ("v", dv), ("g", dv)):
        t(p + n, H * r, D, scale=1.5 * D ** -0.5)
    w[p + "k"] = (0.7 * w[p + "k"].float() + 0.7 * w[p + "q"].float()).to(bf16)   # (keys like queries: an output of nearly nothing would be normed up)
    t(p + "o", D, H * dv, scale=(H * dv) ** -0.5)
    w[p + "norm"] = (1 + 0.3 * torch.randn(dv if "tau" in m else H * dv, generator=g)).to(bf16)
    if "tau" in m:
        t(p + "a1", rank, D, scale=D ** -0.5)
        t(p + "a2", H * d, rank, scale=1.5 * rank ** -0.5)
        t(p + "a2.b", H * d, scale=1.0)


def checkpoint(cfg, seed=0):
    """Random weights under the checkpoint's names."""
    g = gen(seed)
    D, w = cfg["width"], {}

    def t(name, *shape, scale=1.0):
        w[name] = (torch.randn(*shape, generator=g) * scale).to(bf16)

    t("embed", cfg["vocab"], D)
    t("head", cfg["vocab"], D, scale=2 * D ** -0.5)
    t("final.norm", D, scale=0.3)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        t(p + "norm1", D, scale=0.3)
        if L["type"] == "lightning":
            linear_weights(t, w, g, p + "mix.", m, D)
        else:
            left_weights(t, p + "mix.left.", m["left"], D)
            linear_weights(t, w, g, p + "mix.right.", m["right"], D, rank=3 + 2 * i)
            for side in ("left", "right"):
                w[p + f"mix.{side}.out"] = (1 + 0.3 * torch.randn(D, generator=g)).to(bf16)
        if L["mlp"]:
            t(p + "norm2", D, scale=0.3)
            for n in ("gate", "up"):
                t(p + f"mlp.{n}", L["mlp"]["ff"], D, scale=1.5 * D ** -0.5)
            t(p + "mlp.down", D, L["mlp"]["ff"], scale=L["mlp"]["ff"] ** -0.5)
    return w


CONFIGS = {
    # both kinds, unequal sizes, a span that runs three times, one layer without feed-forward
    "mixed": config([lightning(), parallel(), parallel(left(heads=3, kv_heads=1, dim=16, vdim=8, size=7), right(heads=3, dim=24, vdim=8, tau=2.0), ff=0),
                     lightning(heads=1, dim=24, vdim=40, decay=(0.9,), ff=24)], loop=dict(start=1, stop=3, times=3)),
    # sizes that are no multiple of 8, everything that can be 1 is 1, no loop
    "odd": config([parallel(left(heads=3, kv_heads=3, dim=13, vdim=11, size=5), right(heads=1, dim=7, vdim=9, tau=1.0), ff=13),
                   lightning(heads=2, dim=5, vdim=3, decay=(1.0, 0.7), ff=9)], width=37, vocab=51, eps=1e-3, scale=1.0, mult=1.0, cap=30.0),
    # chunks of one token, a loop over the whole stack, a loop of one layer at the end
    "ones": config([parallel(left(heads=1, kv_heads=1, dim=8, vdim=8, size=1), right(heads=1, dim=8, vdim=8)), lightning(heads=1, dim=8, vdim=8, decay=(0.8,))],
                   width=24, vocab=40, loop=dict(start=0, stop=2, times=2)),
    "last": config([lightning(), parallel()], width=40, loop=dict(start=1, stop=2, times=2)),
    # wide heads: every matrix-pipe instantiation, fused gate / up shape (ff % 128 == 0, width % 64 == 0)
    "wide": config([parallel(left(heads=8, kv_heads=2, dim=96, vdim=128, size=100), right(heads=2, dim=136, vdim=160, tau=16.0), ff=128),
                    lightning(heads=2, dim=72, vdim=64, decay=(0.62, 0.999), ff=256)], width=128, vocab=130),
    # wider than every matrix-pipe form
    "huge": config([parallel(left(heads=2, kv_heads=1, dim=264, vdim=24, size=9), right(heads=1, dim=260, vdim=16))], width=32, vocab=40),
    # more query heads per key head than one group of 16, strong and weak decays: blocks whose state forgets everything
    "steep": config([parallel(left(heads=20, kv_heads=1, dim=16, vdim=16, size=70), right(heads=2, dim=16, vdim=16, tau=0.05)),
                     lightning(heads=3, dim=8, vdim=8, decay=(0.0, 0.001, 1.0))], width=40, vocab=64),
    # heads for whole state lines a workgroup in a batch of 16
    "many": config([lightning(heads=16, dim=72, vdim=64, decay=[0.6 + 0.025 * i for i in range(16)], ff=24),
                    parallel(left(heads=16, kv_heads=4, dim=8, vdim=8, size=9), right(heads=16, dim=24, vdim=40, tau=4.0), ff=24)], width=64, vocab=60),
    # a head of more than 16384 rows, and a reduction of several rounds of the decode kernels' waves
    "vocabulary": config([lightning(heads=1, dim=8, vdim=8, decay=(0.9,), ff=24)], width=24, vocab=16411),
    "broad": config([parallel(ff=24)], width=2061, vocab=45),
}


def build(cfg, w, dev, dtype):
    from aria_amd.kozipel import KozipelForCausalLM

    return KozipelForCausalLM.from_tensors(cfg, w, dev, dtype)


def model_tol(cfg, w, toks, dtype):
    """float32: a fixed bound.  bf16: three times the worst row of the oracle with 16-bit tensors between its exact operations."""
    if dtype == f32:
        return 5e-5
    return 3 * max(logit_err(O.forward(cfg, w, t, cast=O.to_bf16), O.forward(cfg, w, t)) for t in toks)


# ------------------------------------------------------------------------------------------ mechanisms
def case_rms_stream(dev, dtype, T=5, n=37, D=40):
    from aria_amd import ops

    def pad(x):
        return torch.cat([x, torch.zeros(*x.shape[:-1], D - n, dtype=x.dtype)], -1)

    def want_norm(x, w):
        return O.rms(x[..., :n], 1e-3) * w[:n].double()

    tol = 2e-6 if dtype == f32 else 3e-3
    table, ids = pad(rnd(11, n, seed=1, dtype=dtype)), torch.tensor([3, 0, 10, 3, 7], dtype=torch.int32)[:T]
    w1, w2, w3 = (pad(rnd(n, seed=s, dtype=f32)) for s in (2, 3, 4))
    x = torch.full((T, D), float("nan"), device=dev)      # the first pass does not read the stream
    kw = dict(ids=ids.to(dev), table=table.to(dev))
    h = ops.rms_stream(x, n, 1e-3, w1.to(dev), scale=2.5, **kw)
    emb = 2.5 * table.double()[ids.long()]
    assert rel(x, emb) < 1e-7 and rel(h[:, :n], want_norm(emb, w1)) < tol and not h[:, n:].any()
    y, y2 = (pad(rnd(T, n, seed=s, scale=3, dtype=dtype)) for s in (5, 6))
    h = ops.rms_stream(x, n, 1e-3, w2.to(dev), y=y.to(dev), mult=0.3)
    x1 = emb + 0.3 * y.double()
    assert rel(x, x1) < 2e-6 and rel(h[:, :n], want_norm(x1, w2)) < tol
    pair = pad(0.5 * (want_norm(y.double(), w2) + want_norm(y2.double(), w3)))
    h = ops.rms_stream(x, n, 1e-3, w1.to(dev), y=y.to(dev), mult=0.7, pair=(y2.to(dev), w2.to(dev), w3.to(dev)), scale=1.5, **kw)   # + the embedding again
    x2 = x1 + 0.7 * pair + 1.5 * table.double()[ids.long()]
    assert rel(x, x2) < 2e-6 and rel(h[:, :n], want_norm(x2, w1)) < tol and not x[:, n:].any()
    assert ops.rms_stream(x, n, 1e-3, None, y=y.to(dev)) is None
    z = torch.zeros(T, D, dtype=dtype, device=dev)       # eps lies inside the root
    tiny = torch.full((T, D), 1e-3, device=dev)
    h = ops.rms_stream(tiny, D, 1e-3, torch.ones(D, device=dev), y=z)
    assert rel(h, torch.full((T, D), 1e-3 / (1e-6 + 1e-3) ** 0.5).double()) < (2e-6 if dtype == f32 else 4e-3)


def case_softcap_and_relu_gate(dev, dtype):
    from aria_amd import ops

    x = rnd(3, 33, seed=1, scale=40, dtype=f32)
    assert rel(ops.softcap_(x.clone().to(dev), 15.0), 15 * torch.tanh(x.double() / 15)) < 2e-6
    gu = rnd(5, 48, seed=2, scale=2, dtype=dtype)
    got = ops.act_rows(gu.to(dev)[:, 24:], gate=gu.to(dev)[:, :24], relu=True)
    assert rel(got, gu[:, :24].double().clamp_min(0) * gu[:, 24:].double()) < (1e-6 if dtype == f32 else 3e-3)


def case_relu_glu(dev, M, ff, K):
    """The one-launch gated pair against GEMM + elementwise pass (both round gate and up to bf16 first; a long GEMM may sum in another order)."""
    from aria_amd import ops

    x, w = rnd(M, K, seed=1).to(dev), rnd(2 * ff, K, seed=2, scale=K ** -0.5).to(dev)
    got, gu = ops.relu_glu(x, w), ops.gemm(x, w)
    assert rel(got, ops.act_rows(gu[:, ff:], gate=gu[:, :ff], relu=True).cpu().double()) < (1e-7 if K < 1024 else 2e-3)
    y = x.cpu().double() @ w.cpu().double().T
    assert rel(got, y[:, :ff].clamp_min(0) * y[:, ff:]) < 1e-2


def case_norm_gate(dev, dtype, T=5):
    from aria_amd import ops

    for groups, cols, n, shared, silu in ((3, 24, 21, True, True), (1, 72, 63, False, False), (2, 520, 520, True, False)):
        o, gate = rnd(T, groups * cols, seed=1, dtype=dtype), rnd(T, groups * cols + 16, seed=2, scale=2, dtype=dtype)
        o.view(T, groups, cols)[..., n:] = 0
        w = rnd(cols if shared else groups * cols, seed=3, dtype=f32)
        got = ops.norm_gate(o.to(dev), gate.to(dev)[:, 8:8 + groups * cols], w.to(dev), groups, n, 1e-3, silu)
        v = o.double().view(T, groups, cols)
        v = v / torch.sqrt((v * v).sum(-1, keepdim=True) / n + 1e-3) * w.double().view(-1 if shared else groups, cols if shared else cols)
        g = gate[:, 8:8 + groups * cols].double()
        want = v.view(T, -1) * (O.silu(g) if silu else O.sigmoid(g))
        assert rel(got, want) < (2e-6 if dtype == f32 else 4e-3)


def _mixer(kind, m, dev, dtype, D, seed=0, w=None, rank=5):
    from aria_amd.layers import ChunkAttention, LinearAttention, MixerGroup

    if w is None:
        w, g = {}, gen(seed)

        def t(name, *shape, scale=1.0):
            w[name] = (torch.randn(*shape, generator=g) * scale).to(bf16)

        left_weights(t, "", m, D) if kind == "chunk" else linear_weights(t, w, g, "", m, D, rank)
    if kind == "chunk":
        part = ChunkAttention(w, heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], size=m["mask"]["size"], scale=m["scale"], width=D, dtype=dtype)
    elif kind == "gated":
        part = LinearAttention(w, heads=m["heads"], dim=m["dim"], vdim=m["vdim"], tau=m["tau"], q_scale=m["dim"] ** -0.5, eps=EPS, width=D, dtype=dtype)
    else:
        part = LinearAttention(w, heads=m["heads"], dim=m["dim"], vdim=m["vdim"], decay=m["decay"], silu_inputs=True, norm_heads=False, gate="sigmoid", eps=EPS,
                               width=D, dtype=dtype)
    oracle = {"chunk": O.chunked_mixer, "gated": O.gated_linear_mixer, "lightning": O.lightning_mixer}[kind]
    wd = {"m." + k: v.double() for k, v in w.items()}

    def want(h, cast=O.exact):
        return oracle(h.double(), wd, "m", m, *(() if kind == "chunk" else (EPS,)), cast)

    return MixerGroup([part], D, dtype=dtype).to(dev), want


def case_mixer(dev, dtype, kind, m, lens, tail=3, D=32, portion=()):
    """A mixer alone: packed prompts of unequal lengths, portions of all of them, then single tokens, against the oracle of each sequence by itself.  What
    no sequence has written is NaN: it must not be read."""
    from aria_amd.serving import StepBatch

    group, want = _mixer(kind, m, dev, dtype, D)
    total = tail + sum(portion)
    B, cap = len(lens), max(lens) + total
    caches = group.new_cache(B + 1, (cap + 7) // 8 * 8, dev)
    caches[0].rows.fill_(float("nan"))
    hs = [rnd(n + total, D, seed=40 + i) for i, n in enumerate(lens)]
    ref = [want(h) for h in hs]
    slots, at = list(range(B, 0, -1)), [0] * B
    # bf16: three times the oracle's own error with 16-bit tensors between its operations (a query that is nearly orthogonal to its keys is normed up)
    rounded = torch.cat([want(h, O.to_bf16) for h in hs])
    tol = 2e-5 if dtype == f32 else 3 * rel(rounded, torch.cat(ref))
    for step in ["prompt"] + list(portion) + [1] * tail:
        ns = list(lens) if step == "prompt" else [step] * B
        b = StepBatch.build([[0] * n for n in ns], slots, at, None, dev)
        got = group(torch.cat([h[a:a + n] for h, a, n in zip(hs, at, ns)]).to(dtype).to(dev), b, caches)["y"]
        err = rel(got, torch.cat([x[a:a + n] for x, a, n in zip(ref, at, ns)]))
        assert err < tol, (step, at, err)
        at = [a + n for a, n in zip(at, ns)]


def case_one_key_stands_out(dev, dtype, size, positions, n, cut=None):
    """Every query asks for ONE row's key: inside that row's chunk the output is its value alone, from the next chunk on nothing of it -- wherever the row
    lies in its chunk, in prompts and in decoding."""
    from aria_amd.serving import StepBatch

    D = 64
    m = left(heads=2, kv_heads=1, dim=32, vdim=32, size=size, scale=4.0)
    z = lambda *s: torch.zeros(*s, dtype=bf16)  # noqa: E731
    eye = torch.eye(32).to(bf16)
    w = {"q": z(64, D), "k": z(32, D), "v": z(32, D), "o": torch.cat([torch.cat([eye, eye], 1), z(32, 64)])}
    w["q"][:32, 32:], w["q"][32:, 32:], w["k"][:, :32], w["v"][:, :32] = eye, eye, eye, eye
    group, want = _mixer("chunk", m, dev, dtype, D, w=w)
    for far in positions:
        h = rnd(n, D, seed=far + 1, scale=0.3)
        h[:, 31], h[far, :32], h[far, 31] = 0, 0, 3     # the only row with this key direction ...
        h[:, 32:], h[:, 63] = 0, 1                      # ... and every query asks for it
        ref = want(h)
        inside = [i for i in range(far, n) if i // size == far // size]
        outside = [i for i in range(far + 1, n) if i // size != far // size]
        assert all(float(ref[i, 31]) > 5 for i in inside) and all(abs(float(ref[i, 31])) < 1e-6 for i in outside)
        caches, c = group.new_cache(1, n + 3, dev), cut or max(1, n - 4)
        b = StepBatch.build([[0] * c], [0], [0], None, dev)
        got = [group(h[:c].to(dtype).to(dev), b, caches)["y"]]
        for p in range(c, n):
            got.append(group(h[p:p + 1].to(dtype).to(dev), StepBatch.build([[0]], [0], [p], None, dev), caches)["y"])
        err = (torch.cat(got).cpu().double() - ref).abs().amax(-1)
        assert float(err.max()) < (1e-3 if dtype == f32 else 0.1), (far, int(err.argmax()), float(err.max()))


def case_far_memory(dev, dtype, n, kinds=("gated", "lightning")):
    """One early row writes a value that slow decays keep; the rows behind it write nothing.  Every later output shows it, over every block and chunk of the
    prompt and in decoding; a lost state would show zeros."""
    from aria_amd.serving import StepBatch

    D, z = 16, lambda *s: torch.zeros(*s, dtype=bf16)  # noqa: E731
    for kind in kinds:
        m = dict(heads=1, dim=8, vdim=8, **(dict(tau=1000.0) if kind == "gated" else dict(decay=[0.9995])))
        w = {"q": z(8, D), "k": z(8, D), "v": z(8, D), "g": z(8, D), "o": z(D, 8), "norm": torch.ones(8, dtype=bf16)}
        w["q"][0, 15], w["k"][0, 0], w["v"][3, 1], w["g"][:, 15], w["o"][3, 3] = 2, 2, 2, 3, 1
        if kind == "gated":
            w.update({"a1": z(1, D), "a2": z(8, 1), "a2.b": z(8)})
        group, want = _mixer(kind, m, dev, dtype, D, w=w)
        for at in (0, 1, 63, 64):
            h = torch.zeros(n, D, dtype=bf16)
            h[:, 15], h[at, 0], h[at, 1] = 1, 1, 1
            ref = want(h)
            assert float(ref[at:, 3].min()) > 0.5 and (at == 0 or float(ref[:at].abs().max()) < 1e-6)
            caches, c = group.new_cache(1, n, dev), n - 3
            got = [group(h[:c].to(dtype).to(dev), StepBatch.build([[0] * c], [0], [0], None, dev), caches)["y"]]
            for p in range(c, n):
                got.append(group(h[p:p + 1].to(dtype).to(dev), StepBatch.build([[0]], [0], [p], None, dev), caches)["y"])
            err = (torch.cat(got).cpu().double() - ref).abs().amax(-1)
            assert float(err.max()) < (1e-4 if dtype == f32 else 0.03), (kind, at, int(err.argmax()), float(err.max()))


def case_linear_chunks_agree(dev, kind, m, lens, starts, per_chunk, steep=False):
    """The matrix-pipe form cut into chunks of ``per_chunk`` blocks against the token-by-token form, outputs and states, from zero and from carried states."""
    from aria_amd import ops
    from aria_amd.serving import StepBatch

    group, _ = _mixer(kind, m, dev, bf16, 32)
    part = group.parts[0]
    shape, T = part.shape(), sum(lens)
    proj = rnd(T, shape.ldp, seed=3)
    if steep:
        proj[:, shape.a_off:] *= 40           # decays from 1 down to (nearly) 0 in one block
    for off, width, real, H in ((shape.q_off, shape.dp, shape.d, shape.H), (shape.k_off, shape.dp, shape.d, shape.H), (shape.v_off, shape.dvp, shape.dv, shape.H)):
        proj[:, off:off + H * width].view(T, H, width)[..., real:] = 0
    state = torch.randn(len(lens) + 1, shape.H, shape.dp, shape.dvp, generator=gen(5))
    state[:, :, shape.d:] = 0
    state[..., shape.dv:] = 0
    b = StepBatch.build([[0] * n for n in lens], list(range(len(lens), 0, -1)), starts, None, dev)
    s1, s2 = state.clone().to(dev), state.clone().to(dev)
    o1 = ops.linear_step(shape, proj.to(dev), s1, b)
    plain = b.linear_tables
    b.linear_tables = lambda block, per: plain(block, per_chunk)
    o2 = ops.linear_chunks(shape, proj.to(dev), s2, b)
    assert torch.equal(s1[0].cpu(), state[0]) and torch.equal(s2[0].cpu(), state[0])       # a slot that is not in the batch stays as it is
    assert rel(o2, o1.cpu().double()) < 1.2e-2 and rel(s2, s1.cpu().double()) < 8e-3


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
        toks = [tokens(cfg, n + tail, seed=i + 10 * round_) for i, n in enumerate(lens)]
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
    m, toks = build(cfg, w, dev, dtype), tokens(cfg, n, seed=5)
    want, tol = O.forward(cfg, w, toks), model_tol(cfg, w, [toks], dtype)
    for sizes in ([n], [1] * n, [2] * (n // 2) + [n % 2], [7, 2, 5, n - 14], [n - 3, 2, 1], [1, n - 1]):
        sched, at, got = Scheduler(m, n + 2), 0, []
        for k in [s for s in sizes if s]:
            got.append(sched.step(["a"], [toks[at:at + k]], [list(range(k))]).cpu())
            at += k
        assert logit_err(torch.cat(got), want) < tol, sizes


def case_continuation_beside_decode(dev, dtype, name="mixed"):
    """A step that carries a portion of one request and single tokens of others."""
    from aria_amd.serving import Scheduler

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=4)
    m = build(cfg, w, dev, dtype)
    a, b = tokens(cfg, 24, seed=1), tokens(cfg, 6, seed=2)
    sched = Scheduler(m, 30)
    sched.step(["a", "b"], [a[:5], b[:4]], [[], []])
    g1 = sched.step(["b", "a"], [[b[4]], a[5:23]], [[0], list(range(18))])
    g2 = sched.step(["a", "b"], [[a[23]], [b[5]]])
    wa, wb, tol = O.forward(cfg, w, a), O.forward(cfg, w, b), model_tol(cfg, w, [a, b], dtype)
    assert logit_err(g1, torch.cat([wb[4:5], wa[5:23]])) < tol
    assert logit_err(g2, torch.stack([wa[23], wb[5]])) < tol


def case_rows_do_not_depend_on_company(dev, dtype, name="mixed", n=11, companies=(0, 4, 17)):
    """Logits of one request alone, in a batch of 5 and in a batch past the one-call decode limit, on different slots."""
    from aria_amd import kozipel
    from aria_amd.serving import Scheduler

    assert kozipel.DECODE_ROWS < 17
    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=6)
    m = build(cfg, w, dev, dtype)
    toks, res = tokens(cfg, n, seed=1), []
    for company in companies:
        sched = Scheduler(m, n + 1)
        ids = [f"x{i}" for i in range(company)] + ["a"]
        ps = [tokens(cfg, 1 + i % 7, seed=20 + i) for i in range(company)]
        got = [sched.step(ids, ps + [toks[:n - 2]])[-1]]
        for s in (n - 2, n - 1):
            got.append(sched.step(ids, [[1 + i] for i in range(company)] + [[toks[s]]])[-1])
        res.append(torch.stack(got).cpu().double())
    for r in res[1:]:
        assert logit_err(r, res[0]) < model_tol(cfg, w, [toks], dtype) * (0.1 if dtype == f32 else 1)


def case_passes_keep_their_own_cache(dev, dtype):
    """The passes of a repeated span have caches and states of their own, and equal a stack with the tensors copied out -- but for the embedding, which
    comes back in front of every pass after the first."""
    from aria_amd.serving import Scheduler

    cfg = config([parallel(), lightning()], width=24, vocab=40, loop=dict(start=0, stop=2, times=2))
    w = checkpoint(cfg, seed=2)
    m, toks = build(cfg, w, dev, dtype), tokens(cfg, 9)
    s = Scheduler(m, 12)
    s.step(["a"], [toks[:6]], [[]])
    got = torch.cat([s.step(["a"], [[t]]) for t in toks[6:]])
    assert len(m.caches) == 4
    for i in (0, 1):
        for a, b in zip(m.caches[i], m.caches[i + 2]):
            assert a.rows.shape == b.rows.shape and a.rows.data_ptr() != b.rows.data_ptr() and not torch.equal(a.rows, b.rows)
    plain = dict({k: v for k, v in cfg.items() if k != "loop"}, layers=cfg["layers"] * 2)
    w2 = dict(w, **{f"l{i + 2}" + k[2:]: v for k, v in w.items() for i in (0, 1) if k.startswith(f"l{i}.")})
    other = O.forward(plain, w2, toks)[6:]
    want, tol = O.forward(cfg, w, toks)[6:], model_tol(cfg, w, [toks], dtype)
    assert logit_err(got, want) < tol and logit_err(other, want) > 10 * tol      # (the copied-out stack without the embedding is another model)


def case_stream_after_every_layer(dev, dtype, name="mixed", n=6):
    from aria_amd.serving import StepBatch

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=9)
    m, toks = build(cfg, w, dev, dtype), tokens(cfg, n)
    want = O.forward(cfg, w, toks, want_layers=True)[1]
    m.setup_caches(1, n)
    trace = []
    m.step(StepBatch.build([toks], [0], [0], None, dev), trace)
    assert len(trace) == len(want) == len(m.config.runs)
    for got, x in zip(trace, want):
        assert got.dtype == f32 and rel(got[:, :cfg["width"]], x) < (1e-5 if dtype == f32 else 3e-2)


def case_greedy_generation(dev, dtype, name="mixed", n_new=6, tmp=None):
    """Greedy tokens through serving.generate (registry, loader, scheduler, sampling) equal the oracle's argmax chain wherever that is not a tie."""
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
        assert dtype != f32 or a == g[:cut]
    sampled = serving.generate(m, prompts[:2], 4, temperature=1.0, top_k=5)
    assert all(0 <= t < cfg["vocab"] for s in sampled for t in s) and [len(s) for s in sampled] == [4, 4]


def case_long_decode(dev, dtype, prompt=3, steps=150, name="mixed"):
    """Many single tokens after a short prompt, over many chunks, against the oracle at every step."""
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


def case_slot_used_again(dev, dtype, name="mixed"):
    """A one-token request on a slot whose last owner went far: neither its state nor its chunk shows."""
    from aria_amd.serving import Scheduler

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=14)
    m = build(cfg, w, dev, dtype)
    s = Scheduler(m, 40)
    s.step(["old"], [tokens(cfg, 30, seed=1)], [[]])
    s.finish("old")
    toks = tokens(cfg, 4, seed=2)
    got = torch.cat([s.step(["new"], [[t]]) for t in toks])
    assert s.slots == 1 and logit_err(got, O.forward(cfg, w, toks)) < model_tol(cfg, w, [toks], dtype)


def case_graph_replay(dev, name="mixed", n=70, steps=3):
    """The one-call decode step captured into a HIP graph: every replay, with eager work between, equals the eager step."""
    from aria_amd.serving import Scheduler, StepBatch

    cfg = CONFIGS[name]
    w = checkpoint(cfg, seed=6)
    m = build(cfg, w, dev, bf16)
    toks = tokens(cfg, n, seed=1)

    def prompt():
        s = Scheduler(m, n + 8)
        s.step(["a"], [toks[:n - steps]])
        return s

    s = prompt()
    eager = [s.step(["a"], [[t]]).clone() for t in toks[n - steps:]]
    b = StepBatch.build([[toks[n - steps]]], [0], [n - steps], [0], dev)
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
        prompt()                                  # (the recurrence goes on from its state: every round starts from the prompt's)
        for j in range(steps):
            ids.fill_(toks[n - steps + j])
            pos.fill_(n - steps + j)
            g.replay()
            torch.cuda.synchronize()
            assert logit_err(out, eager[j].cpu().double()) < 1e-3, (r, j)
            torch.randn(1 << 16, device=dev).sum().item()


def case_bad_inputs(dev):
    import pytest

    from aria_amd.kozipel import KozipelConfig
    from aria_amd.serving import Scheduler

    cfg = CONFIGS["last"]
    m = build(cfg, checkpoint(cfg), dev, f32)
    s = Scheduler(m, 8)
    with pytest.raises(ValueError):
        s.step(["a"], [list(range(9))])
    s.step(["a"], [[1, 2]])
    with pytest.raises(RuntimeError):
        s.step(["b"], [[1]])
    one = cfg["layers"][0]
    for bad in (dict(cfg, layers=[dict(one, type="other")]), dict(cfg, layers=[dict(one, mlp=dict(kind="moe"))]), dict(cfg, loop=dict(start=1, stop=3, times=2)),
                dict(cfg, loop=dict(start=0, stop=1, times=0))):
        with pytest.raises(ValueError):
            KozipelConfig.from_dict(bad)
    with pytest.raises(ValueError):
        build(config([lightning(heads=2, decay=(0.5,))]), checkpoint(config([lightning(heads=2, decay=(0.5,))])), dev, f32)
    c = KozipelConfig.from_dict(cfg)
    assert [(r.layer, r.again) for r in c.runs] == [(0, False), (1, False), (1, True)] == O.layer_runs(cfg)
    assert [r.layer for r in KozipelConfig.from_dict(dict(cfg, loop=None)).runs] == [0, 1]
    assert (c.eps, c.residual_mult, c.logit_softcap, c.embedding_scale) == (EPS, 0.5, 12.0, 2.0)
