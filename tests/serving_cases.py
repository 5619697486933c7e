"""The serving layer: the scheduler driving a gptfast (Aria) decoder, Duguzen and Kozipel alike, the command line, the trace runner.  Shared by
tests/test_emu_serving.py (CPU) and tests/test_gpu_serving.py (hardware)."""
import io
import json
import os

import torch

from tests import kozipel_cases as K
from tests import latent_cases as L

bf16, f32 = torch.bfloat16, torch.float32


def gptfast_toy(dev, head_dim=64):
    from aria_amd import gptfast as G

    args = G.ModelArgs(block_size=64, vocab_size=136, n_layer=2, n_head=2, dim=2 * head_dim, intermediate_size=40, n_local_heads=2, rope_base=10000.0,
                       norm_eps=1e-5, num_experts=8, router_topk=3, num_shared_experts=2)
    m, g = G.Transformer(args), L.gen(5)
    with torch.no_grad():
        for n, p in m.named_parameters():
            p.copy_((1 + 0.1 * torch.randn(p.shape, generator=g)).to(bf16) if "norm" in n else (torch.randn(p.shape, generator=g) * 0.08).to(bf16))
    return m.to(dev).eval()


def case_gptfast_batch(dev, engine=True):
    """Unequal requests of one batch give each request's own logits bit for bit (its sequence runs by itself on its slot), with the decode engine and
    with the tile path; the tile path also equals one prefill of the whole prefix.  Slots are used again by a second batch."""
    from aria_amd.serving import Scheduler

    m = gptfast_toy(dev)
    m.use_decode_engine = engine
    toks = [torch.randint(0, 136, (n,), generator=L.gen(n)).tolist() for n in (7, 3, 5)]

    def alone(t):
        s = Scheduler(m, 16)
        return torch.cat([s.step(["x"], [t[:-2]], [[0, len(t) - 3]])] + [s.step(["x"], [[i]]) for i in t[-2:]]).cpu()

    want = [alone(t) for t in toks]
    if not engine:
        for t, x in zip(toks, want):
            m.setup_caches(1, 16)
            with torch.no_grad():
                whole = m(torch.tensor([t], device=dev))[0].float().cpu()
            assert L.rel(x, whole[[0, len(t) - 3, len(t) - 2, len(t) - 1]]) < 2e-2
    sched = Scheduler(m, 16)
    for _ in range(2):
        got = sched.step(["a", "b", "c"], [t[:-2] for t in toks], [[0, len(t) - 3] for t in toks]).cpu()
        assert torch.equal(got, torch.cat([x[:2] for x in want]))
        for back in (2, 1):
            got = sched.step(["c", "a", "b"], [[toks[i][-back]] for i in (2, 0, 1)]).cpu()
            assert torch.equal(got, torch.stack([want[i][4 - back] for i in (2, 0, 1)]))
        for r in "bca":
            sched.finish(r)


def case_gptfast_generate(dev):
    """serving.generate on the gptfast decoder: greedy continuation equals arg-max over full prefills wherever that is not a tie."""
    from aria_amd import serving

    m = gptfast_toy(dev)
    m.use_decode_engine = False       # (a bf16 router's close calls may fall either way between the engine and the tile path)
    prompts = [[5, 9, 77], [100, 3, 8, 20, 1]]
    for p, g in zip(prompts, serving.generate(m, prompts, 3, temperature=0)):
        m.setup_caches(1, 16)
        with torch.no_grad():
            lg = m(torch.tensor([p + g], device=dev))[0].float().cpu()
        for i, t in enumerate(g):
            row = lg[len(p) + i - 1]
            assert float(row.max() - row[t]) <= 0.05 * float(row.std())


DESIGNS = {"duguzen": (L, "equal"), "kozipel": (K, "last")}   # cases module, configuration


def write_model(tmp, design="duguzen", seed=12):
    from safetensors.torch import save_file

    cases, name = DESIGNS[design]
    cfg = cases.CONFIGS[name]
    w = cases.checkpoint(cfg, seed=seed)
    (tmp / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp / "model.safetensors"))
    return cfg, w


def case_command_line(dev, tmp, design="duguzen"):
    from aria_amd import inference as I
    from aria_amd import registry, serving

    cfg, _ = write_model(tmp, design)
    a = I.parse_arguments(["--base_model_path", str(tmp), "--prompt_ids", "5,17,3", "--prompt_ids", "9", "--max_new_tokens", "3", "--temperature", "0",
                           "--dtype", "float32"])
    got = I.generate_ids(a, dev)
    m = registry.load_model(str(tmp), dev, f32)
    assert got == serving.generate(m, [[5, 17, 3], [9]], 3, temperature=0) and all(0 <= t < cfg["vocab"] for g in got for t in g)


def case_trace_run(dev, tmp, dtype="float32", design="duguzen"):
    """Steps in, logits out: the files, the order of rows, ``done`` lines, requests that end, a second batch, and the values against the oracle."""
    import numpy as np

    from aria_amd import trace_run

    cases = DESIGNS[design][0]
    O = cases.O
    cfg, w = write_model(tmp, design)
    out = tmp / "out"
    out.mkdir()
    draw = L.clear_tokens if cases is L else (lambda cfg, w, n, seed: L.tokens(cfg, n, seed))
    a, b, c = ([int(t) for t in draw(cfg, w, n, seed=n)] for n in (6, 4, 3))
    steps = [dict(step=0, entries=[dict(id="a", tokens=a[:5], want=[0, 4]), dict(id="b", tokens=b[:2], want=[])], end=[]),
             dict(step=1, entries=[dict(id="b", tokens=[b[2]], want=[]), dict(id="a", tokens=[a[5]], want=[])], end=["a"]),
             dict(step=2, entries=[dict(id="b", tokens=[b[3]], want=[0])], end=["b"]),
             dict(step=3, entries=[dict(id="a", tokens=c, want=[2, 1])], end=["a"])]
    said = io.StringIO()
    rc = trace_run.main(["--model", str(tmp), "--dtype", dtype, "--out", str(out), "--max-tokens", "12"], io.StringIO("".join(json.dumps(s) + "\n" for s in steps)),
                        said, dev)
    assert rc == 0 and said.getvalue().split("\n")[:-1] == [f"done {i}" for i in range(4)]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
    want = {0: O.forward(cfg, w, a)[[0, 4]], 2: O.forward(cfg, w, b)[[3]], 3: O.forward(cfg, w, c)[[2, 1]]}
    for n, x in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(x.shape).copy())
        assert L.logit_err(got, x) < (5e-5 if dtype == "float32" else cases.model_tol(cfg, w, [a, b, c], bf16)), n


def case_registry():
    import pytest

    from aria_amd import registry

    assert registry.architecture({"architecture": "Duguzen"}) == "Duguzen"
    assert registry.architecture({"architectures": ["AriaForConditionalGeneration"]}) == registry.architecture({"model_type": "aria"})
    assert registry.resolve({"architecture": "Duguzen"})[1].__name__ == "DuguzenForCausalLM"
    assert registry.resolve({"architecture": "Kozipel"})[1].__name__ == "KozipelForCausalLM"
    with pytest.raises(ValueError):
        registry.architecture({"architecture": "nothing"})
