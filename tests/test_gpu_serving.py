"""Scheduler, command line and trace runner on hardware (-m gpu)."""
import json
import os
import subprocess
import sys

import pytest
import torch

from tests import serving_cases as C

pytestmark = pytest.mark.gpu
DEV = "cuda"


@pytest.fixture(scope="module", autouse=True)
def real_library():
    from aria_amd import hip

    assert not hip.is_emulated() and hip.get_lib().path.endswith("libaria_hip.so") and torch.cuda.is_available()
    yield


@pytest.mark.parametrize("engine", [False, True])
def test_gptfast_batch(engine):
    C.case_gptfast_batch(DEV, engine)


def test_gptfast_generate():
    C.case_gptfast_generate(DEV)


designs = pytest.mark.parametrize("design", sorted(C.DESIGNS))


@designs
def test_command_line(tmp_path, design):
    C.case_command_line(DEV, tmp_path, design)


@designs
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run(tmp_path, dtype, design):
    C.case_trace_run(DEV, tmp_path, dtype, design)


@designs
def test_trace_run_program(tmp_path, design):
    """bin/trace_run as a program: a step a line, an answer before the next."""
    cfg, _ = C.write_model(tmp_path, design)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = subprocess.Popen([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "bfloat16", "--out", str(tmp_path),
                          "--max-tokens", "8"], stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    try:
        for n, toks in enumerate(([1, 2, 3], [4], [5])):
            p.stdin.write(json.dumps(dict(step=n, entries=[dict(id="x", tokens=toks, want=[0])], end=["x"] if n == 2 else [])) + "\n")
            p.stdin.flush()
            assert p.stdout.readline().strip() == f"done {n}"
            assert os.path.getsize(tmp_path / f"{n}.f32") == 4 * cfg["vocab"]
        p.stdin.close()
        assert p.wait(timeout=60) == 0
    finally:
        p.kill()
