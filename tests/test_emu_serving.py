"""Scheduler, command line and trace runner on CPU through the SIMT emulator."""
import pytest

from tests import serving_cases as C

DEV = "cpu"


@pytest.fixture(scope="module", autouse=True)
def emu():
    from tests.emu import emu_lib

    emu_lib.install()
    yield
    emu_lib.uninstall()


def test_gptfast_batch():
    C.case_gptfast_batch(DEV, engine=False)   # (the engine's emulated form takes a minute: on hardware only)


def test_gptfast_generate():
    C.case_gptfast_generate(DEV)


designs = pytest.mark.parametrize("design", sorted(C.DESIGNS))


@designs
def test_command_line(tmp_path, design):
    C.case_command_line(DEV, tmp_path, design)


@designs
def test_trace_run(tmp_path, design):
    C.case_trace_run(DEV, tmp_path, design=design)


def test_registry():
    C.case_registry()


def test_trace_run_refuses_a_dtype_the_model_does_not_have(tmp_path):
    import io
    import json

    from aria_amd import trace_run

    (tmp_path / "config.json").write_text(json.dumps({"architectures": ["AriaForConditionalGeneration"]}))
    assert trace_run.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "4"], io.StringIO(""), io.StringIO(), DEV) == 3
