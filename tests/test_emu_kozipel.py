"""Chunk-local attention, linear attention and Kozipel through the SIMT emulator (CPU): tests/kozipel_cases.py at small sizes."""
import pytest
import torch

from tests import kozipel_cases as C

bf16, f32 = torch.bfloat16, torch.float32
DEV = "cpu"
both = pytest.mark.parametrize("dtype", [bf16, f32], ids=["bf16", "f32"])


@pytest.fixture(scope="module", autouse=True)
def emu():
    from tests.emu import emu_lib

    emu_lib.install()
    yield
    emu_lib.uninstall()


@both
def test_rms_stream(dtype):
    C.case_rms_stream(DEV, dtype)


@both
def test_softcap_and_relu_gate(dtype):
    C.case_softcap_and_relu_gate(DEV, dtype)


@pytest.mark.parametrize("M,ff,K", [(5, 24, 16), (70, 128, 64)])
def test_relu_glu(M, ff, K):
    C.case_relu_glu(DEV, M, ff, K)


@both
def test_norm_gate(dtype):
    C.case_norm_gate(DEV, dtype)


@both
@pytest.mark.parametrize("kind,m,lens,portion", [
    ("chunk", C.left(), (30, 1, 13), (5, 2)), ("chunk", C.left(heads=3, kv_heads=3, dim=13, vdim=11, size=4), (9, 4), (9,)),
    ("gated", C.right(), (70, 1), (3, 2)), ("gated", C.right(heads=1, dim=7, vdim=9, tau=1.0), (5, 3), ()),
    ("lightning", C.lightning()["mixer"], (66, 2), (4,))])
def test_mixer(dtype, kind, m, lens, portion):
    C.case_mixer(DEV, dtype, kind, m, lens, tail=2, portion=portion)


@both
def test_one_key_stands_out(dtype):
    C.case_one_key_stands_out(DEV, dtype, 6, [0, 5, 6, 11], 16, cut=10)


@both
def test_far_memory(dtype):
    C.case_far_memory(DEV, dtype, 135, kinds=("gated",) if dtype == f32 else ("gated", "lightning"))


@pytest.mark.parametrize("defer", [False, True])
@pytest.mark.parametrize("kind,m,steep", [("gated", C.right(heads=1, dim=20, vdim=72, tau=4.0), False), ("gated", C.right(heads=1, dim=100, vdim=24, tau=0.5), True),
                                          ("lightning", C.lightning(heads=2, dim=130, vdim=8, decay=(0.6, 0.0))["mixer"], False)])
def test_linear_chunks_agree(kind, m, steep, defer, monkeypatch):
    if defer:
        monkeypatch.setenv("ARIA_EMU_GLDS_DEFER", "1")
    C.case_linear_chunks_agree(DEV, kind, m, (150, 3), [0, 9], 1, steep)


@pytest.mark.parametrize("dtype,name", [(bf16, "odd"), (f32, "odd"), (f32, "mixed"), (bf16, "ones"), (bf16, "steep"), (bf16, "huge"), (bf16, "vocabulary")])
def test_model(dtype, name):
    C.case_model(DEV, dtype, name, lens=(4, 1, 2), tail=2)


def test_portions():
    C.case_portions(DEV, f32, "last", n=15)


@both
def test_continuation_beside_decode(dtype):
    C.case_continuation_beside_decode(DEV, dtype, "last")


def test_passes_keep_their_own_cache():
    C.case_passes_keep_their_own_cache(DEV, bf16)


@both
def test_stream_after_every_layer(dtype):
    C.case_stream_after_every_layer(DEV, dtype, n=3)


def test_slot_used_again():
    C.case_slot_used_again(DEV, bf16, "last")


@both
def test_greedy_generation(dtype, tmp_path):
    C.case_greedy_generation(DEV, dtype, "last", n_new=3, tmp=tmp_path)


def test_bad_inputs():
    C.case_bad_inputs(DEV)
