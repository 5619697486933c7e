"""Chunk-local attention, linear attention and Kozipel on hardware (-m gpu): tests/kozipel_cases.py against the gfx950 library, at sizes that cross tile
borders and reach every kernel instantiation."""
import pytest
import torch

from tests import kozipel_cases as C

bf16, f32 = torch.bfloat16, torch.float32
pytestmark = pytest.mark.gpu
DEV = "cuda"
both = pytest.mark.parametrize("dtype", [bf16, f32], ids=["bf16", "f32"])


@pytest.fixture(scope="module", autouse=True)
def real_library():
    from aria_amd import hip

    assert not hip.is_emulated()
    assert hip.get_lib().path.endswith("libaria_hip.so")   # raises if the library is missing: no fallback
    assert torch.cuda.is_available()
    yield


@both
def test_rms_stream(dtype):
    C.case_rms_stream(DEV, dtype)
    for n, D in ((2048, 2048), (2561, 2568), (8000, 8000), (9000, 9008)):
        C.case_rms_stream(DEV, dtype, n=n, D=D)


@both
def test_softcap_and_relu_gate(dtype):
    C.case_softcap_and_relu_gate(DEV, dtype)


@pytest.mark.parametrize("M,ff,K", [(5, 24, 16), (300, 128, 64), (700, 640, 256), (257, 256, 2560)])
def test_relu_glu(M, ff, K):
    C.case_relu_glu(DEV, M, ff, K)


@both
def test_norm_gate(dtype):
    C.case_norm_gate(DEV, dtype)


@both
@pytest.mark.parametrize("kind,m,lens,portion", [
    ("chunk", C.left(), (30, 1, 13), (5, 2)), ("chunk", C.left(heads=3, kv_heads=3, dim=13, vdim=11, size=4), (9, 4), (9,)),
    ("chunk", C.left(heads=4, kv_heads=1, dim=100, vdim=64, size=65), (300, 129, 64), (70,)),          # 128 / 128 columns
    ("chunk", C.left(heads=6, kv_heads=3, dim=160, vdim=128, size=300), (700, 299, 300), (5,)),        # 192 / 128 columns
    ("chunk", C.left(heads=3, kv_heads=1, dim=200, vdim=250, size=257), (520, 514), (3,)),             # 256 / 256 columns
    ("chunk", C.left(heads=2, kv_heads=2, dim=264, vdim=300, size=40), (50, 3), (45,)),                # wider than every matrix-pipe form
    ("gated", C.right(), (70, 1), (3, 2)), ("gated", C.right(heads=1, dim=7, vdim=9, tau=1.0), (5, 3), ()),
    ("gated", C.right(heads=3, dim=72, vdim=130, tau=16.0), (300, 64, 129), (70,)), ("gated", C.right(heads=2, dim=200, vdim=300, tau=16.0), (257, 128), (2,)),
    ("gated", C.right(heads=1, dim=300, vdim=20, tau=16.0), (40,), (2,)),
    ("lightning", C.lightning()["mixer"], (66, 2), (4,)), ("lightning", C.lightning(heads=4, dim=128, vdim=128, decay=(0.61, 0.9, 0.99, 0.999))["mixer"], (513, 70), (65,))])
def test_mixer(dtype, kind, m, lens, portion):
    C.case_mixer(DEV, dtype, kind, m, lens, portion=portion, D=64 if max(lens) > 100 else 32)


@both
def test_one_key_stands_out(dtype):
    C.case_one_key_stands_out(DEV, dtype, 64, [0, 1, 63, 64, 100, 127, 128], 140, cut=122)
    C.case_one_key_stands_out(DEV, dtype, 100, [0, 99, 100, 163, 164, 199, 200], 215)
    C.case_one_key_stands_out(DEV, dtype, 1, [0, 4, 5], 9)


@both
def test_far_memory(dtype):
    C.case_far_memory(DEV, dtype, 700)


@pytest.mark.parametrize("per_chunk", [1, 3])
@pytest.mark.parametrize("kind,m,steep", [
    ("gated", C.right(heads=1, dim=20, vdim=72, tau=4.0), False), ("gated", C.right(heads=2, dim=100, vdim=24, tau=0.5), True),
    ("gated", C.right(heads=4, dim=256, vdim=512, tau=16.0), False), ("gated", C.right(heads=2, dim=256, vdim=200, tau=4.0), True),
    ("lightning", C.lightning(heads=2, dim=130, vdim=8, decay=(0.6, 0.0))["mixer"], False), ("lightning", C.lightning(heads=3, dim=128, vdim=128)["mixer"], False),
    ("lightning", C.lightning(heads=2, dim=40, vdim=300, decay=(1.0, 0.05))["mixer"], False)])
def test_linear_chunks_agree(kind, m, steep, per_chunk):
    C.case_linear_chunks_agree(DEV, kind, m, (450, 3, 64, 129), [0, 9, 0, 64], per_chunk, steep)


@both
@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_model(dtype, name):
    C.case_model(DEV, dtype, name)


@both
@pytest.mark.parametrize("name", ["mixed", "wide", "steep"])
def test_model_long_unequal_prompts(dtype, name):
    C.case_model(DEV, dtype, name, lens=(150, 3, 67, 64, 65), tail=6)


@both
def test_model_sixteen_requests(dtype):
    C.case_model(DEV, dtype, "many", lens=tuple(1 + 5 * i % 17 for i in range(16)), tail=4)


@both
@pytest.mark.parametrize("dim", [40, 128, 250, 400, 700])
def test_recurrence_of_many_sequences(dtype, dim):
    """whole state lines a workgroup (and, past 512 channels, half ones)"""
    C.case_mixer(DEV, dtype, "gated", C.right(heads=8, dim=dim, vdim=72, tau=16.0), (2, 3, 1) * 14, tail=2)
    C.case_mixer(DEV, dtype, "lightning", C.lightning(heads=8, dim=dim, vdim=72, decay=[0.5 + 0.06 * i for i in range(8)])["mixer"], (2, 3, 1) * 14, tail=2)


@both
def test_portions(dtype):
    C.case_portions(DEV, dtype)
    C.case_portions(DEV, dtype, "wide", n=205)


@both
def test_continuation_beside_decode(dtype):
    C.case_continuation_beside_decode(DEV, dtype)


@both
@pytest.mark.parametrize("name", ["mixed", "wide", "vocabulary", "broad"])
def test_rows_do_not_depend_on_company(dtype, name):
    C.case_rows_do_not_depend_on_company(DEV, dtype, name)


@both
def test_passes_keep_their_own_cache(dtype):
    C.case_passes_keep_their_own_cache(DEV, dtype)


@both
def test_stream_after_every_layer(dtype):
    C.case_stream_after_every_layer(DEV, dtype)


@both
def test_slot_used_again(dtype):
    C.case_slot_used_again(DEV, dtype)


@both
def test_greedy_generation(dtype, tmp_path):
    C.case_greedy_generation(DEV, dtype, tmp=tmp_path)


@both
def test_long_decode(dtype):
    C.case_long_decode(DEV, dtype)


@both
def test_long_decode_wide(dtype):
    C.case_long_decode(DEV, dtype, prompt=60, steps=80, name="wide")


def test_graph_replay():
    C.case_graph_replay(DEV)


def test_bad_inputs():
    C.case_bad_inputs(DEV)
