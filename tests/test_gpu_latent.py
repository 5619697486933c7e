"""Latent-attention family and Duguzen on hardware (-m gpu): tests/latent_cases.py against the gfx950 library, at sizes that cross tile borders and
reach every kernel instantiation."""
import pytest
import torch

from tests import latent_cases as C

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
def test_dyt_stream(dtype):
    C.case_dyt_stream(DEV, dtype)
    C.case_dyt_stream(DEV, dtype, T=5, D=2048)


@both
def test_activations(dtype):
    C.case_activations(DEV, dtype)


@pytest.mark.parametrize("M,N,K", [(5, 24, 16), (300, 520, 264), (512, 768, 1024), (4096, 3080, 256), (1024, 2560, 4096)])   # every kernel family, split tiles
def test_gemm_relu_squared(M, N, K):
    C.case_gemm_relu_squared(DEV, M, N, K)


@pytest.mark.parametrize("M,N,K", [(5, 9, 4), (70, 66, 20), (300, 257, 516)])
def test_gemm_f32(M, N, K):
    C.case_gemm_f32(DEV, M, N, K)


@pytest.mark.parametrize("E,groups,keep,k", [(8, 2, 1, 2), (12, 4, 2, 3), (6, 1, 1, 1), (8, 8, 3, 3), (64, 8, 3, 6), (100, 10, 4, 12), (256, 8, 4, 8)])
def test_route_groups(E, groups, keep, k):
    C.case_route_groups(DEV, 200, E, groups, keep, k)


def test_sort_wide():
    C.case_sort_wide(DEV, T=300, E=100)
    C.case_sort_wide(DEV, T=300, E=256)


@both
@pytest.mark.parametrize("m,lens", [
    (C.mixer(), (7, 1, 12)), (C.mixer(heads=2, dim=13, rot_dim=6, vdim=11, kv_rank=21), (3, 2)),
    (C.mixer(heads=1, dim=100, rot_dim=60, vdim=70, kv_rank=72), (300, 65)),            # 192 / 128 columns
    (C.mixer(heads=3, dim=160, rot_dim=40, vdim=200, kv_rank=136), (130, 64)),          # 256 / 256 columns
    (C.mixer(heads=2, dim=280, rot_dim=8, vdim=60, kv_rank=48), (90, 3)),               # wider than every flash form
    (C.mixer(heads=4, dim=40, rot_dim=24, vdim=64, kv_rank=64), (513, 255, 256, 257))])
def test_latent_attention(dtype, m, lens):
    C.case_latent_attention(DEV, dtype, m, lens)


@pytest.mark.parametrize("heads,R", [(1, 128), (17, 140), (16, 256), (40, 512), (16, 500), (2, 600)])
def test_latent_attention_kernel_classes(heads, R):
    C.case_latent_attention(DEV, bf16, C.mixer(heads=heads, dim=32, rot_dim=32, vdim=32, kv_rank=R), (70, 200), tail=2)


@both
def test_one_key_stands_out(dtype):
    C.case_one_key_stands_out(DEV, dtype, [0, 1, 2, 62, 63, 64, 65, 127, 128, 191, 192, 255, 256, 257, 500, 511, 512, 515], 520)


def test_splits_agree():
    C.case_splits_agree(DEV)


@both
@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_model(dtype, name):
    C.case_model(DEV, dtype, name)


@both
def test_model_long_unequal_prompts(dtype):
    C.case_model(DEV, dtype, "sharp", lens=(150, 3, 67, 64, 65), tail=6)


@both
def test_portions(dtype):
    C.case_portions(DEV, dtype)


@both
def test_continuation_beside_decode(dtype):
    C.case_continuation_beside_decode(DEV, dtype)


@both
@pytest.mark.parametrize("name", ["mixed", "vocabulary", "broad"])
def test_rows_do_not_depend_on_company(dtype, name):
    C.case_rows_do_not_depend_on_company(DEV, dtype, name)


@both
def test_borrowed_layers_keep_their_own_cache(dtype):
    C.case_borrowed_layers_keep_their_own_cache(DEV, dtype)


@both
def test_stream_after_every_layer(dtype):
    C.case_stream_after_every_layer(DEV, dtype)


@both
def test_greedy_generation(dtype, tmp_path):
    C.case_greedy_generation(DEV, dtype, tmp=tmp_path)


@both
def test_long_decode(dtype):
    C.case_long_decode(DEV, dtype)


def test_graph_replay():
    C.case_graph_replay(DEV)


def test_bad_inputs():
    C.case_bad_inputs(DEV)
