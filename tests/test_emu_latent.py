"""Latent-attention family and Duguzen through the SIMT emulator (CPU): tests/latent_cases.py at small sizes."""
import pytest
import torch

from tests import latent_cases as C

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
def test_dyt_stream(dtype):
    C.case_dyt_stream(DEV, dtype)


@both
def test_activations(dtype):
    C.case_activations(DEV, dtype)


@pytest.mark.parametrize("M,N,K", [(5, 24, 16), (70, 136, 72)])
def test_gemm_relu_squared(M, N, K):
    C.case_gemm_relu_squared(DEV, M, N, K)


@pytest.mark.parametrize("M,N,K", [(5, 9, 4), (70, 66, 20)])
def test_gemm_f32(M, N, K):
    C.case_gemm_f32(DEV, M, N, K)


@pytest.mark.parametrize("E,groups,keep,k", [(8, 2, 1, 2), (12, 4, 2, 3), (6, 1, 1, 1), (8, 8, 3, 3), (100, 10, 4, 12)])
def test_route_groups(E, groups, keep, k):
    C.case_route_groups(DEV, 9, E, groups, keep, k)


def test_sort_wide():
    C.case_sort_wide(DEV, T=12)


@both
@pytest.mark.parametrize("m,lens", [(C.mixer(), (7, 1, 12)), (C.mixer(heads=2, dim=13, rot_dim=6, vdim=11, kv_rank=21), (3, 2)),
                                    (C.mixer(heads=1, dim=100, rot_dim=60, vdim=70, kv_rank=72), (5,))])
def test_latent_attention(dtype, m, lens):
    C.case_latent_attention(DEV, dtype, m, lens, tail=2)


@pytest.mark.parametrize("heads,R", [(17, 140), (2, 600)])
def test_latent_attention_kernel_classes(heads, R):
    C.case_latent_attention(DEV, bf16, C.mixer(heads=heads, dim=8, rot_dim=8, vdim=8, kv_rank=R), (3,), tail=1)


@both
def test_one_key_stands_out(dtype):
    C.case_one_key_stands_out(DEV, dtype, [0, 1, 63, 64, 65], 68)


@pytest.mark.parametrize("dtype,name", [(bf16, "odd"), (f32, "odd"), (f32, "mixed"), (bf16, "broad"), (bf16, "vocabulary")])
def test_model(dtype, name):
    C.case_model(DEV, dtype, name, lens=(4, 1, 2), tail=2)


def test_portions():
    C.case_portions(DEV, f32, "equal", n=15)


@both
def test_continuation_beside_decode(dtype):
    C.case_continuation_beside_decode(DEV, dtype)


def test_borrowed_layers_keep_their_own_cache():
    C.case_borrowed_layers_keep_their_own_cache(DEV, bf16)


@both
def test_stream_after_every_layer(dtype):
    C.case_stream_after_every_layer(DEV, dtype, n=3)


@both
def test_greedy_generation(dtype, tmp_path):
    C.case_greedy_generation(DEV, dtype, n_new=4, tmp=tmp_path)


def test_bad_inputs():
    C.case_bad_inputs(DEV)
