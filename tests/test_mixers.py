"""Layer mechanisms (tah_amd.mixers, include/tah_mixers.h), each alone, against the plain oracle: on the CPU execution build
at small sizes, on the GPU at those and at larger ones."""
import pytest

from tests import emu_util
from tests import zedudra_cases as D
from tests import zozosun_cases as Z

needs_clang = pytest.mark.skipif(not emu_util.have_host_clang(), reason="host clang++ not available")
BOTH = pytest.mark.parametrize("dtype", ["f32", "bf16"])


def delta(heads, kv, dim, vdim, conv, eps=1e-4):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv, "eps": eps}


def latent(heads, dim, rot, vdim, rank, window, base=50.0, scale=0.4):
    return Z.latent_of(heads, dim, rot, vdim, rank, window, base, scale)["mixer"]


# (sizes, lengths, portions per sequence)
DELTA_SMALL = [(delta(2, 1, 6, 5, 3), (5, 3), ((2, 3), (3,))), (delta(2, 2, 12, 8, 4), (7, 2), ((7,), (2,))),
               (delta(2, 1, 16, 32, 3), (5, 4), ((3, 2), (4,))),
               (delta(2, 1, 16, 16, 4), (100, 49), ((50, 50), (49,)))]   # long enough for the chunked form
DELTA_GPU = DELTA_SMALL + [
    (delta(6, 3, 40, 24, 4), (70, 33), ((37, 2, 31), (2, 31))), (delta(4, 4, 64, 64, 2), (130, 5), ((128, 2), (3, 2))),
    (delta(8, 2, 128, 128, 4), (200, 65), ((64, 17, 119), (65,))), (delta(2, 1, 256, 96, 4), (40, 40), ((40,), (17, 23))),
    (delta(3, 1, 17, 130, 1), (30, 9), ((16, 14), (9,))), (delta(2, 2, 100, 256, 5), (21, 2), ((5, 16), (2,))),
    (delta(5, 5, 32, 512, 3), (19, 18), ((19,), (2, 16))), (delta(4, 2, 128, 64, 4), (333, 97), ((96, 64, 173), (97,))),
    (delta(2, 1, 256, 32, 2), (161, 70), ((100, 61), (70,))), (delta(6, 3, 32, 48, 4), (520, 520), ((255, 265), (256, 264))),
]
# (sizes, prompt, portions, decoded tokens, ring capacity)
LATENT_SMALL = [(latent(2, 8, 4, 6, 10, 4), 9, (2, 5, 2), 3, None), (latent(1, 32, 6, 16, 40, 3), 6, (6,), 2, 5)]
LATENT_GPU = LATENT_SMALL + [
    (latent(3, 24, 8, 20, 48, 40), 150, (64, 2, 84), 45, None), (latent(16, 128, 64, 128, 512, 100), 300, (300,), 70, 130),
    (latent(20, 64, 32, 64, 96, 65), 129, (1 + 63, 65), 66, 65), (latent(5, 64, 16, 200, 64, 7), 40, (7, 2, 31), 9, None),
    (latent(2, 96, 32, 96, 288, 128), 260, (128, 132), 4, 200), (latent(33, 32, 32, 32, 32, 2), 20, (20,), 3, None),
    (latent(4, 200, 40, 48, 700, 33), 70, (3, 67), 5, None), (latent(2, 400, 6, 300, 64, 9), 21, (21,), 3, None),
    (latent(2, 32, 2, 16, 960, 5), 12, (12,), 2, None),
]
MOE_SMALL = [(5, 40, 12, 4, 2, 9), (3, 32, 32, 3, 1, 0)]
MOE_GPU = MOE_SMALL + [(32, 96, 48, 16, 4, 64), (200, 160, 96, 8, 8, 32), (700, 256, 192, 64, 6, 128), (31, 512, 100, 7, 3, 0), (300, 72, 40, 5, 5, 17)]
# (sizes, prompt, portions, decoded tokens, further arguments): windows inside, at and across the 64-key tiles and the 32-key
# passes, kept tokens that fill tiles of their own, more query heads than a tile or a pass takes, heads of up to 256
WINDOW_SMALL = [(D.window_of(2, 1, 12, 6, 4, 2), 11, (2, 7, 2), 4, {}), (D.window_of(2, 2, 32, 32, 6, 3), 13, (13,), 2, {}),
                (D.window_of(2, 1, 16, 8, 5, 1), 7, (5, 2), 3, dict(own_values=20, adjacent=False, gate=False))]
WINDOW_GPU = WINDOW_SMALL + [
    (D.window_of(16, 8, 128, 64, 64, 4), 200, (64, 2, 63, 71), 70, {}), (D.window_of(10, 2, 128, 48, 33, 3), 150, (150,), 40, {}),
    (D.window_of(20, 1, 64, 32, 65, 1), 140, (1 + 62, 2, 75), 66, {}), (D.window_of(5, 5, 24, 24, 128, 7), 260, (130, 130), 9, {}),
    (D.window_of(33, 1, 96, 2, 31, 5), 90, (33, 57), 34, {}), (D.window_of(4, 2, 160, 40, 40, 70), 180, (90, 90), 45, {}),
    (D.window_of(6, 2, 256, 256, 100, 130), 310, (200, 2, 108), 12, {}), (D.window_of(2, 2, 300, 20, 9, 2), 40, (40,), 12, {}),
    (D.window_of(4, 1, 128, 64, 1, 0), 70, (35, 35), 5, {}), (D.window_of(4, 4, 128, 128, 600, 64), 700, (300, 400), 20, {}),
    (D.window_of(9, 3, 40, 0, 17, 3), 80, (80,), 20, {}), (D.window_of(8, 1, 128, 64, 50, 4), 120, (60, 60), 30, dict(max_len=4000)),
    (D.window_of(8, 2, 64, 64, 40, 2), 130, (65, 65), 45, dict(own_values=64)), (D.window_of(4, 2, 128, 32, 50, 4), 130, (130,), 20, dict(own_values=72, gate=False)),
    (D.window_of(4, 1, 48, 24, 20, 3), 70, (70,), 22, dict(own_values=100, adjacent=False)),
]
GROUPS = [(5, 44, 4), (3, 96, 3), (2, 64, 8)]
GROUPS_GPU = GROUPS + [(32, 2048, 8), (40, 2048, 1), (3, 1920, 16), (7, 5000, 5), (2, 600, 200), (6, 16384, 2), (4, 24, 24), (9, 1000, 8)]
CONVS = [(20, 4, 3), (32, 1, 1), (24, 2, 4), (16, 1, 6)]
CONVS_GPU = CONVS + [(2048, 8, 4), (600, 3, 2), (1000, 8, 9), (72, 1, 33)]
EXPERTS_SMALL = [(5, 40, 12, 6, 2, 3, 2, 0.7), (3, 32, 32, 4, 1, 1, 1, 1.5)]
EXPERTS_GPU = EXPERTS_SMALL + [(32, 96, 48, 16, 4, 4, 2, 1.0), (200, 160, 96, 8, 3, 2, 1, 7.0), (700, 256, 192, 64, 6, 8, 4, 0.5), (300, 72, 40, 130, 5, 65, 20, 1.0),
                               (31, 512, 100, 256, 8, 128, 64, 2.0), (20, 64, 32, 9, 2, 9, 5, 1.0)]


# ── CPU execution build ──────────────────────────────────────────────────────────────────────────────────────────────
@needs_clang
@BOTH
def test_rows_on_cpu_shim(dtype):
    with emu_util.emulated():
        Z.rows_case("cpu", Z.DTYPES[dtype])


@needs_clang
def test_linear_batches_on_cpu_shim():
    with emu_util.emulated():
        Z.linear_batch_case("cpu", 3, 16, 32, 3)


@needs_clang
@BOTH
@pytest.mark.parametrize("case", range(len(DELTA_SMALL)))
def test_delta_rule_on_cpu_shim(dtype, case):
    m, lens, cuts = DELTA_SMALL[case]
    with emu_util.emulated():
        Z.delta_case("cpu", Z.DTYPES[dtype], m, lens, cuts, steps=2)


@needs_clang
@BOTH
@pytest.mark.parametrize("case", range(len(LATENT_SMALL)))
def test_latent_attention_on_cpu_shim(dtype, case):
    m, total, cuts, steps, cap = LATENT_SMALL[case]
    with emu_util.emulated():
        Z.latent_case("cpu", Z.DTYPES[dtype], m, total, cuts, steps, cap)


@needs_clang
@BOTH
@pytest.mark.parametrize("case", range(len(MOE_SMALL)))
def test_mixture_of_experts_on_cpu_shim(dtype, case):
    with emu_util.emulated():
        Z.moe_case("cpu", Z.DTYPES[dtype], *MOE_SMALL[case])


@needs_clang
@BOTH
@pytest.mark.parametrize("case", range(len(WINDOW_SMALL)))
def test_window_attention_on_cpu_shim(dtype, case):
    m, total, cuts, steps, kw = WINDOW_SMALL[case]
    with emu_util.emulated():
        D.window_case("cpu", Z.DTYPES[dtype], m, total, cuts, steps, **kw)


@needs_clang
@BOTH
def test_norms_over_groups_on_cpu_shim(dtype):
    with emu_util.emulated():
        for case in GROUPS:
            D.group_norm_case("cpu", Z.DTYPES[dtype], *case)


@needs_clang
@BOTH
def test_input_convolution_on_cpu_shim(dtype):
    with emu_util.emulated():
        for case in CONVS:
            D.conv_case("cpu", Z.DTYPES[dtype], *case)


@needs_clang
@BOTH
def test_activations_on_cpu_shim(dtype):
    with emu_util.emulated():
        D.activation_case("cpu", Z.DTYPES[dtype], 2, 16, 32)


@needs_clang
@BOTH
@pytest.mark.parametrize("case", range(len(EXPERTS_SMALL)))
def test_grouped_experts_on_cpu_shim(dtype, case):
    with emu_util.emulated():
        D.moe_case("cpu", Z.DTYPES[dtype], *EXPERTS_SMALL[case])


# ── GPU ──────────────────────────────────────────────────────────────────────────────────────────────────────────────
@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("rows,width,cols", [(5, 72, 96), (32, 2048, 2048), (40, 100, 104), (3, 5000, 5024), (2, 16384, 16384)])
def test_rows_gpu(dtype, rows, width, cols):
    Z.rows_case("cuda", Z.DTYPES[dtype], rows, width, cols)


@pytest.mark.gpu
@pytest.mark.parametrize("rows,n,k,batch", [(3, 16, 32, 3), (32, 512, 128, 16), (20, 128, 512, 16), (7, 48, 96, 1), (32, 96, 256, 5)])
def test_linear_batches_gpu(rows, n, k, batch):
    Z.linear_batch_case("cuda", rows, n, k, batch)


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("case", range(len(DELTA_GPU)))
def test_delta_rule_gpu(dtype, case):
    m, lens, cuts = DELTA_GPU[case]
    Z.delta_case("cuda", Z.DTYPES[dtype], m, lens, cuts, steps=4)


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("case", range(len(LATENT_GPU)))
def test_latent_attention_gpu(dtype, case):
    m, total, cuts, steps, cap = LATENT_GPU[case]
    Z.latent_case("cuda", Z.DTYPES[dtype], m, total, cuts, steps, cap)


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("case", range(len(MOE_GPU)))
def test_mixture_of_experts_gpu(dtype, case):
    Z.moe_case("cuda", Z.DTYPES[dtype], *MOE_GPU[case])


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("case", range(len(WINDOW_GPU)))
def test_window_attention_gpu(dtype, case):
    m, total, cuts, steps, kw = WINDOW_GPU[case]
    D.window_case("cuda", Z.DTYPES[dtype], m, total, cuts, steps, **kw)


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("case", range(len(GROUPS_GPU)))
def test_norms_over_groups_gpu(dtype, case):
    D.group_norm_case("cuda", Z.DTYPES[dtype], *GROUPS_GPU[case])


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("case", range(len(CONVS_GPU)))
def test_input_convolution_gpu(dtype, case):
    D.conv_case("cuda", Z.DTYPES[dtype], *CONVS_GPU[case], cuts=((50, 2, 33), (1 + 2, 64)))


@pytest.mark.gpu
@BOTH
def test_activations_gpu(dtype):
    D.activation_case("cuda", Z.DTYPES[dtype])
    D.activation_case("cuda", Z.DTYPES[dtype], 32, 480, 256)


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("case", range(len(EXPERTS_GPU)))
def test_grouped_experts_gpu(dtype, case):
    D.moe_case("cuda", Z.DTYPES[dtype], *EXPERTS_GPU[case])
