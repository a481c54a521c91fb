// Residual rows of a layer-by-layer decoder, gfx950: token rows into the residual stream, the norm of a sublayer's
// output with its residual sum, and element-wise activations.  HBM-bound; one workgroup per row, eight columns per
// thread and pass, everything between load and store in float32.
#include <hip/hip_runtime.h>

#include "mixer_device.h"

namespace tah {
namespace {

constexpr int kRowThreads = 256;
constexpr int kMaxUnits = 8;  // eight-column units per thread: rows of up to 16384 columns

template <class E>
__global__ __launch_bounds__(kRowThreads) void embed_rows_kernel(const tah_embed_rows_args p) {
    const int row = blockIdx.x, tid = threadIdx.x;
    if (tid == 0 && p.pos) {
        const bool act = !p.finished || p.finished[row] == 0;
        p.slot[row] = act ? p.slot_base + row : -1;
        p.q_pos[row] = act ? p.pos[row] : -1;
        p.active[row] = act ? 1 : 0;
    }
    int64_t t = p.tok[row];
    t = t < 0 ? 0 : (t >= p.vocab ? p.vocab - 1 : t);
    const E* e = static_cast<const E*>(p.embed) + t * p.cols;
    for (int c = 8 * tid; c < p.cols; c += 8 * kRowThreads) {
        float v[8];
        load8(e + c, v);
        store8(p.x + (int64_t)row * p.cols + c, v);
        if (p.xe) store8(static_cast<E*>(p.xe) + (int64_t)row * p.cols + c, v);
        if (p.x_packed) static_cast<bf16x8*>(p.x_packed)[rows_form_unit(row, c)] = to_bf16x8(v);
    }
}

// U: units per thread
template <class E, int U>
__global__ __launch_bounds__(kRowThreads) void residual_norm_kernel(const tah_residual_norm_args p) {
    __shared__ float red[kRowThreads / kWave];
    const int row = blockIdx.x, tid = threadIdx.x;
    float y[U][8], x[U][8];
    float ss = 0.f;
    const float ys = p.y_scale ? p.y_scale[row] : 1.0f;
#pragma unroll
    for (int u = 0; u < U; ++u) {
        const int c = 8 * (tid + u * kRowThreads);
#pragma unroll
        for (int i = 0; i < 8; ++i) y[u][i] = x[u][i] = 0.f;
        if (c < p.cols) {
            load8(p.x + (int64_t)row * p.cols + c, x[u]);
            if (p.y) {
                load8(static_cast<const E*>(p.y) + (int64_t)row * p.y_row_stride + c, y[u]);
#pragma unroll
                for (int i = 0; i < 8; ++i) y[u][i] *= ys;
            }
        }
    }
    if (p.experts) {
        for (int j = 0; j < p.top; ++j) {
            const float w = p.weight[(int64_t)row * p.top + j];
            const E* e = static_cast<const E*>(p.experts) + ((int64_t)p.index[(int64_t)row * p.top + j] * p.index_scale + (int64_t)row * p.index_row) * p.experts_row_stride;
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int c = 8 * (tid + u * kRowThreads);
                if (c < p.cols) {
                    float v[8];
                    load8(e + c, v);
#pragma unroll
                    for (int i = 0; i < 8; ++i) y[u][i] += w * v[i];
                }
            }
        }
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
        for (int i = 0; i < 8; ++i) ss += y[u][i] * y[u][i];
    ss = block_sum<kRowThreads / kWave>(ss, red);
    const float r = 1.0f / sqrtf(ss / (float)p.width + p.eps);
    float sx = 0.f;
#pragma unroll
    for (int u = 0; u < U; ++u) {
        const int c = 8 * (tid + u * kRowThreads);
        if (c < p.cols) {
            float k[8];
            load8(p.coef + c, k);
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                x[u][i] += y[u][i] * r * k[i];
                sx += x[u][i] * x[u][i];
            }
            store8(p.x + (int64_t)row * p.cols + c, x[u]);
            if (p.xe) store8(static_cast<E*>(p.xe) + (int64_t)row * p.cols + c, x[u]);
            if (p.x_packed) static_cast<bf16x8*>(p.x_packed)[rows_form_unit(row, c)] = to_bf16x8(x[u]);
        }
    }
    if (!p.final_coef) return;
    sx = block_sum<kRowThreads / kWave>(sx, red);
    const float rx = 1.0f / sqrtf(sx / (float)p.width + p.eps);
#pragma unroll
    for (int u = 0; u < U; ++u) {
        const int c = 8 * (tid + u * kRowThreads);
        if (c < p.cols) {
            float k[8];
            load8(p.final_coef + c, k);
#pragma unroll
            for (int i = 0; i < 8; ++i) k[i] *= x[u][i] * rx;
            if (p.normed) store8(static_cast<E*>(p.normed) + (int64_t)row * p.cols + c, k);
            if (p.normed_packed) static_cast<bf16x8*>(p.normed_packed)[rows_form_unit(row, c)] = to_bf16x8(k);
        }
    }
}

template <class E, int KIND>
__global__ __launch_bounds__(kRowThreads) void activate_rows_kernel(const E* in, int64_t in_rs, E* out, int64_t out_rs, int cols) {
    const int row = blockIdx.y;
    const int c = 8 * (blockIdx.x * kRowThreads + threadIdx.x);
    if (c >= cols) return;
    float a[8];
    load8(in + (int64_t)row * in_rs + c, a);
    if constexpr (KIND == TAH_ROWS_GELU_TANH) {
#pragma unroll
        for (int i = 0; i < 8; ++i) a[i] = gelu_tanh_exact(a[i]);
    } else {
        float b[8];
        load8(in + (int64_t)row * in_rs + cols + c, b);
#pragma unroll
        for (int i = 0; i < 8; ++i) a[i] = silu_exact(a[i]) * b[i];
    }
    store8(out + (int64_t)row * out_rs + c, a);
}

template <class E>
void launch_residual(const tah_residual_norm_args& p, hipStream_t st) {
    const int units = (p.cols / 8 + kRowThreads - 1) / kRowThreads;
    if (units <= 1) hipLaunchKernelGGL((residual_norm_kernel<E, 1>), dim3(p.rows), dim3(kRowThreads), 0, st, p);
    else if (units <= 2) hipLaunchKernelGGL((residual_norm_kernel<E, 2>), dim3(p.rows), dim3(kRowThreads), 0, st, p);
    else if (units <= 4) hipLaunchKernelGGL((residual_norm_kernel<E, 4>), dim3(p.rows), dim3(kRowThreads), 0, st, p);
    else hipLaunchKernelGGL((residual_norm_kernel<E, kMaxUnits>), dim3(p.rows), dim3(kRowThreads), 0, st, p);
}

template <class E>
void launch_activate(const void* in, int64_t in_rs, void* out, int64_t out_rs, int rows, int cols, int kind, hipStream_t st) {
    const dim3 grid((cols / 8 + kRowThreads - 1) / kRowThreads, rows);
    if (kind == TAH_ROWS_GELU_TANH)
        hipLaunchKernelGGL((activate_rows_kernel<E, TAH_ROWS_GELU_TANH>), grid, dim3(kRowThreads), 0, st, static_cast<const E*>(in), in_rs,
                           static_cast<E*>(out), out_rs, cols);
    else
        hipLaunchKernelGGL((activate_rows_kernel<E, TAH_ROWS_SILU_MUL>), grid, dim3(kRowThreads), 0, st, static_cast<const E*>(in), in_rs,
                           static_cast<E*>(out), out_rs, cols);
}

bool dtype_ok(int32_t d) { return d == TAH_DT_BF16 || d == TAH_DT_F32; }

}  // namespace
}  // namespace tah

extern "C" int tah_embed_rows(const tah_embed_rows_args* a, tah_stream_t stream) {
    using namespace tah;
    if (!a) return TAH_E_NULL;
    if (a->rows < 0 || a->vocab <= 0 || a->cols <= 0 || a->cols % 8 != 0 || !dtype_ok(a->dtype)) return TAH_E_SHAPE;
    if (a->x_packed && (a->rows > 32 || a->cols % 32 != 0)) return TAH_E_SHAPE;
    if (a->rows == 0) return TAH_OK;
    if (!a->tok || !a->embed || !a->x || (a->pos && (!a->slot || !a->q_pos || !a->active))) return TAH_E_NULL;
    if (!aligned_16(a->embed) || !aligned_16(a->x) || !aligned_16(a->xe) || !aligned_16(a->x_packed)) return TAH_E_ALIGN;
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (a->dtype == TAH_DT_BF16) hipLaunchKernelGGL((embed_rows_kernel<__bf16>), dim3(a->rows), dim3(kRowThreads), 0, st, *a);
    else hipLaunchKernelGGL((embed_rows_kernel<float>), dim3(a->rows), dim3(kRowThreads), 0, st, *a);
    return launch_status();
}

extern "C" int tah_residual_norm(const tah_residual_norm_args* a, tah_stream_t stream) {
    using namespace tah;
    if (!a) return TAH_E_NULL;
    if (a->rows < 0 || a->width <= 0 || a->cols < a->width || a->cols % 8 != 0 || a->cols > 8 * kRowThreads * kMaxUnits ||
        !dtype_ok(a->dtype) || a->top < 0)
        return TAH_E_SHAPE;
    if ((a->x_packed || a->normed_packed) && (a->rows > 32 || a->cols % 32 != 0)) return TAH_E_SHAPE;
    if (a->rows == 0) return TAH_OK;
    if (!a->x || !a->coef || (a->experts && (!a->index || !a->weight))) return TAH_E_NULL;
    if ((a->normed || a->normed_packed) && !a->final_coef) return TAH_E_NULL;
    const void* ptrs[] = {a->y, a->experts, a->coef, a->final_coef, a->x, a->xe, a->x_packed, a->normed, a->normed_packed};
    for (const void* q : ptrs)
        if (!aligned_16(q)) return TAH_E_ALIGN;
    if ((a->y && (a->y_row_stride % 8 != 0 || a->y_row_stride < a->cols)) ||
        (a->experts && (a->experts_row_stride % 8 != 0 || a->experts_row_stride < a->cols)))
        return TAH_E_ALIGN;
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (a->dtype == TAH_DT_BF16) launch_residual<__bf16>(*a, st);
    else launch_residual<float>(*a, st);
    return launch_status();
}

extern "C" int tah_activate_rows(const void* in, int64_t in_rs, void* out, int64_t out_rs, int32_t rows, int32_t cols, int32_t kind,
                                 int32_t dtype, tah_stream_t stream) {
    using namespace tah;
    if (rows < 0 || rows > 65535 * 16 || cols < 0 || cols % 8 != 0 || !dtype_ok(dtype) || (kind != TAH_ROWS_GELU_TANH && kind != TAH_ROWS_SILU_MUL))
        return TAH_E_SHAPE;
    if (rows == 0 || cols == 0) return TAH_OK;
    if (!in || !out) return TAH_E_NULL;
    if (!aligned_16(in) || !aligned_16(out) || in_rs % 8 != 0 || out_rs % 8 != 0) return TAH_E_ALIGN;
    hipStream_t st = static_cast<hipStream_t>(stream);
    for (int32_t r = 0; r < rows; r += 65535) {  // (the grid's second dimension)
        const int32_t n = rows - r < 65535 ? rows - r : 65535;
        if (dtype == TAH_DT_BF16)
            launch_activate<__bf16>(static_cast<const __bf16*>(in) + r * in_rs, in_rs, static_cast<__bf16*>(out) + r * out_rs, out_rs, n, cols, kind, st);
        else
            launch_activate<float>(static_cast<const float*>(in) + r * in_rs, in_rs, static_cast<float*>(out) + r * out_rs, out_rs, n, cols, kind, st);
    }
    return launch_status();
}
