// Residual rows of a layer-by-layer decoder, gfx950: token rows into the residual stream, the norm of a sublayer's
// output with its residual sum and the norm and short convolution in front of the next one, and element-wise
// activations.  HBM-bound; one workgroup per row, eight columns per thread and pass, everything between load and store in
// float32.
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
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] *= p.scale;
        store8(p.x + (int64_t)row * p.cols + c, v);
        if (p.xe) store8(static_cast<E*>(p.xe) + (int64_t)row * p.cols + c, v);
        if (p.x_packed) static_cast<bf16x8*>(p.x_packed)[rows_form_unit(row, c)] = to_bf16x8(v);
    }
}

// Sum of a row's values over its group, one partial sum s[u] per thread and unit, for each of the thread's units.
// GROUPS: several groups of group_units units each, added up inside a wave where the groups divide it; else through LDS:
// `unit_sums` of as many floats as the row has units, `group_sum` of as many as it has groups.  `red`: a float per wave.
template <int U, bool GROUPS>
__device__ __forceinline__ void group_sums(float (&s)[U], int units, int groups, int group_units, float* red, float* unit_sums, float* group_sum) {
    const int tid = threadIdx.x;
    if constexpr (!GROUPS) {
        float t = 0.f;
#pragma unroll
        for (int u = 0; u < U; ++u) t += s[u];
        t = block_sum<kRowThreads / kWave>(t, red);
#pragma unroll
        for (int u = 0; u < U; ++u) s[u] = t;
    } else if (group_units <= kWave && (group_units & (group_units - 1)) == 0) {
        for (int d = group_units / 2; d >= 1; d >>= 1) {
#pragma unroll
            for (int u = 0; u < U; ++u) s[u] += __shfl_xor(s[u], d);
        }
    } else {
#pragma unroll
        for (int u = 0; u < U; ++u)
            if (tid + u * kRowThreads < units) unit_sums[tid + u * kRowThreads] = s[u];
        __syncthreads();
        for (int g = tid / kWave; g < groups; g += kRowThreads / kWave) {
            float t = 0.f;
            for (int i = tid % kWave; i < group_units; i += kWave) t += unit_sums[g * group_units + i];
            t = wave_sum(t);
            if (tid % kWave == 0) group_sum[g] = t;
        }
        __syncthreads();
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int g = (tid + u * kRowThreads) / group_units;
            s[u] = group_sum[g < groups ? g : groups - 1];  // (columns behind the last group hold zeros)
        }
    }
}

constexpr int kMaxGroups = 256;

// U: units per thread
template <class E, int U, bool GROUPS>
__global__ __launch_bounds__(kRowThreads) void residual_norm_kernel(const tah_residual_norm_args p) {
    __shared__ float red[kRowThreads / kWave], unit_sums[GROUPS ? U * kRowThreads : 1], group_sum[GROUPS ? kMaxGroups : 1];
    const int row = blockIdx.x, tid = threadIdx.x;
    const int units = p.cols / 8, group_units = GROUPS ? p.group_cols / 8 : units;
    const float count = GROUPS ? (float)(p.width / p.groups) : (float)p.width;
    float y[U][8], x[U][8];
    const bool add = p.y || p.experts;
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
    float s[U];
    if (add) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            s[u] = 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) s[u] += y[u][i] * y[u][i];
        }
        group_sums<U, GROUPS>(s, units, p.groups, group_units, red, unit_sums, group_sum);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
        const int c = 8 * (tid + u * kRowThreads);
        float sx = 0.f;
        if (c < p.cols) {
            if (add) {
                const float r = 1.0f / sqrtf(s[u] / count + p.eps);
                float k[8];
                load8(p.coef + c, k);
#pragma unroll
                for (int i = 0; i < 8; ++i) x[u][i] += y[u][i] * r * k[i];
                store8(p.x + (int64_t)row * p.cols + c, x[u]);
            }
#pragma unroll
            for (int i = 0; i < 8; ++i) sx += x[u][i] * x[u][i];
            if (p.xe) store8(static_cast<E*>(p.xe) + (int64_t)row * p.cols + c, x[u]);
            if (p.x_packed) static_cast<bf16x8*>(p.x_packed)[rows_form_unit(row, c)] = to_bf16x8(x[u]);
        }
        s[u] = sx;
    }
    if (!p.next_coef) return;
    group_sums<U, GROUPS>(s, units, p.groups, group_units, red, unit_sums, group_sum);
    const int slot = p.conv ? p.slot[row] : -1, pos = p.conv ? p.pos[row] : -1;
    const bool live = slot >= 0 && slot < p.nslots && pos >= 0;
#pragma unroll
    for (int u = 0; u < U; ++u) {
        const int c = 8 * (tid + u * kRowThreads);
        if (c < p.cols) {
            const float rx = 1.0f / sqrtf(s[u] / count + p.eps);
            float k[8];
            load8(p.next_coef + c, k);
#pragma unroll
            for (int i = 0; i < 8; ++i) k[i] *= x[u][i] * rx;
            if (p.conv) {
                E* const ring = static_cast<E*>(p.conv_state) + (int64_t)(live ? slot : 0) * p.taps * p.cols + c;
                float h[8], w[8];
#pragma unroll
                for (int i = 0; i < 8; ++i) k[i] = (float)(E)k[i];
                load8(p.conv + (int64_t)(p.taps - 1) * p.cols + c, w);
                if (live) store8(ring + (int64_t)(pos % p.taps) * p.cols, k);  // (in the place of a token no row reads any more)
#pragma unroll
                for (int i = 0; i < 8; ++i) k[i] += w[i] * k[i];
                for (int d = 1; live && d < p.taps && d <= pos; ++d) {
                    load8(ring + (int64_t)((pos - d) % p.taps) * p.cols, h);
                    load8(p.conv + (int64_t)(p.taps - 1 - d) * p.cols + c, w);
#pragma unroll
                    for (int i = 0; i < 8; ++i) k[i] += w[i] * h[i];
                }
            }
            if (p.normed) store8(static_cast<E*>(p.normed) + (int64_t)row * p.cols + c, k);
            if (p.normed_packed) static_cast<bf16x8*>(p.normed_packed)[rows_form_unit(row, c)] = to_bf16x8(k);
        }
    }
}

// One thread per eight channels and tile of a portion's rows.  The first tile of a portion reads the slot's earlier inputs and
// enters the portion's last ones, so that no other workgroup looks at what it replaces (taps - 1 <= kConvRows).
constexpr int kConvRows = 32;

template <class E>
__global__ __launch_bounds__(kWave) void conv_rows_kernel(const E* h, const float* conv, E* state, const tah_portions P, E* out, int cols, int taps,
                                                          int nslots) {
    int tile = blockIdx.y, b = 0, row0 = 0, row_end = 0;
    if (!find_tile(P.cu, P.nseq, kConvRows, tile, b, row0, row_end)) return;
    const int c = 8 * (blockIdx.x * kWave + threadIdx.x);
    if (c >= cols) return;
    const int first = P.cu[b], last = P.cu[b + 1], slot = P.slot[b], pos0 = P.pos0[b];
    const bool live = slot >= 0 && slot < nslots;
    E* const ring = state + (int64_t)(live ? slot : 0) * taps * cols + c;
    // the input d rows in front of row r
    auto input = [&](int r, int d, float (&v)[8]) __attribute__((always_inline)) {
        const int at = r - d, pos = pos0 + at - first;
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = 0.f;
        if (at >= first) load8(h + (int64_t)at * cols + c, v);
        else if (pos >= 0 && live) load8(ring + (int64_t)(pos % taps) * cols, v);
    };
    for (int r = row0; r < row_end; ++r) {
        float y[8], v[8], w[8];
        load8(h + (int64_t)r * cols + c, y);
        load8(conv + (int64_t)(taps - 1) * cols + c, w);
#pragma unroll
        for (int i = 0; i < 8; ++i) y[i] += w[i] * y[i];
        for (int d = 1; d < taps; ++d) {
            input(r, d, v);
            load8(conv + (int64_t)(taps - 1 - d) * cols + c, w);
#pragma unroll
            for (int i = 0; i < 8; ++i) y[i] += w[i] * v[i];
        }
        store8(out + (int64_t)r * cols + c, y);
    }
    if (row0 != first || !live) return;
    for (int r = last - taps + 1 > first ? last - taps + 1 : first; r < last; ++r) {
        float v[8];
        load8(h + (int64_t)r * cols + c, v);
        store8(ring + (int64_t)((pos0 + r - first) % taps) * cols, v);
    }
}

// The same for up to four taps: a thread asks for all of its rows, and the inputs in front of them, before it uses the first.
constexpr int kFewTaps = 4, kFewRows = 16;

template <class E>
__global__ __launch_bounds__(kWave) void conv_few_rows_kernel(const E* h, const float* conv, E* state, const tah_portions P, E* out, int cols, int taps,
                                                              int nslots) {
    int tile = blockIdx.y, b = 0, row0 = 0, row_end = 0;
    if (!find_tile(P.cu, P.nseq, kFewRows, tile, b, row0, row_end)) return;
    const int c = 8 * (blockIdx.x * kWave + threadIdx.x);
    if (c >= cols) return;
    const int first = P.cu[b], last = P.cu[b + 1], slot = P.slot[b], pos0 = P.pos0[b];
    const bool live = slot >= 0 && slot < nslots;
    E* const ring = state + (int64_t)(live ? slot : 0) * taps * cols + c;
    constexpr int kFront = kFewTaps - 1;
    E v[kFront + kFewRows][8];  // row row0 - kFront + i; rows nobody reads repeat one that is there
    bool there[kFront];
#pragma unroll
    for (int i = 0; i < kFront; ++i) {
        const int at = row0 - kFront + i, pos = pos0 + at - first;
        there[i] = at >= first || (live && pos >= 0 && kFront - i < taps);
        const E* const src = at >= first || !there[i] ? h + (int64_t)(at >= first ? at : row0) * cols + c : ring + (int64_t)(pos % taps) * cols;
        __builtin_memcpy(v[i], src, sizeof(v[i]));
    }
#pragma unroll
    for (int i = 0; i < kFewRows; ++i) __builtin_memcpy(v[kFront + i], h + (int64_t)(row0 + i < row_end ? row0 + i : row0) * cols + c, sizeof(v[i]));
    float w[kFewTaps][8];  // of the input d rows back
#pragma unroll
    for (int d = 0; d < kFewTaps; ++d) {
        load8(conv + (int64_t)(d < taps ? taps - 1 - d : 0) * cols + c, w[d]);
#pragma unroll
        for (int e = 0; e < 8; ++e) w[d][e] = d < taps ? w[d][e] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < kFewRows; ++i) {
        float y[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) y[e] = (float)v[kFront + i][e] + w[0][e] * (float)v[kFront + i][e];
#pragma unroll
        for (int d = 1; d < kFewTaps; ++d) {
            const bool on = kFront + i - d >= kFront || there[kFront + i - d < kFront ? kFront + i - d : 0];
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] += on ? w[d][e] * (float)v[kFront + i - d][e] : 0.f;
        }
        if (row0 + i < row_end) store8(out + (int64_t)(row0 + i) * cols + c, y);
    }
    if (row0 != first || !live) return;
    for (int r = last - taps + 1 > first ? last - taps + 1 : first; r < last; ++r) {
        float x[8];
        load8(h + (int64_t)r * cols + c, x);
        store8(ring + (int64_t)((pos0 + r - first) % taps) * cols, x);
    }
}

template <class E, int KIND>
__global__ __launch_bounds__(kRowThreads) void activate_rows_kernel(const E* in, int64_t in_rs, E* out, int64_t out_rs, int cols, float c0, float c1) {
    const int row = blockIdx.y;
    const int c = 8 * (blockIdx.x * kRowThreads + threadIdx.x);
    if (c >= cols) return;
    float a[8];
    load8(in + (int64_t)row * in_rs + c, a);
    if constexpr (KIND == TAH_ROWS_GELU_TANH) {
#pragma unroll
        for (int i = 0; i < 8; ++i) a[i] = gelu_tanh_exact(a[i]);
    } else if constexpr (KIND == TAH_ROWS_XIELU) {
#pragma unroll
        for (int i = 0; i < 8; ++i) a[i] = xielu(a[i], c0, c1);
    } else {
        float b[8];
        load8(in + (int64_t)row * in_rs + cols + c, b);
#pragma unroll
        for (int i = 0; i < 8; ++i) a[i] = KIND == TAH_ROWS_SILU_MUL ? silu_exact(a[i]) * b[i] : clamped_gate_exact(a[i], b[i], c0, c1);
    }
    store8(out + (int64_t)row * out_rs + c, a);
}

template <class E, bool GROUPS>
void launch_residual(const tah_residual_norm_args& p, hipStream_t st) {
    const int units = (p.cols / 8 + kRowThreads - 1) / kRowThreads;
    if (units <= 1) hipLaunchKernelGGL((residual_norm_kernel<E, 1, GROUPS>), dim3(p.rows), dim3(kRowThreads), 0, st, p);
    else if (units <= 2) hipLaunchKernelGGL((residual_norm_kernel<E, 2, GROUPS>), dim3(p.rows), dim3(kRowThreads), 0, st, p);
    else if (units <= 4) hipLaunchKernelGGL((residual_norm_kernel<E, 4, GROUPS>), dim3(p.rows), dim3(kRowThreads), 0, st, p);
    else hipLaunchKernelGGL((residual_norm_kernel<E, kMaxUnits, GROUPS>), dim3(p.rows), dim3(kRowThreads), 0, st, p);
}

template <class E>
void launch_conv(const void* h, const float* conv, void* state, const tah_portions& p, void* out, int cols, int taps, int nslots, hipStream_t st) {
    const bool few = taps <= kFewTaps;
    const dim3 grid((cols / 8 + kWave - 1) / kWave, p.rows / (few ? kFewRows : kConvRows) + p.nseq);
    auto* const f = few ? &conv_few_rows_kernel<E> : &conv_rows_kernel<E>;
    hipLaunchKernelGGL(f, grid, dim3(kWave), 0, st, static_cast<const E*>(h), conv, static_cast<E*>(state), p, static_cast<E*>(out), cols, taps, nslots);
}

template <class E>
void launch_activate(const void* in, int64_t in_rs, void* out, int64_t out_rs, int rows, int cols, int kind, float c0, float c1, hipStream_t st) {
    const dim3 grid((cols / 8 + kRowThreads - 1) / kRowThreads, rows);
    auto* const f = kind == TAH_ROWS_GELU_TANH ? &activate_rows_kernel<E, TAH_ROWS_GELU_TANH>
                    : kind == TAH_ROWS_XIELU   ? &activate_rows_kernel<E, TAH_ROWS_XIELU>
                    : kind == TAH_ROWS_SILU_MUL ? &activate_rows_kernel<E, TAH_ROWS_SILU_MUL>
                                                : &activate_rows_kernel<E, TAH_ROWS_CLAMPED_GATE>;
    hipLaunchKernelGGL(f, grid, dim3(kRowThreads), 0, st, static_cast<const E*>(in), in_rs, static_cast<E*>(out), out_rs, cols, c0, c1);
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
    if (a->groups <= 0 || a->groups > kMaxGroups || a->width % a->groups != 0 ||
        (a->groups > 1 && (a->group_cols % 8 != 0 || a->group_cols < a->width / a->groups || (int64_t)a->groups * a->group_cols > a->cols)))
        return TAH_E_SHAPE;
    if (a->conv && (a->taps <= 0 || a->nslots <= 0)) return TAH_E_SHAPE;
    if ((a->x_packed || a->normed_packed) && (a->rows > 32 || a->cols % 32 != 0)) return TAH_E_SHAPE;
    if (a->rows == 0) return TAH_OK;
    if (!a->x || ((a->y || a->experts) && !a->coef) || (a->experts && (!a->index || !a->weight))) return TAH_E_NULL;
    if ((a->normed || a->normed_packed || a->conv) && !a->next_coef) return TAH_E_NULL;
    if (a->conv && (!a->conv_state || !a->slot || !a->pos)) return TAH_E_NULL;
    const void* ptrs[] = {a->y, a->experts, a->coef, a->next_coef, a->x, a->xe, a->x_packed, a->normed, a->normed_packed, a->conv, a->conv_state};
    for (const void* q : ptrs)
        if (!aligned_16(q)) return TAH_E_ALIGN;
    if ((a->y && (a->y_row_stride % 8 != 0 || a->y_row_stride < a->cols)) ||
        (a->experts && (a->experts_row_stride % 8 != 0 || a->experts_row_stride < a->cols)))
        return TAH_E_ALIGN;
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (a->groups > 1) {
        if (a->dtype == TAH_DT_BF16) launch_residual<__bf16, true>(*a, st);
        else launch_residual<float, true>(*a, st);
    } else {
        if (a->dtype == TAH_DT_BF16) launch_residual<__bf16, false>(*a, st);
        else launch_residual<float, false>(*a, st);
    }
    return launch_status();
}

extern "C" int tah_conv_rows(const void* h, const float* conv, void* conv_state, const tah_portions* p, void* out, int32_t cols, int32_t taps,
                             int32_t nslots, int32_t dtype, tah_stream_t stream) {
    using namespace tah;
    if (!p) return TAH_E_NULL;
    if (p->rows < 0 || p->nseq < 0 || cols <= 0 || cols % 8 != 0 || taps <= 0 || taps - 1 > kConvRows || nslots <= 0 || !dtype_ok(dtype) ||
        p->rows / kFewRows + p->nseq > 65535)
        return TAH_E_SHAPE;
    if (p->rows == 0 || p->nseq == 0) return TAH_OK;
    if (!h || !conv || !conv_state || !out || !p->cu || !p->slot || !p->pos0) return TAH_E_NULL;
    if (!aligned_16(h) || !aligned_16(conv) || !aligned_16(conv_state) || !aligned_16(out)) return TAH_E_ALIGN;
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (dtype == TAH_DT_BF16) launch_conv<__bf16>(h, conv, conv_state, *p, out, cols, taps, nslots, st);
    else launch_conv<float>(h, conv, conv_state, *p, out, cols, taps, nslots, st);
    return launch_status();
}

extern "C" int tah_activate_rows(const void* in, int64_t in_rs, void* out, int64_t out_rs, int32_t rows, int32_t cols, int32_t kind,
                                 float c0, float c1, int32_t dtype, tah_stream_t stream) {
    using namespace tah;
    if (rows < 0 || rows > 65535 * 16 || cols < 0 || cols % 8 != 0 || !dtype_ok(dtype) || kind < TAH_ROWS_GELU_TANH || kind > TAH_ROWS_CLAMPED_GATE)
        return TAH_E_SHAPE;
    if (rows == 0 || cols == 0) return TAH_OK;
    if (!in || !out) return TAH_E_NULL;
    if (!aligned_16(in) || !aligned_16(out) || in_rs % 8 != 0 || out_rs % 8 != 0) return TAH_E_ALIGN;
    hipStream_t st = static_cast<hipStream_t>(stream);
    for (int32_t r = 0; r < rows; r += 65535) {  // (the grid's second dimension)
        const int32_t n = rows - r < 65535 ? rows - r : 65535;
        if (dtype == TAH_DT_BF16)
            launch_activate<__bf16>(static_cast<const __bf16*>(in) + r * in_rs, in_rs, static_cast<__bf16*>(out) + r * out_rs, out_rs, n, cols, kind, c0, c1, st);
        else
            launch_activate<float>(static_cast<const float*>(in) + r * in_rs, in_rs, static_cast<float*>(out) + r * out_rs, out_rs, n, cols, kind, c0, c1, st);
    }
    return launch_status();
}
