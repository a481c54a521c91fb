// Gated delta rule, gfx950.  Per head and token, with a float32 state S [dim, vdim] per sequence:
//     S = g S;   u = beta (v - S^T k);   S = S + k u^T;   o = S^T q.
// Both the step and the scan use  o = g S_old^T q + (k . q) u  for the read-out: S_old^T k and S_old^T q are then
// independent reductions of one pass over the state, and the write follows in a second pass over registers.
//
//  * delta_step_kernel: one token per row.  One workgroup per (row, head) holds the head's state in registers between
//    its load and its store -- the state crosses HBM once in each direction, which is all the step costs (64 KB each
//    way at 128 x 128) -- and does everything around it: short convolution on the projections, unit norms, decay,
//    output norm and gate.
//  * delta_prepare_kernel / delta_scan_kernel / delta_finish_kernel: portions of many tokens.  Columns of the state do
//    not interact, so a head is split over workgroups of 16 columns: a wave owns 4 columns, 16 lanes share a column's
//    rows and reduce over them with DPP row rotations; k and q of the next 16 tokens are fetched while the current 16
//    run.
//  * delta_chunk_kernel / delta_chunk_scan_kernel: the same for long portions, 32 tokens at a time, on the float32
//    matrix instruction.  With G_t the running sum of the decays' logarithms since the chunk's start and S the state
//    there, the chunk's writes u satisfy
//        u_t + beta_t sum_{s<t} exp(G_t - G_s) (k_t . k_s) u_s = beta_t (v_t - exp(G_t) S^T k_t),
//    a unit lower triangular system.  The first kernel solves it for all chunks at once, for the two parts of the right
//    hand side: U0 (from v) and W (from k), so that u = U0 - W S; and forms P[t][s] = exp(G_t - G_s) (q_t . k_s), s <= t.
//    The second walks the chunks of a sequence: u = U0 - W S, o_t = exp(G_t) S^T q_t + (P u)_t,
//    S <- exp(G_last) S + sum_s exp(G_last - G_s) k_s u_s^T, a workgroup holding sixteen columns of a head's state.
//  State and inputs are float32 throughout: no reduced-precision matrix instruction touches the recurrence.
//
// The convolution's inputs of the last `taps` tokens are kept as a ring (token p at p % taps): a step writes the entry
// that no row of the step reads, so workgroups that share channels need no order among themselves.
#include <hip/hip_runtime.h>

#include "mixer_device.h"

namespace tah {
namespace {

constexpr int kDeltaThreads = 256;
constexpr float kUnitEps = 1e-6f;

__device__ __forceinline__ int proj_col(const tah_delta_layer& L, int ch) {
    const int qk = L.kv_heads * L.dim;
    return ch < qk ? L.q_col + ch : (ch < 2 * qk ? L.k_col + ch - qk : L.v_col + ch - 2 * qk);
}
__device__ __forceinline__ float decay_log(const tah_delta_layer& L, float a, int h) {
    return -expf(L.a_log[h]) * softplus_exact(a + L.dt_bias[h]);
}

// LDS floats of delta_step_kernel
inline int step_lds(int dim, int vdim, int vec) { return 2 * dim + 2 * vdim + 2 * kDeltaThreads * vec + 16; }

// VEC: state columns per thread (4 or 1); NR: state rows per thread kept in registers, 0: any number, read twice.
template <class E, int VEC, int NR>
__global__ __launch_bounds__(kDeltaThreads) void delta_step_kernel(const tah_delta_layer L, const int32_t* slots, const int32_t* poss,
                                                                   E* out, int64_t out_rs, __bf16* out_packed, int out_cols) {
    HIP_DYNAMIC_SHARED(float, sm)
    float* const sq_ = sm;                     // q [dim]
    float* const sk_ = sq_ + L.dim;            // k [dim]
    float* const sv_ = sk_ + L.dim;            // v [vdim]
    float* const su_ = sv_ + L.vdim;           // u [vdim]
    float* const part = su_ + L.vdim;          // [2][row groups][columns]
    float* const red = part + 2 * kDeltaThreads * VEC;
    const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x;
    const int slot = slots[row], pos = poss[row];
    const int group = L.heads / L.kv_heads, kh = h / group;
    const int ct = (L.vdim + VEC - 1) / VEC;   // threads across the columns
    const int rg = kDeltaThreads / ct;         // row groups
    const bool dead = slot < 0 || slot >= L.nslots || pos < 0;
    const E* pr = static_cast<const E*>(L.proj) + (int64_t)row * L.proj_row_stride;
    if (dead) {  // a dropped row: zeros (uniform per workgroup)
        for (int v = tid; v < L.vdim; v += kDeltaThreads) {
            if (out) out[row * out_rs + h * L.vdim + v] = (E)0.f;
            if (out_packed) out_packed[rows_form_elem(row, h * L.vdim + v)] = (__bf16)0.f;
        }
    } else {
        const int c0 = (tid % ct) * VEC, r0 = tid / ct;
        const bool holder = r0 < rg;
        float* const S = L.state + (((int64_t)slot * L.heads + h) * L.dim) * L.vdim + c0;
        const bool fresh = pos == 0;
        float s[NR > 0 ? NR : 1][VEC];
        if constexpr (NR > 0) {
#pragma unroll
            for (int n = 0; n < NR; ++n) {
                const int i = r0 + rg * n;
#pragma unroll
                for (int e = 0; e < VEC; ++e) s[n][e] = 0.f;
                if (holder && i < L.dim && !fresh) {
                    if constexpr (VEC == 4) {
                        const f32x4 x = *reinterpret_cast<const f32x4*>(S + (int64_t)i * L.vdim);
#pragma unroll
                        for (int e = 0; e < 4; ++e) s[n][e] = x[e];
                    } else s[n][0] = S[(int64_t)i * L.vdim];
                }
            }
        }
        // short convolution of this head's q, k and v channels
        const int qk = L.kv_heads * L.dim, nch = 2 * qk + L.heads * L.vdim;
        E* const cs = static_cast<E*>(L.conv_state) + (int64_t)slot * L.taps * nch;
        for (int i = tid; i < 2 * L.dim + L.vdim; i += kDeltaThreads) {
            const int ch = i < L.dim ? kh * L.dim + i : (i < 2 * L.dim ? qk + kh * L.dim + i - L.dim : 2 * qk + h * L.vdim + i - 2 * L.dim);
            const E cur = pr[proj_col(L, ch)];
            const float* w = L.conv + (int64_t)ch * L.taps;
            float y = w[L.taps - 1] * (float)cur;
            for (int d = 1; d < L.taps; ++d)
                if (pos - d >= 0) y += w[L.taps - 1 - d] * (float)cs[(int64_t)((pos - d) % L.taps) * nch + ch];
            if (i >= 2 * L.dim || h % group == 0) cs[(int64_t)(pos % L.taps) * nch + ch] = cur;
            sq_[i] = silu_exact(y);  // q, k and v lie one after another
        }
        const float g = expf(decay_log(L, (float)pr[L.a_col + h], h));
        const float beta = sigmoid_exact((float)pr[L.b_col + h]);
        __syncthreads();
        float qq = 0.f, kk = 0.f, kq = 0.f;
        for (int i = tid; i < L.dim; i += kDeltaThreads) {
            const float q = sq_[i], k = sk_[i];
            qq += q * q;
            kk += k * k;
            kq += k * q;
        }
        qq = wave_sum(qq);
        kk = wave_sum(kk);
        kq = wave_sum(kq);
        if (tid % kWave == 0) {
            red[tid / kWave] = qq;
            red[4 + tid / kWave] = kk;
            red[8 + tid / kWave] = kq;
        }
        // S_old^T k and S_old^T q over this thread's rows (k and q not yet unit vectors: a factor, applied below)
        float ak[VEC], aq[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) ak[e] = aq[e] = 0.f;
        auto accumulate = [&](const float* x, int i) __attribute__((always_inline)) {
            const float k = sk_[i], q = sq_[i];
#pragma unroll
            for (int e = 0; e < VEC; ++e) {
                ak[e] += x[e] * k;
                aq[e] += x[e] * q;
            }
        };
        auto fetch = [&](int i, float* x) __attribute__((always_inline)) {
            if constexpr (VEC == 4) {
                const f32x4 y = *reinterpret_cast<const f32x4*>(S + (int64_t)i * L.vdim);
#pragma unroll
                for (int e = 0; e < 4; ++e) x[e] = y[e];
            } else x[0] = S[(int64_t)i * L.vdim];
        };
        if constexpr (NR > 0) {
#pragma unroll
            for (int n = 0; n < NR; ++n) {
                const int i = r0 + rg * n;
                if (i < L.dim) accumulate(s[n], i);
            }
        } else if (holder && !fresh) {
            for (int i = r0; i < L.dim; i += rg) {
                float x[VEC];
                fetch(i, x);
                accumulate(x, i);
            }
        }
        if (holder) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) {
                part[r0 * ct * VEC + c0 + e] = ak[e];
                part[kDeltaThreads * VEC + r0 * ct * VEC + c0 + e] = aq[e];
            }
        }
        __syncthreads();
        qq = (red[0] + red[1]) + (red[2] + red[3]);
        kk = (red[4] + red[5]) + (red[6] + red[7]);
        kq = (red[8] + red[9]) + (red[10] + red[11]);
        const float rq = 1.0f / sqrtf((float)L.dim) / sqrtf(qq + kUnitEps), rk = 1.0f / sqrtf(kk + kUnitEps);
        kq *= rq * rk;
        float oo = 0.f;
        for (int v = tid; v < L.vdim; v += kDeltaThreads) {
            float xk = 0.f, xq = 0.f;
            for (int r = 0; r < rg; ++r) {
                xk += part[r * ct * VEC + v];
                xq += part[kDeltaThreads * VEC + r * ct * VEC + v];
            }
            const float u = beta * (sv_[v] - g * (xk * rk));
            const float o = g * (xq * rq) + kq * u;
            su_[v] = u;
            sv_[v] = o;  // (each entry is read and rewritten by one thread)
            oo += o * o;
        }
        __syncthreads();
        oo = block_sum<kDeltaThreads / kWave>(oo, red);
        auto write = [&](const float* x, int i) __attribute__((always_inline)) {
            const float k = sk_[i] * rk;
            float y[VEC];
#pragma unroll
            for (int e = 0; e < VEC; ++e) y[e] = g * x[e] + k * su_[c0 + e];
            if constexpr (VEC == 4) *reinterpret_cast<f32x4*>(S + (int64_t)i * L.vdim) = f32x4{y[0], y[1], y[2], y[3]};
            else S[(int64_t)i * L.vdim] = y[0];
        };
        if constexpr (NR > 0) {
#pragma unroll
            for (int n = 0; n < NR; ++n) {
                const int i = r0 + rg * n;
                if (holder && i < L.dim) write(s[n], i);
            }
        } else if (holder) {
            for (int i = r0; i < L.dim; i += rg) {
                float x[VEC];
#pragma unroll
                for (int e = 0; e < VEC; ++e) x[e] = 0.f;
                if (!fresh) fetch(i, x);
                write(x, i);
            }
        }
        const float r = 1.0f / sqrtf(oo / (float)L.vdim + L.eps);
        for (int v = tid; v < L.vdim; v += kDeltaThreads) {
            const float y = sv_[v] * r * L.norm[v] * silu_exact((float)pr[L.gate_col + h * L.vdim + v]);
            if (out) out[row * out_rs + h * L.vdim + v] = (E)y;
            if (out_packed) out_packed[rows_form_elem(row, h * L.vdim + v)] = (__bf16)y;
        }
    }
    if (h == L.heads - 1) {
        for (int c = L.heads * L.vdim + tid; c < out_cols; c += kDeltaThreads) {
            if (out) out[row * out_rs + c] = (E)0.f;
            if (out_packed) out_packed[rows_form_elem(row, c)] = (__bf16)0.f;
        }
    }
}

// ---- portions ------------------------------------------------------------------------------------------------
constexpr int kPrepTokens = 16;  // tokens per wave

// blockIdx.y: q heads, k heads, v heads, then one for the gates.  NCH: 64-channel pieces of a head.
template <class E, int NCH>
__global__ __launch_bounds__(kDeltaThreads) void delta_prepare_kernel(const tah_delta_layer L, const tah_portions P, float* q, float* k, float* v,
                                                                      float* lg, float* beta) {
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave, hs = blockIdx.y;
    const int t0 = (blockIdx.x * (kDeltaThreads / kWave) + wave) * kPrepTokens;
    const E* proj = static_cast<const E*>(L.proj);
    const int qk = L.kv_heads * L.dim, nch = 2 * qk + L.heads * L.vdim;
    if (hs == 2 * L.kv_heads + L.heads) {
        for (int t = t0; t < t0 + kPrepTokens && t < P.rows; ++t) {
            const E* pr = proj + (int64_t)t * L.proj_row_stride;
            for (int h = lane; h < L.heads; h += kWave) {
                lg[(int64_t)t * L.heads + h] = decay_log(L, (float)pr[L.a_col + h], h);
                beta[(int64_t)t * L.heads + h] = sigmoid_exact((float)pr[L.b_col + h]);
            }
        }
        return;
    }
    const bool is_q = hs < L.kv_heads, is_v = hs >= 2 * L.kv_heads;
    const int d = is_v ? L.vdim : L.dim;
    const int head = is_q ? hs : (is_v ? hs - 2 * L.kv_heads : hs - L.kv_heads);
    const int ch0 = is_q ? head * L.dim : (is_v ? 2 * qk + head * L.vdim : qk + head * L.dim);
    const int col0 = (is_q ? L.q_col : (is_v ? L.v_col : L.k_col)) + head * d;
    float* const dst = is_q ? q : (is_v ? v : k);
    const int nheads = is_v ? L.heads : L.kv_heads;
    const float out_scale = is_q ? 1.0f / sqrtf((float)L.dim) : 1.0f;
    for (int t = t0; t < t0 + kPrepTokens && t < P.rows; ++t) {
        const int b = P.row_seq[t];
        const int first = P.cu[b], pos = P.pos0[b] + t - first, slot = P.slot[b];
        const E* cs = static_cast<const E*>(L.conv_state) + (int64_t)(slot < 0 ? 0 : slot) * L.taps * nch;
        float y[NCH], ss = 0.f;
#pragma unroll
        for (int n = 0; n < NCH; ++n) {
            const int c = lane + kWave * n;
            y[n] = 0.f;
            if (c < d) {
                const float* w = L.conv + (int64_t)(ch0 + c) * L.taps;
                for (int j = 0; j < L.taps; ++j) {
                    float x = 0.f;
                    if (t - j >= first) x = (float)proj[(int64_t)(t - j) * L.proj_row_stride + col0 + c];
                    else if (pos - j >= 0 && slot >= 0) x = (float)cs[(int64_t)((pos - j) % L.taps) * nch + ch0 + c];
                    y[n] += w[L.taps - 1 - j] * x;
                }
                y[n] = silu_exact(y[n]);
            }
            ss += y[n] * y[n];
        }
        float r = 1.0f;
        if (!is_v) r = out_scale / sqrtf(wave_sum(ss) + kUnitEps);
#pragma unroll
        for (int n = 0; n < NCH; ++n) {
            const int c = lane + kWave * n;
            if (c < d) dst[((int64_t)t * nheads + head) * d + c] = y[n] * r;
        }
    }
}

__device__ __forceinline__ float silu_act(float x, __bf16*) { return x * fast_rcp(1.0f + fast_exp2(-x * kLog2e)); }  // an activation of a bf16 model
__device__ __forceinline__ float silu_act(float x, float*) { return silu_exact(x); }

// The same for heads of whole eight-channel units, a power of two of them: a thread owns eight channels and keeps the
// last inputs of its convolutions in registers; the lanes of a q or k head add up their squares.  grid.y: 256 units
// each, then one for the gates.
template <class E, int TAPS>
__global__ __launch_bounds__(kDeltaThreads) void delta_prepare_units_kernel(const tah_delta_layer L, const tah_portions P, float* q, float* k, float* v,
                                                                            float* lg, float* beta) {
    const int tid = threadIdx.x, t0 = blockIdx.x * kPrepTokens, tn = t0 + kPrepTokens < P.rows ? t0 + kPrepTokens : P.rows;
    const E* const proj = static_cast<const E*>(L.proj);
    if (blockIdx.y == gridDim.y - 1) {
        for (int i = tid; i < (tn - t0) * L.heads; i += kDeltaThreads) {
            const int t = t0 + i / L.heads, h = i % L.heads;
            const E* pr = proj + (int64_t)t * L.proj_row_stride;
            lg[(int64_t)t * L.heads + h] = decay_log(L, (float)pr[L.a_col + h], h);
            beta[(int64_t)t * L.heads + h] = sigmoid_exact((float)pr[L.b_col + h]);
        }
        return;
    }
    const int qk = L.kv_heads * L.dim, nch = 2 * qk + L.heads * L.vdim;
    int ch = 8 * (blockIdx.y * kDeltaThreads + tid);
    const bool on = ch < nch;
    ch = on ? ch : 0;  // (lanes past the end take part in the sums of nobody)
    const bool is_q = ch < qk, is_v = ch >= 2 * qk;
    const E* const src = proj + proj_col(L, ch);
    float* const dst = is_q ? q + ch : (is_v ? v + ch - 2 * qk : k + ch - qk);
    const int64_t dst_rs = is_v ? (int64_t)L.heads * L.vdim : qk;
    const int lanes = L.dim / 8;  // of a q or k head
    const float scale = is_q ? 1.0f / sqrtf((float)L.dim) : 1.0f;
    float w[TAPS][8], hist[TAPS > 1 ? TAPS - 1 : 1][8];
#pragma unroll
    for (int i = 0; i < 8; ++i)
#pragma unroll
        for (int j = 0; j < TAPS; ++j) w[j][i] = L.conv[(int64_t)(ch + i) * TAPS + j];
    constexpr int kAhead = 4;
    for (int tb = t0; tb < tn; tb += kAhead) {
        float x[kAhead][8];
#pragma unroll
        for (int a = 0; a < kAhead; ++a) load8(src + (int64_t)(tb + a < tn ? tb + a : tn - 1) * L.proj_row_stride, x[a]);
#pragma unroll
        for (int a = 0; a < kAhead; ++a) {
            const int t = tb + a;
            if (t >= tn) break;
            const int b = P.row_seq[t], first = P.cu[b];
            if (t == t0 || t == first) {  // what came before: earlier rows of the portion, the state, or nothing
                const int pos = P.pos0[b] + t - first, slot = P.slot[b];
                const E* cs = static_cast<const E*>(L.conv_state) + (int64_t)(slot < 0 ? 0 : slot) * TAPS * nch + ch;
#pragma unroll
                for (int j = 1; j < TAPS; ++j) {
                    if (t - j >= first) load8(src + (int64_t)(t - j) * L.proj_row_stride, hist[j - 1]);
                    else if (pos - j >= 0 && slot >= 0) load8(cs + (int64_t)((pos - j) % TAPS) * nch, hist[j - 1]);
                    else {
#pragma unroll
                        for (int i = 0; i < 8; ++i) hist[j - 1][i] = 0.f;
                    }
                }
            }
            float y[8], ss = 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                float s = w[TAPS - 1][i] * x[a][i];
#pragma unroll
                for (int j = 1; j < TAPS; ++j) s += w[TAPS - 1 - j][i] * hist[j - 1][i];
                y[i] = silu_act(s, static_cast<E*>(nullptr));
                ss += y[i] * y[i];
            }
            for (int m = 1; m < lanes; m <<= 1) ss += __shfl_xor(ss, m);
            const float r = is_v ? 1.0f : scale / sqrtf(ss + kUnitEps);
#pragma unroll
            for (int i = 0; i < 8; ++i) y[i] *= r;
            if (on) store8(dst + (int64_t)t * dst_rs, y);
#pragma unroll
            for (int j = TAPS - 1; j > 1; --j)
#pragma unroll
                for (int i = 0; i < 8; ++i) hist[j - 1][i] = hist[j - 2][i];
            if constexpr (TAPS > 1) {
#pragma unroll
                for (int i = 0; i < 8; ++i) hist[0][i] = x[a][i];
            }
        }
    }
}

// The convolution's inputs of a portion's last tokens, into the ring.  (After delta_prepare_kernel has read the old ones.)
template <class E>
__global__ __launch_bounds__(kDeltaThreads) void conv_tail_kernel(const tah_delta_layer L, const tah_portions P) {
    const int b = blockIdx.y, slot = P.slot[b];
    const int nch = 2 * L.kv_heads * L.dim + L.heads * L.vdim, ch = blockIdx.x * kDeltaThreads + threadIdx.x;
    if (ch >= nch || slot < 0 || slot >= L.nslots) return;
    const int first = P.cu[b], last = P.cu[b + 1] - 1, pos_last = P.pos0[b] + last - first;
    E* cs = static_cast<E*>(L.conv_state) + (int64_t)slot * L.taps * nch + ch;
    const E* src = static_cast<const E*>(L.proj) + proj_col(L, ch);
    for (int d = 0; d < L.taps && last - d >= first; ++d) cs[(int64_t)((pos_last - d) % L.taps) * nch] = src[(int64_t)(last - d) * L.proj_row_stride];
}

constexpr int kScanTokens = 16, kScanCols = 16;

// sum over the 16 lanes of a DPP row, in every lane of it
__device__ __forceinline__ float row16_sum(float x) {
    x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x128, 0xf, 0xf, false));
    x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x124, 0xf, 0xf, false));
    x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x122, 0xf, 0xf, false));
    x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x121, 0xf, 0xf, false));
    return x;
}

// grid (column blocks of 16, heads, sequences).  NB: 64-row pieces of the state; lane r of 16 holds rows 64 b + 4 r ... + 3.
template <int NB>
__global__ __launch_bounds__(kDeltaThreads) void delta_scan_kernel(const tah_delta_layer L, const tah_portions P, const float* q, const float* k,
                                                                   const float* v, const float* lg, const float* beta, float* o) {
    constexpr int kDim = 64 * NB;
    __shared__ __align__(16) float kb[kScanTokens][kDim], qb[kScanTokens][kDim];
    __shared__ float vb[kScanTokens][kScanCols], ob[kScanTokens][kScanCols], gb[kScanTokens], bb[kScanTokens], kqb[kScanTokens];
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
    const int h = blockIdx.y, b = blockIdx.z, kh = h / (L.heads / L.kv_heads);
    const int r = lane % 16, lc = wave * 4 + lane / 16, col = blockIdx.x * kScanCols + lc;
    const int first = P.cu[b], n = P.cu[b + 1] - first, slot = P.slot[b], pos0 = P.pos0[b];
    if (n <= 0 || slot < 0 || slot >= L.nslots) return;
    float* const S = L.state + ((int64_t)slot * L.heads + h) * L.dim * L.vdim;
    float s[NB][4];
#pragma unroll
    for (int x = 0; x < NB; ++x)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int i = 64 * x + 4 * r + e;
            s[x][e] = (pos0 > 0 && col < L.vdim && i < L.dim) ? S[(int64_t)i * L.vdim + col] : 0.f;
        }
    // a thread's share of 16 tokens: NB four-row pieces of k and of q, one v, and (32 threads) a gate
    f32x4 nk[NB], nq[NB];
    float nv = 0.f, ng = 0.f;
    const bool vec = L.dim % 4 == 0;
    auto fetch = [&](int c0) __attribute__((always_inline)) {
#pragma unroll
        for (int x = 0; x < NB; ++x) {
            const int u = tid + kDeltaThreads * x, t = u / (kDim / 4), i = 4 * (u % (kDim / 4));
            nk[x] = nq[x] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (c0 + t < n && i < L.dim) {
                const int64_t at = ((int64_t)(first + c0 + t) * L.kv_heads + kh) * L.dim + i;
                if (vec) {
                    nk[x] = *reinterpret_cast<const f32x4*>(k + at);
                    nq[x] = *reinterpret_cast<const f32x4*>(q + at);
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (i + e < L.dim) {
                            nk[x][e] = k[at + e];
                            nq[x][e] = q[at + e];
                        }
                }
            }
        }
        const int t = tid / kScanCols, c = blockIdx.x * kScanCols + tid % kScanCols;
        nv = (c0 + t < n && c < L.vdim) ? v[((int64_t)(first + c0 + t) * L.heads + h) * L.vdim + c] : 0.f;
        if (tid < 2 * kScanTokens) {
            const int tt = tid % kScanTokens;
            ng = c0 + tt < n ? (tid < kScanTokens ? lg : beta)[(int64_t)(first + c0 + tt) * L.heads + h] : 0.f;
        }
    };
    fetch(0);
    for (int c0 = 0; c0 < n; c0 += kScanTokens) {
#pragma unroll
        for (int x = 0; x < NB; ++x) {
            const int u = tid + kDeltaThreads * x, t = u / (kDim / 4), i = 4 * (u % (kDim / 4));
            *reinterpret_cast<f32x4*>(&kb[t][i]) = nk[x];
            *reinterpret_cast<f32x4*>(&qb[t][i]) = nq[x];
        }
        vb[tid / kScanCols][tid % kScanCols] = nv;
        if (tid < kScanTokens) gb[tid] = expf(ng);
        else if (tid < 2 * kScanTokens) bb[tid - kScanTokens] = ng;
        __syncthreads();
        if (c0 + kScanTokens < n) fetch(c0 + kScanTokens);
        {   // k . q of four tokens per wave, sixteen lanes each
            const int t = wave * 4 + lane / 16;
            float x = 0.f;
#pragma unroll
            for (int e = 0; e < kDim / 64; ++e) {
                const f32x4 a = *reinterpret_cast<const f32x4*>(&kb[t][64 * e + 4 * r]), c = *reinterpret_cast<const f32x4*>(&qb[t][64 * e + 4 * r]);
                x += (a[0] * c[0] + a[1] * c[1]) + (a[2] * c[2] + a[3] * c[3]);
            }
            x = row16_sum(x);
            if (r == 0) kqb[t] = x;
        }
        __syncthreads();
        const int m = n - c0 < kScanTokens ? n - c0 : kScanTokens;
        for (int t = 0; t < m; ++t) {
            f32x4 kt[NB];
            float xk = 0.f, xq = 0.f;
#pragma unroll
            for (int x = 0; x < NB; ++x) {
                kt[x] = *reinterpret_cast<const f32x4*>(&kb[t][64 * x + 4 * r]);
                const f32x4 qt = *reinterpret_cast<const f32x4*>(&qb[t][64 * x + 4 * r]);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    xk += s[x][e] * kt[x][e];
                    xq += s[x][e] * qt[e];
                }
            }
            xk = row16_sum(xk);
            xq = row16_sum(xq);
            const float g = gb[t];
            const float u = bb[t] * (vb[t][lc] - g * xk);
            if (r == 0) ob[t][lc] = g * xq + kqb[t] * u;
#pragma unroll
            for (int x = 0; x < NB; ++x)
#pragma unroll
                for (int e = 0; e < 4; ++e) s[x][e] = g * s[x][e] + kt[x][e] * u;
        }
        __syncthreads();
        {
            const int t = tid / kScanCols, c = blockIdx.x * kScanCols + tid % kScanCols;
            if (t < m && c < L.vdim) o[((int64_t)(first + c0 + t) * L.heads + h) * L.vdim + c] = ob[t][tid % kScanCols];
        }
    }
#pragma unroll
    for (int x = 0; x < NB; ++x)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int i = 64 * x + 4 * r + e;
            if (col < L.vdim && i < L.dim) S[(int64_t)i * L.vdim + col] = s[x][e];
        }
}

// ---- long portions, 32 tokens at a time -------------------------------------------------------------------------
constexpr int kChunk = 32;
constexpr int kChunkThreads = 128;

__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// running sums of a chunk's decay logarithms: lane t < 32 ends with G_t (lanes of 32 and more repeat lane 31; rows past the
// end do not decay)
__device__ __forceinline__ float chunk_decay(const float* lg, int heads, int h, int row0, int n, int lane) {
    float x = lane < n ? lg[(int64_t)(row0 + lane) * heads + h] : 0.f;
#pragma unroll
    for (int o = 1; o < kChunk; o <<= 1) {
        const float y = __shfl_up(x, o);
        if (lane >= o && lane < kChunk) x += y;
    }
    return __shfl(x, lane < kChunk ? lane : kChunk - 1);
}

// what the first kernel leaves per (chunk, head), in floats: W [32][dim], U0 [32][vdim], P [32][32], and
// exp(G_t), exp(G_last - G_t) [32] each
__device__ __host__ __forceinline__ int chunk_floats(int dim, int vdim) { return kChunk * (dim + vdim + kChunk + 2); }

// grid (chunk slots, heads).  NT: 16-wide tiles of dim.
template <int NT>
__global__ __launch_bounds__(kChunkThreads) void delta_chunk_kernel(const tah_delta_layer L, const tah_portions P, const float* q, const float* k,
                                                                    const float* v, const float* lg, const float* beta, float* work) {
    constexpr int D = 16 * NT, kStride = D + 4;
    __shared__ __align__(16) float kl[kChunk][kStride], ql[kChunk][kStride];
    __shared__ __align__(16) float al[kChunk][kChunk + 4];
    __shared__ float gl[kChunk], bl[kChunk], be[kChunk];  // G, beta, beta exp(G)
    int slot = blockIdx.x, b = 0, row0 = 0, row_end = 0;
    if (!find_tile(P.cu, P.nseq, kChunk, slot, b, row0, row_end)) return;
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, c = lane % 16, g = lane / 16;
    const int h = blockIdx.y, kh = h / (L.heads / L.kv_heads), n = row_end - row0;
    float* const out = work + ((int64_t)blockIdx.x * L.heads + h) * chunk_floats(D, L.vdim);
    float* const out_u = out + kChunk * D;
    float* const out_p = out_u + kChunk * L.vdim;
    for (int u = tid; u < kChunk * D / 4; u += kChunkThreads) {
        const int t = u / (D / 4), i = 4 * (u % (D / 4));
        f32x4 x = {0.f, 0.f, 0.f, 0.f}, y = x;
        if (t < n) {
            const int64_t at = ((int64_t)(row0 + t) * L.kv_heads + kh) * D + i;
            x = *reinterpret_cast<const f32x4*>(k + at);
            y = *reinterpret_cast<const f32x4*>(q + at);
        }
        *reinterpret_cast<f32x4*>(&kl[t][i]) = x;
        *reinterpret_cast<f32x4*>(&ql[t][i]) = y;
    }
    if (wave == 0) {
        const float x = chunk_decay(lg, L.heads, h, row0, n, lane);
        const float last = __shfl(x, kChunk - 1);
        if (lane < kChunk) {
            gl[lane] = x;
            bl[lane] = lane < n ? beta[(int64_t)(row0 + lane) * L.heads + h] : 0.f;
            be[lane] = bl[lane] * expf(x);
            out_p[kChunk * kChunk + lane] = expf(x);
            out_p[kChunk * kChunk + kChunk + lane] = expf(last - x);
        }
    }
    __syncthreads();
    // six tiles of 16 x 16: the lower ones of K K^T and of Q K^T
    for (int id = wave; id < 6; id += kChunkThreads / kWave) {
        const bool is_p = id >= 3;
        const int i = id % 3 == 0 ? 0 : 1, j = id % 3 == 2 ? 1 : 0;
        const float* const a = is_p ? &ql[16 * i + c][4 * g] : &kl[16 * i + c][4 * g];
        const float* const bb = &kl[16 * j + c][4 * g];
        f32x4 acc = {0.f, 0.f, 0.f, 0.f}, acc2 = acc;
#pragma unroll
        for (int s = 0; s < NT; ++s) {
            const f32x4 x = *reinterpret_cast<const f32x4*>(a + 16 * s), y = *reinterpret_cast<const f32x4*>(bb + 16 * s);
#pragma unroll
            for (int e = 0; e < 4; e += 2) {
                acc = mfma_f32(x[e], y[e], acc);
                acc2 = mfma_f32(x[e + 1], y[e + 1], acc2);
            }
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = 16 * i + 4 * g + r, s = 16 * j + c;
            const float w = t >= s ? (acc[r] + acc2[r]) * expf(gl[t] - gl[s]) : 0.f;
            if (is_p) out_p[t * kChunk + s] = w;
            else al[t][s] = bl[t] * w;
        }
    }
    if (wave == kChunkThreads / kWave - 1) {  // the tile above the diagonal
#pragma unroll
        for (int r = 0; r < 4; ++r) out_p[(4 * g + r) * kChunk + 16 + c] = 0.f;
    }
    __syncthreads();
    // the triangular system, two columns of the right hand sides per thread (a matrix entry, read from LDS by all lanes at
    // once, then serves two): columns of v, then of k
    const int cols = L.vdim + D;  // (even)
    for (int col = tid; col < cols / 2; col += kChunkThreads) {
        float x[2][kChunk];
#pragma unroll
        for (int y = 0; y < 2; ++y) {
            const int i = col + y * (cols / 2);
            if (i >= L.vdim) {
#pragma unroll
                for (int t = 0; t < kChunk; ++t) x[y][t] = be[t] * kl[t][i - L.vdim];
            } else {
#pragma unroll
                for (int t = 0; t < kChunk; ++t) x[y][t] = bl[t] * v[((int64_t)(row0 + (t < n ? t : n - 1)) * L.heads + h) * L.vdim + i];  // (beta is 0 past the end)
            }
        }
#pragma unroll
        for (int t = 1; t < kChunk; ++t) {
            if (t % 2) asm volatile("" ::: "memory");  // (the matrix is read row by row, not all of it into registers)
#pragma unroll
            for (int s4 = 0; s4 < (t + 3) / 4; ++s4) {
                const f32x4 a = *reinterpret_cast<const f32x4*>(&al[t][4 * s4]);
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (4 * s4 + e < t) {
                        x[0][t] -= a[e] * x[0][4 * s4 + e];
                        x[1][t] -= a[e] * x[1][4 * s4 + e];
                    }
            }
        }
#pragma unroll
        for (int y = 0; y < 2; ++y) {
            const int i = col + y * (cols / 2);
            float* const dst = i >= L.vdim ? out + i - L.vdim : out_u + i;
            const int ds = i >= L.vdim ? D : L.vdim;
#pragma unroll
            for (int t = 0; t < kChunk; ++t) dst[t * ds] = x[y][t];
        }
    }
}

// One workgroup per 16-column slice of a (sequence, head).  Workgroups go to the XCDs round robin: the slices of a head are
// placed on one XCD, whose L2 then fetches what they share once.  Waves 0 and 1 form u, waves 2 and 3 the results; a
// wave holds 16 kOwn rows of the state's slice: register r of lane (c, g) of its tile i is S[kOwn (16 wave + c) + i][4 g + r].
template <int NT>
__global__ __launch_bounds__(kDeltaThreads) void delta_chunk_scan_kernel(const tah_delta_layer L, const tah_portions P, const float* q, const float* k,
                                                                         const float* work, float* o) {
    constexpr int D = 16 * NT, kOwn = (NT + 3) / 4;
    typedef __attribute__((__vector_size__(kOwn * sizeof(float)))) float own_t;
    __shared__ __align__(16) float st[16][D + 4];           // S^T
    __shared__ __align__(16) float ut[16][kChunk + 4], us[16][kChunk + 4];  // u^T, and times exp(G_last - G_s)
    const int lane = threadIdx.x % kWave, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave), c = lane % 16, g = lane / 16;
    const int slices = L.vdim / 16, item = blockIdx.x / 8 / slices * 8 + blockIdx.x % 8;
    if (item >= L.heads * P.nseq) return;
    const int h = item % L.heads, b = item / L.heads, kh = h / (L.heads / L.kv_heads), v0 = 16 * (blockIdx.x / 8 % slices);
    const int first = P.cu[b], n = P.cu[b + 1] - first, slot = P.slot[b];
    if (n <= 0 || slot < 0 || slot >= L.nslots) return;
    int64_t chunk0 = 0;  // chunks of the sequences before
    for (int x = 0; x < b; ++x) chunk0 += (P.cu[x + 1] - P.cu[x] + kChunk - 1) / kChunk;
    const int wf = chunk_floats(D, L.vdim), rs = L.kv_heads * D;
    const bool holds = wave * kOwn < NT, fresh = P.pos0[b] == 0;
    const int own = holds ? kOwn * (16 * wave + c) : 0;  // its first row of the state
    float* const S = L.state + ((int64_t)slot * L.heads + h) * D * L.vdim + (int64_t)own * L.vdim + v0 + 4 * g;
    f32x4 s[kOwn];
    auto publish = [&]() __attribute__((always_inline)) {
        if (!holds) return;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            own_t y;
#pragma unroll
            for (int i = 0; i < kOwn; ++i) y[i] = s[i][r];
            *reinterpret_cast<own_t*>(&st[4 * g + r][own]) = y;
        }
    };
#pragma unroll
    for (int i = 0; i < kOwn; ++i)
        s[i] = holds && !fresh ? *reinterpret_cast<const f32x4*>(S + (int64_t)i * L.vdim) : f32x4{0.f, 0.f, 0.f, 0.f};
    publish();
    const bool former = wave < 2;
    const int tr = 16 * (wave % 2);  // the wave's rows of a chunk
    struct Loads {
        f32x4 a[NT], p[2], u0, gam;
        own_t kk[8];
        float all;
    } buf0, buf1;
    const int chunks = (n + kChunk - 1) / kChunk;
    // (uniform bases and 32-bit offsets; no branch around or between the loads of a chunk: the compiler then knows which are
    // still on their way)
    auto fetch = [&](int ch, Loads& x) __attribute__((always_inline)) {
        const int row0 = first + ch * kChunk, m = n - ch * kChunk < kChunk ? n - ch * kChunk : kChunk;
        const float* const w = work + ((chunk0 + ch) * L.heads + h) * wf;
        const float* const wu = w + kChunk * D + v0;
        const float* const wp = w + kChunk * (D + L.vdim);
        const float* const wg = wp + kChunk * kChunk;
        const float* const kb = k + ((int64_t)row0 * L.kv_heads + kh) * D;
        const float* const ab = former ? w : q + ((int64_t)row0 * L.kv_heads + kh) * D;
        const unsigned ao = former ? (tr + c) * D : (tr + c < m ? tr + c : m - 1) * rs;
#pragma unroll
        for (int i = 0; i < NT; ++i) x.a[i] = *reinterpret_cast<const f32x4*>(ab + (ao + 16 * i + 4 * g));
#pragma unroll
        for (int r = 0; r < 4; ++r) x.u0[r] = wu[(unsigned)((tr + 4 * g + r) * L.vdim + c)];
#pragma unroll
        for (int i = 0; i < 2; ++i) x.p[i] = *reinterpret_cast<const f32x4*>(wp + (unsigned)((tr + c) * kChunk + 16 * i + 4 * g));
        x.gam = *reinterpret_cast<const f32x4*>(wg + (unsigned)((former ? kChunk : 0) + tr + 4 * g));
        x.all = wg[kChunk - 1];  // exp(G_last)
#pragma unroll
        for (int y = 0; y < 8; ++y) {
            const int tk = 16 * (y / 4) + 4 * g + y % 4;
            x.kk[y] = *reinterpret_cast<const own_t*>(kb + (unsigned)((tk < m ? tk : m - 1) * rs + own));
        }
    };
    // the results of a chunk are written during the next one, so that no load waits behind a store just issued
    f32x4 done = {0.f, 0.f, 0.f, 0.f};
    auto flush = [&](int ch) __attribute__((always_inline)) {
        if (former || ch < 0) return;
        float* const ob = o + ((int64_t)(first + ch * kChunk) * L.heads + h) * L.vdim + v0;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = tr + 4 * g + r;
            if (ch * kChunk + t < n) ob[(unsigned)(t * L.heads * L.vdim + c)] = done[r];
        }
    };
    auto step = [&](int ch, const Loads& cur, Loads& nxt) __attribute__((always_inline)) {
        fetch(ch + 1 < chunks ? ch + 1 : ch, nxt);
        __builtin_amdgcn_sched_barrier(0);
        // W S or Q S
        f32x4 x0 = {0.f, 0.f, 0.f, 0.f}, x1 = x0;
#pragma unroll
        for (int i = 0; i < NT; ++i) {
            const f32x4 y = *reinterpret_cast<const f32x4*>(&st[c][16 * i + 4 * g]);
            x0 = mfma_f32(cur.a[i][0], y[0], x0);
            x1 = mfma_f32(cur.a[i][1], y[1], x1);
            x0 = mfma_f32(cur.a[i][2], y[2], x0);
            x1 = mfma_f32(cur.a[i][3], y[3], x1);
        }
        flush(ch - 1);
        f32x4 res;
        if (former) {
            f32x4 u, w;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                u[r] = cur.u0[r] - (x0[r] + x1[r]);
                w[r] = u[r] * cur.gam[r];
            }
            *reinterpret_cast<f32x4*>(&ut[c][tr + 4 * g]) = u;
            *reinterpret_cast<f32x4*>(&us[c][tr + 4 * g]) = w;
        } else {
#pragma unroll
            for (int r = 0; r < 4; ++r) res[r] = (x0[r] + x1[r]) * cur.gam[r];
        }
        __syncthreads();
        f32x4 uw[2];
#pragma unroll
        for (int i = 0; i < 2; ++i) uw[i] = *reinterpret_cast<const f32x4*>(&us[c][16 * i + 4 * g]);
#pragma unroll
        for (int i = 0; i < kOwn; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) s[i][r] *= cur.all;
#pragma unroll
        for (int y = 0; y < 8; ++y)
#pragma unroll
            for (int i = 0; i < kOwn; ++i) s[i] = mfma_f32(uw[y / 4][y % 4], cur.kk[y][i], s[i]);
        publish();
        if (!former) {
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                const f32x4 u = *reinterpret_cast<const f32x4*>(&ut[c][16 * i + 4 * g]);
#pragma unroll
                for (int e = 0; e < 4; ++e) res = mfma_f32(cur.p[i][e], u[e], res);
            }
            done = res;
        }
        __syncthreads();
    };
    fetch(0, buf0);
    __syncthreads();
    for (int ch = 0;;) {
        step(ch, buf0, buf1);
        if (++ch == chunks) break;
        step(ch, buf1, buf0);
        if (++ch == chunks) break;
    }
    flush(chunks - 1);
#pragma unroll
    for (int i = 0; i < kOwn; ++i)
        if (holds) *reinterpret_cast<f32x4*>(S + (int64_t)i * L.vdim) = s[i];
}

// one wave per (row, head)
template <class E>
__global__ __launch_bounds__(kDeltaThreads) void delta_finish_kernel(const tah_delta_layer L, const float* o, int64_t items, E* out, int64_t out_rs,
                                                                     int out_cols) {
    const int lane = threadIdx.x % kWave;
    const int64_t it = (int64_t)blockIdx.x * (kDeltaThreads / kWave) + threadIdx.x / kWave;
    if (it >= items) return;
    const int64_t row = it / L.heads;
    const int h = (int)(it % L.heads);
    const float* x = o + it * L.vdim;
    float ss = 0.f;
    for (int v = lane; v < L.vdim; v += kWave) ss += x[v] * x[v];
    const float r = 1.0f / sqrtf(wave_sum(ss) / (float)L.vdim + L.eps);
    const E* gate = static_cast<const E*>(L.proj) + row * L.proj_row_stride + L.gate_col + h * L.vdim;
    E* y = out + row * out_rs;
    for (int v = lane; v < L.vdim; v += kWave) y[h * L.vdim + v] = (E)(x[v] * r * L.norm[v] * silu_exact((float)gate[v]));
    if (h == L.heads - 1)
        for (int c = L.heads * L.vdim + lane; c < out_cols; c += kWave) y[c] = (E)0.f;
}

// the same for values of whole eight-column units, a power of two of them per head: one thread per unit
template <class E>
__global__ __launch_bounds__(kDeltaThreads) void delta_finish_units_kernel(const tah_delta_layer L, const float* o, int64_t units, E* out, int64_t out_rs,
                                                                           int out_cols) {
    int64_t u = (int64_t)blockIdx.x * kDeltaThreads + threadIdx.x;
    const bool on = u < units;
    u = on ? u : units - 1;
    const int per_row = L.heads * L.vdim / 8, lanes = L.vdim / 8;
    const int64_t row = u / per_row;
    const int c = 8 * (int)(u % per_row);
    float x[8], gate[8], nw[8], ss = 0.f;
    load8(o + row * L.heads * L.vdim + c, x);
    load8(static_cast<const E*>(L.proj) + row * L.proj_row_stride + L.gate_col + c, gate);
    load8(L.norm + c % L.vdim, nw);
#pragma unroll
    for (int i = 0; i < 8; ++i) ss += x[i] * x[i];
    for (int m = 1; m < lanes; m <<= 1) ss += __shfl_xor(ss, m);
    const float r = 1.0f / sqrtf(ss / (float)L.vdim + L.eps);
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] = x[i] * r * nw[i] * silu_act(gate[i], static_cast<E*>(nullptr));
    if (!on) return;
    store8(out + row * out_rs + c, x);
    if (c + 8 == L.heads * L.vdim)
        for (int i = c + 8; i < out_cols; ++i) out[row * out_rs + i] = (E)0.f;
}

// a head of d channels is whole eight-channel units, a power of two of them, at most a wave's lanes
bool in_units(int d) { return d % 8 == 0 && d <= 512 && (d & (d - 1)) == 0; }
// projection rows that eight-element loads can address
bool unit_rows(const tah_delta_layer& L) {
    return aligned_16(L.proj) && L.proj_row_stride % 8 == 0 && aligned_16(L.conv_state) && aligned_16(L.norm) && L.q_col % 8 == 0 && L.k_col % 8 == 0 &&
           L.v_col % 8 == 0 && L.gate_col % 8 == 0;
}

int check_layer(const tah_delta_layer* L) {
    if (!L) return TAH_E_NULL;
    if (L->heads <= 0 || L->kv_heads <= 0 || L->heads % L->kv_heads != 0 || L->dim <= 0 || L->vdim <= 0 || L->taps <= 0 || L->nslots <= 0 ||
        (L->dtype != TAH_DT_BF16 && L->dtype != TAH_DT_F32) || L->heads > 65535)
        return TAH_E_SHAPE;
    if (L->dim > 256 || L->vdim > 512) return TAH_E_SHAPE;
    if (!L->proj || !L->conv || !L->a_log || !L->dt_bias || !L->norm || !L->conv_state || !L->state) return TAH_E_NULL;
    if (!aligned_16(L->state)) return TAH_E_ALIGN;
    return TAH_OK;
}
int check_portions(const tah_portions* p) {
    if (!p) return TAH_E_NULL;
    if (p->nseq < 0 || p->rows < 0 || p->nseq > 65535) return TAH_E_SHAPE;
    if (p->nseq > 0 && p->rows > 0 && (!p->cu || !p->slot || !p->pos0 || !p->row_seq)) return TAH_E_NULL;
    return TAH_OK;
}

template <class E, int VEC, int NR>
void launch_step(const tah_delta_layer& L, const int32_t* slot, const int32_t* pos, int rows, void* out, int64_t rs, void* packed, int cols,
                 hipStream_t st) {
    hipLaunchKernelGGL((delta_step_kernel<E, VEC, NR>), dim3(L.heads, rows), dim3(kDeltaThreads), step_lds(L.dim, L.vdim, VEC) * sizeof(float), st,
                       L, slot, pos, static_cast<E*>(out), rs, static_cast<__bf16*>(packed), cols);
}
template <class E>
void dispatch_step(const tah_delta_layer& L, const int32_t* slot, const int32_t* pos, int rows, void* out, int64_t rs, void* packed, int cols,
                   hipStream_t st) {
    if (L.vdim % 4 == 0) {
        const int rg = kDeltaThreads / (L.vdim / 4), nr = (L.dim + rg - 1) / rg;
        if (nr <= 4) launch_step<E, 4, 4>(L, slot, pos, rows, out, rs, packed, cols, st);
        else if (nr <= 8) launch_step<E, 4, 8>(L, slot, pos, rows, out, rs, packed, cols, st);
        else if (nr <= 16) launch_step<E, 4, 16>(L, slot, pos, rows, out, rs, packed, cols, st);
        else launch_step<E, 4, 0>(L, slot, pos, rows, out, rs, packed, cols, st);
    } else {
        launch_step<E, 1, 0>(L, slot, pos, rows, out, rs, packed, cols, st);
    }
}
template <class E>
void launch_prepare(const tah_delta_layer& L, const tah_portions& P, float* q, float* k, float* v, float* lg, float* beta, hipStream_t st) {
    const int nch = 2 * L.kv_heads * L.dim + L.heads * L.vdim;
    const dim3 tail((nch + kDeltaThreads - 1) / kDeltaThreads, P.nseq);
    if (L.taps >= 1 && L.taps <= 4 && in_units(L.dim) && L.vdim % 8 == 0 && unit_rows(L) && aligned_16(q) && aligned_16(k) && aligned_16(v)) {
        const dim3 grid((P.rows + kPrepTokens - 1) / kPrepTokens, (nch / 8 + kDeltaThreads - 1) / kDeltaThreads + 1);
        if (L.taps == 1) hipLaunchKernelGGL((delta_prepare_units_kernel<E, 1>), grid, dim3(kDeltaThreads), 0, st, L, P, q, k, v, lg, beta);
        else if (L.taps == 2) hipLaunchKernelGGL((delta_prepare_units_kernel<E, 2>), grid, dim3(kDeltaThreads), 0, st, L, P, q, k, v, lg, beta);
        else if (L.taps == 3) hipLaunchKernelGGL((delta_prepare_units_kernel<E, 3>), grid, dim3(kDeltaThreads), 0, st, L, P, q, k, v, lg, beta);
        else hipLaunchKernelGGL((delta_prepare_units_kernel<E, 4>), grid, dim3(kDeltaThreads), 0, st, L, P, q, k, v, lg, beta);
        hipLaunchKernelGGL((conv_tail_kernel<E>), tail, dim3(kDeltaThreads), 0, st, L, P);
        return;
    }
    constexpr int per_block = kPrepTokens * (kDeltaThreads / kWave);
    const dim3 grid((P.rows + per_block - 1) / per_block, 2 * L.kv_heads + L.heads + 1);
    const int d = L.dim > L.vdim ? L.dim : L.vdim;
    if (d <= 64) hipLaunchKernelGGL((delta_prepare_kernel<E, 1>), grid, dim3(kDeltaThreads), 0, st, L, P, q, k, v, lg, beta);
    else if (d <= 128) hipLaunchKernelGGL((delta_prepare_kernel<E, 2>), grid, dim3(kDeltaThreads), 0, st, L, P, q, k, v, lg, beta);
    else if (d <= 256) hipLaunchKernelGGL((delta_prepare_kernel<E, 4>), grid, dim3(kDeltaThreads), 0, st, L, P, q, k, v, lg, beta);
    else hipLaunchKernelGGL((delta_prepare_kernel<E, 8>), grid, dim3(kDeltaThreads), 0, st, L, P, q, k, v, lg, beta);
    hipLaunchKernelGGL((conv_tail_kernel<E>), tail, dim3(kDeltaThreads), 0, st, L, P);
}

// Portions long enough, and sizes in whole tiles, for the chunked form.
constexpr int kChunkedFromRows = 48;  // rows per sequence, on average
bool chunked(const tah_delta_layer& L, int rows, int nseq) {
    const bool tiles = L.dim == 16 || L.dim == 32 || L.dim == 64 || L.dim == 128 || L.dim == 256;
    return tiles && L.vdim % 16 == 0 && nseq > 0 && rows / nseq >= kChunkedFromRows;
}
int64_t chunk_slots(int rows, int nseq) { return (int64_t)rows / kChunk + nseq; }

template <int NT>
void launch_chunked(const tah_delta_layer& L, const tah_portions& P, const float* q, const float* k, const float* v, const float* lg, const float* beta,
                    float* o, float* work, hipStream_t st) {
    hipLaunchKernelGGL((delta_chunk_kernel<NT>), dim3((unsigned)chunk_slots(P.rows, P.nseq), L.heads), dim3(kChunkThreads), 0, st, L, P, q, k, v, lg,
                       beta, work);
    hipLaunchKernelGGL((delta_chunk_scan_kernel<NT>), dim3((unsigned)((L.heads * P.nseq + 7) / 8 * 8 * (L.vdim / 16))), dim3(kDeltaThreads), 0, st, L, P, q, k, work, o);
}

template <class E>
void launch_finish(const tah_delta_layer& L, const float* o, int rows, void* out, int64_t out_rs, int out_cols, hipStream_t st) {
    const int64_t items = (int64_t)rows * L.heads;
    if (in_units(L.vdim) && unit_rows(L) && aligned_16(o) && aligned_16(out) && out_rs % 8 == 0) {
        const int64_t units = items * L.vdim / 8;
        hipLaunchKernelGGL((delta_finish_units_kernel<E>), dim3((unsigned)((units + kDeltaThreads - 1) / kDeltaThreads)), dim3(kDeltaThreads), 0, st, L, o,
                           units, static_cast<E*>(out), out_rs, out_cols);
    } else {
        hipLaunchKernelGGL((delta_finish_kernel<E>), dim3((unsigned)((items + kDeltaThreads / kWave - 1) / (kDeltaThreads / kWave))), dim3(kDeltaThreads), 0,
                           st, L, o, items, static_cast<E*>(out), out_rs, out_cols);
    }
}

}  // namespace
}  // namespace tah

extern "C" int tah_delta_step(const tah_delta_layer* L, const int32_t* slot, const int32_t* pos, int32_t rows, void* out, int64_t out_rs,
                              void* out_packed, int32_t out_cols, tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (rows < 0 || rows > 65535 || out_cols < L->heads * L->vdim || (out && rows > 1 && out_rs < out_cols)) return TAH_E_SHAPE;
    if (out_packed && (rows > 32 || out_cols % 32 != 0)) return TAH_E_SHAPE;
    if (L->vdim % 4 != 0 && L->vdim > kDeltaThreads) return TAH_E_SHAPE;
    if (rows == 0) return TAH_OK;
    if (!slot || !pos || (!out && !out_packed)) return TAH_E_NULL;
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (L->dtype == TAH_DT_BF16) dispatch_step<__bf16>(*L, slot, pos, rows, out, out_rs, out_packed, out_cols, st);
    else dispatch_step<float>(*L, slot, pos, rows, out, out_rs, out_packed, out_cols, st);
    return launch_status();
}

extern "C" int tah_delta_prepare(const tah_delta_layer* L, const tah_portions* p, float* q, float* k, float* v, float* lg, float* beta,
                                 tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (const int rc = check_portions(p)) return rc;
    if (2 * L->kv_heads + L->heads + 1 > 65535) return TAH_E_SHAPE;
    if (p->rows == 0 || p->nseq == 0) return TAH_OK;
    if (!q || !k || !v || !lg || !beta) return TAH_E_NULL;
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (L->dtype == TAH_DT_BF16) launch_prepare<__bf16>(*L, *p, q, k, v, lg, beta, st);
    else launch_prepare<float>(*L, *p, q, k, v, lg, beta, st);
    return launch_status();
}

extern "C" size_t tah_delta_scan_workspace(const tah_delta_layer* L, int32_t nseq, int32_t rows) {
    using namespace tah;
    if (check_layer(L) != TAH_OK || nseq <= 0 || rows <= 0 || !chunked(*L, rows, nseq)) return 0;
    return (size_t)(chunk_slots(rows, nseq) * L->heads * chunk_floats(L->dim, L->vdim)) * sizeof(float);
}

extern "C" int tah_delta_scan(const tah_delta_layer* L, const tah_portions* p, const float* q, const float* k, const float* v, const float* lg,
                              const float* beta, float* o, void* workspace, size_t workspace_bytes, tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (const int rc = check_portions(p)) return rc;
    if (p->rows == 0 || p->nseq == 0) return TAH_OK;
    if (!q || !k || !v || !lg || !beta || !o) return TAH_E_NULL;
    if (!aligned_16(q) || !aligned_16(k)) return TAH_E_ALIGN;
    const dim3 grid((L->vdim + kScanCols - 1) / kScanCols, L->heads, p->nseq);
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (const size_t need = tah_delta_scan_workspace(L, p->nseq, p->rows)) {
        if (!workspace || workspace_bytes < need) return TAH_E_WORKSPACE;
        if (!aligned_16(workspace)) return TAH_E_ALIGN;
        float* const w = static_cast<float*>(workspace);
        if (L->dim == 16) launch_chunked<1>(*L, *p, q, k, v, lg, beta, o, w, st);
        else if (L->dim == 32) launch_chunked<2>(*L, *p, q, k, v, lg, beta, o, w, st);
        else if (L->dim == 64) launch_chunked<4>(*L, *p, q, k, v, lg, beta, o, w, st);
        else if (L->dim == 128) launch_chunked<8>(*L, *p, q, k, v, lg, beta, o, w, st);
        else launch_chunked<16>(*L, *p, q, k, v, lg, beta, o, w, st);
        return launch_status();
    }
    if (L->dim <= 64) hipLaunchKernelGGL((delta_scan_kernel<1>), grid, dim3(kDeltaThreads), 0, st, *L, *p, q, k, v, lg, beta, o);
    else if (L->dim <= 128) hipLaunchKernelGGL((delta_scan_kernel<2>), grid, dim3(kDeltaThreads), 0, st, *L, *p, q, k, v, lg, beta, o);
    else hipLaunchKernelGGL((delta_scan_kernel<4>), grid, dim3(kDeltaThreads), 0, st, *L, *p, q, k, v, lg, beta, o);
    return launch_status();
}

extern "C" int tah_delta_finish(const tah_delta_layer* L, const float* o, int32_t rows, void* out, int64_t out_rs, int32_t out_cols,
                                tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (rows < 0 || out_cols < L->heads * L->vdim || (rows > 1 && out_rs < out_cols)) return TAH_E_SHAPE;
    if (rows == 0) return TAH_OK;
    if (!o || !out) return TAH_E_NULL;
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (L->dtype == TAH_DT_BF16) launch_finish<__bf16>(*L, o, rows, out, out_rs, out_cols, st);
    else launch_finish<float>(*L, o, rows, out, out_rs, out_cols, st);
    return launch_status();
}
