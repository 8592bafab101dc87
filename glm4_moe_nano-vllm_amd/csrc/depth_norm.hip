// depth_norm.hip — what happens between two sublayers of a decoder whose sublayers read the 32-bit residual as it is, are closed by an
// RMS norm in groups, and whose layers hand on a learned average over all depths:
//
//     x_out  = x_in + norm(y) * g_post               norm: every one of `groups` equal parts divided by its own root mean square
//     x_next = sum_j coef[j] depth_j + coef[n] x_out  (optional; depth_j: n earlier rows of the same token, one plane each)
//     h      = x_next + conv(x_next)                 (optional; depthwise, causal, TAPS taps)      or
//     h      = norm(x_next) * g_pre                  (optional)
//
// in one launch (many rows: two).  y is the finished sublayer's output, or — pair_pos — the rows of a token's k experts, summed with their fp32 weights.
// gfx950 only.  Roofline: HBM — every row is read and written once.
//
// A part of the vector belongs to lanes of one wave (up to 512 columns) or to whole waves, eight columns per lane: with parts of at most
// 512 columns no sum leaves its wave, and the kernel has no barrier.  A workgroup takes one row.
// The convolution's inputs of the TAPS-1 tokens in front of it are recomputed (rows of the same step) or come from the sequence's
// state rows, which are double-buffered: a step reads row set state_in and writes row set state_out.  Everything is fp32 up to the store
// of h, the same arithmetic for a token of this step as for one whose row was kept.
//
// Steps of many rows take two launches, norm and average (every row for itself) and depth_conv: re-reading x_next costs four bytes a
// column; with runs of sixteen rows, recomputing the TAPS-1 in front cost a fifth of rows that are k experts and several depths
// wide.
#include "common.h"

namespace {

struct DepthArgs {
    const float* x_in;         // [T, ld], row r or row_index[r]
    const int32_t* row_index;  // optional gather of x_in / y / depth rows (no convolution then)
    int64_t ld;                // pitch of x_in, x_out, x_next and the depth rows
    const void* y;             // [T, ldy], or with pair_pos [n_rows, ldy], or nullptr
    int64_t ldy;
    const int32_t* pair_pos;   // [T, k] row of y of the token's j-th expert (outside [0, n_rows): none)
    const float* pair_w;       // [T, k]
    int k;
    int64_t n_rows;
    const float* g_post;       // [wp]
    float* x_out;              // or nullptr
    void* x_cast;              // x_out in the activation dtype, or nullptr
    int64_t ldc;
    const float* depth;        // plane j at depth + j * depth_stride, or nullptr
    int64_t depth_stride;
    int n_depth;
    const float* coef;         // [n_depth + 1]
    float* x_next;             // or nullptr
    const float* g_pre;        // [wp] or nullptr
    const bf16_t* conv_w;      // [TAPS][wp]
    float* state;              // [state rows][TAPS-1][wp]
    const int32_t *pos, *seq_of, *q_start, *state_in, *state_out;
    int64_t n_state;
    void* h;                   // [T, ldh] or nullptr
    int64_t ldh;
    int act_f32;
    int64_t T;
    int width, wp, groups, gs;
    int lpg, gpw, wpg, cpw;    // lanes per part inside a wave, parts per wave; waves per part, columns per wave
    float eps;
};

struct Col8 {
    float v[8];
};
__device__ __forceinline__ Col8 dn_zero() { return {{0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}}; }

// n of the eight columns at p are there; VEC: all of them or none, 16-byte aligned
template <bool VEC>
__device__ __forceinline__ Col8 dn_ldf(const float* p, int n) {
    Col8 o = dn_zero();
    if constexpr (VEC) {
        if (n) {
            const f32x4_t a = *reinterpret_cast<const f32x4_t*>(p), b = *reinterpret_cast<const f32x4_t*>(p + 4);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                o.v[i] = a[i];
                o.v[4 + i] = b[i];
            }
        }
    } else {
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (i < n) o.v[i] = p[i];
    }
    return o;
}
template <bool VEC>
__device__ __forceinline__ void dn_stf(float* p, const Col8& o, int n) {
    if constexpr (VEC) {
        if (n) {
            *reinterpret_cast<f32x4_t*>(p) = f32x4_t{o.v[0], o.v[1], o.v[2], o.v[3]};
            *reinterpret_cast<f32x4_t*>(p + 4) = f32x4_t{o.v[4], o.v[5], o.v[6], o.v[7]};
        }
    } else {
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (i < n) p[i] = o.v[i];
    }
}
template <bool VEC>
__device__ __forceinline__ Col8 dn_ldh(const bf16_t* p, int n) {
    Col8 o = dn_zero();
    if constexpr (VEC) {
        if (n) {
            const u32x4_t u = *reinterpret_cast<const u32x4_t*>(p);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                o.v[2 * i] = bflo(u[i]);
                o.v[2 * i + 1] = bfhi(u[i]);
            }
        }
    } else {
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (i < n) o.v[i] = bf2f(p[i]);
    }
    return o;
}
template <bool VEC>
__device__ __forceinline__ Col8 dn_ld(const void* p, int64_t off, int f32, int n) {
    return f32 ? dn_ldf<VEC>(reinterpret_cast<const float*>(p) + off, n) : dn_ldh<VEC>(reinterpret_cast<const bf16_t*>(p) + off, n);
}
template <bool VEC>
__device__ __forceinline__ void dn_st(void* p, int64_t off, int f32, const Col8& o, int n) {
    if (f32) {
        dn_stf<VEC>(reinterpret_cast<float*>(p) + off, o, n);
        return;
    }
    bf16_t* q = reinterpret_cast<bf16_t*>(p) + off;
    if constexpr (VEC) {
        if (n) *reinterpret_cast<u32x4_t*>(q) = u32x4_t{pack2bf(o.v[0], o.v[1]), pack2bf(o.v[2], o.v[3]), pack2bf(o.v[4], o.v[5]), pack2bf(o.v[6], o.v[7])};
    } else {
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (i < n) q[i] = f2bf(o.v[i]);
    }
}
__device__ __forceinline__ float dn_sumsq(const Col8& a) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) s += a.v[i] * a.v[i];
    return s;
}

// this lane's columns: nc of eight from column c
__device__ __forceinline__ void dn_columns(const DepthArgs& a, int lane, int wid, int& c, int& nc) {
    int gi, o;
    if (a.wpg == 1) {
        gi = wid * a.gpw + lane / a.lpg;
        o = (lane % a.lpg) * 8;
        if (lane / a.lpg >= a.gpw) gi = a.groups;
    } else {
        gi = wid / a.wpg;
        o = (wid % a.wpg) * a.cpw + lane * 8;
        if (lane * 8 >= a.cpw) o = a.gs;
    }
    nc = gi < a.groups ? min(8, max(0, a.gs - o)) : 0;
    c = nc ? gi * a.gs + o : 0;
}
// 1 / root mean square of this lane's part
__device__ __forceinline__ float dn_part_rms(const DepthArgs& a, const Col8& v, int lane, int wid, float (*s_red)[16], int& par) {
    float q = dn_sumsq(v);
    for (int s = 1; s < a.lpg; s <<= 1) q += __shfl_xor(q, s, 64);
    if (a.wpg > 1) {
        if (lane == 0) s_red[par][wid] = q;
        __syncthreads();
        q = 0.f;
        const int w0 = wid / a.wpg * a.wpg;
        for (int i = 0; i < a.wpg; ++i) q += s_red[par][w0 + i];
        par ^= 1;
    }
    return 1.0f / sqrtf(q / (float)a.gs + a.eps);
}
// x_out and x_next of one row (the row of x_in, y and the depths), the loads together
template <bool VEC>
__device__ __forceinline__ void dn_row(const DepthArgs& a, int64_t row, int c, int nc, int lane, int wid, float (*s_red)[16], int& par, Col8& x, Col8& xn) {
    x = dn_ldf<VEC>(a.x_in + row * a.ld + c, nc);
    const float* d = a.depth ? a.depth + row * a.ld + c : nullptr;
    Col8 e0[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) e0[u] = a.depth && u < a.n_depth ? dn_ldf<VEC>(d + u * a.depth_stride, nc) : dn_zero();
    if (a.y) {
        Col8 y = dn_zero();
        if (!a.pair_pos) {
            y = dn_ld<VEC>(a.y, row * a.ldy + c, a.act_f32, nc);
        } else if (VEC && !a.act_f32) {
            for (int j0 = 0; j0 < a.k; j0 += 8) {  // eight experts' rows in flight
                u32x4_t e[8];
                float we[8];
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const int p = j0 + j < a.k ? a.pair_pos[row * a.k + j0 + j] : -1;
                    const bool ok = p >= 0 && p < a.n_rows;
                    we[j] = ok ? a.pair_w[row * a.k + j0 + j] : 0.f;
                    e[j] = u32x4_t{0, 0, 0, 0};
                    if (ok && nc) e[j] = *reinterpret_cast<const u32x4_t*>(reinterpret_cast<const bf16_t*>(a.y) + (int64_t)p * a.ldy + c);
                }
#pragma unroll
                for (int j = 0; j < 8; ++j)
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        y.v[2 * i] = fmaf(we[j], bflo(e[j][i]), y.v[2 * i]);
                        y.v[2 * i + 1] = fmaf(we[j], bfhi(e[j][i]), y.v[2 * i + 1]);
                    }
            }
        } else {
            for (int j = 0; j < a.k; ++j) {
                const int p = a.pair_pos[row * a.k + j];
                if (p < 0 || p >= a.n_rows) continue;
                const Col8 e = dn_ld<VEC>(a.y, (int64_t)p * a.ldy + c, a.act_f32, nc);
#pragma unroll
                for (int i = 0; i < 8; ++i) y.v[i] = fmaf(a.pair_w[row * a.k + j], e.v[i], y.v[i]);
            }
        }
        const Col8 gq = dn_ldf<VEC>(a.g_post + c, nc);
        const float ry = dn_part_rms(a, y, lane, wid, s_red, par);
#pragma unroll
        for (int i = 0; i < 8; ++i) x.v[i] = x.v[i] + y.v[i] * ry * gq.v[i];
    }
    xn = x;
    if (!a.depth) return;
    Col8 avg = dn_zero();
#pragma unroll
    for (int u = 0; u < 4; ++u)
        if (u < a.n_depth) {
#pragma unroll
            for (int i = 0; i < 8; ++i) avg.v[i] = fmaf(a.coef[u], e0[u].v[i], avg.v[i]);
        }
    for (int j = 4; j < a.n_depth; j += 4) {
        Col8 e[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) e[u] = j + u < a.n_depth ? dn_ldf<VEC>(d + (j + u) * a.depth_stride, nc) : dn_zero();
#pragma unroll
        for (int u = 0; u < 4; ++u)
            if (j + u < a.n_depth) {
#pragma unroll
                for (int i = 0; i < 8; ++i) avg.v[i] = fmaf(a.coef[j + u], e[u].v[i], avg.v[i]);
            }
    }
    const float cx = a.coef[a.n_depth];
#pragma unroll
    for (int i = 0; i < 8; ++i) xn.v[i] = fmaf(cx, x.v[i], avg.v[i]);
}

// One row per workgroup.  TAPS > 1: with the convolution, for which the TAPS-1 rows in front are computed as well, as far as they are of
// this step.
template <int TAPS, bool VEC>
__global__ __launch_bounds__(1024) void depth_norm_kernel(const DepthArgs a) {
    constexpr int HALO = TAPS - 1;
    __shared__ float s_red[2][16];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    int c, nc, par = 0;
    dn_columns(a, lane, wid, c, nc);
    const int64_t r = blockIdx.x;
    Col8 x, xn, hist[TAPS];
    int s = 0, qs = 0, qe = 0;
    int64_t sin = 0, lo = r;
    if constexpr (TAPS > 1) {
        s = a.seq_of[r];
        qs = a.q_start[s];
        qe = a.q_start[s + 1];
        sin = min(max((int64_t)a.state_in[s], (int64_t)0), a.n_state - 1);
        lo = max(r - HALO, (int64_t)qs);
        const int p = a.pos[r];
#pragma unroll
        for (int k = 1; k < TAPS; ++k)  // what lies in front of the portion
            hist[k - 1] = dn_ldf<VEC>(a.state + (sin * HALO + (r - k < qs ? HALO - (qs - (r - k)) : 0)) * a.wp + c, p - k >= 0 && r - k < qs ? nc : 0);
        for (int64_t q = lo; q < r; ++q) {
            dn_row<VEC>(a, q, c, nc, lane, wid, s_red, par, x, xn);
#pragma unroll
            for (int k = 1; k < TAPS; ++k)
                if (r - q == k) hist[k - 1] = xn;
        }
    }
    dn_row<VEC>(a, a.row_index ? (int64_t)a.row_index[r] : r, c, nc, lane, wid, s_red, par, x, xn);
    if (a.x_out) dn_stf<VEC>(a.x_out + r * a.ld + c, x, nc);
    if (a.x_cast) dn_st<VEC>(a.x_cast, r * a.ldc + c, a.act_f32, x, nc);
    if (a.depth && a.x_next) dn_stf<VEC>(a.x_next + r * a.ld + c, xn, nc);
    if (tid < a.wp - a.width) {  // padding columns are zeros
        const int pc = a.width + tid;
        if (a.x_cast) {
            if (a.act_f32) reinterpret_cast<float*>(a.x_cast)[r * a.ldc + pc] = 0.f;
            else reinterpret_cast<bf16_t*>(a.x_cast)[r * a.ldc + pc] = 0;
        }
        if (a.h) {
            if (a.act_f32) reinterpret_cast<float*>(a.h)[r * a.ldh + pc] = 0.f;
            else reinterpret_cast<bf16_t*>(a.h)[r * a.ldh + pc] = 0;
        }
    }
    if (!a.h) return;
    Col8 h = xn;
    if (a.g_pre) {
        const Col8 gp = dn_ldf<VEC>(a.g_pre + c, nc);
        const float rx = dn_part_rms(a, xn, lane, wid, s_red, par);
#pragma unroll
        for (int i = 0; i < 8; ++i) h.v[i] = xn.v[i] * rx * gp.v[i];
    }
    if constexpr (TAPS > 1) {
        Col8 acc = dn_zero();
#pragma unroll
        for (int k = HALO; k >= 0; --k) {
            const Col8 w = dn_ldh<VEC>(a.conv_w + (int64_t)(TAPS - 1 - k) * a.wp + c, nc);
#pragma unroll
            for (int i = 0; i < 8; ++i) acc.v[i] = acc.v[i] + w.v[i] * (k ? hist[k ? k - 1 : 0].v[i] : xn.v[i]);
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) h.v[i] = xn.v[i] + acc.v[i];
        const int64_t so = a.state_out[s];
        const int e = qe - 1 - (int)r;  // tokens of the portion behind this one
        if (e < HALO && so >= 0 && so < a.n_state && a.pos[r] >= 0) {
            dn_stf<VEC>(a.state + (so * HALO + (HALO - 1 - e)) * a.wp + c, xn, nc);
            if (e == 0)  // a portion shorter than the history: the older inputs move up
                for (int i = 0; i < HALO - (qe - qs); ++i)
                    dn_stf<VEC>(a.state + (so * HALO + i) * a.wp + c, dn_ldf<VEC>(a.state + (sin * HALO + i + (qe - qs)) * a.wp + c, nc), nc);
        }
    }
    dn_st<VEC>(a.h, r * a.ldh + c, a.act_f32, h, nc);
}

// h = x + conv(x) and the state, eight columns per thread down a run of rows, the next row's load in flight
template <int TAPS>
__global__ __launch_bounds__(256) void depth_conv_kernel(const DepthArgs a, const float* __restrict__ xs, int tr) {
    constexpr int HALO = TAPS - 1;
    const int c = (blockIdx.y * 256 + threadIdx.x) * 8;
    if (c >= a.wp) return;
    const int nc = min(8, a.width - c);   // (the padding columns of x are not written by anyone)
    const int64_t r0 = (int64_t)blockIdx.x * tr, r1 = min(r0 + tr, a.T);
    auto load = [&](const float* p) {
        Col8 v = dn_ldf<true>(p, 8);
#pragma unroll
        for (int i = 0; i < 8; ++i) v.v[i] = i < nc ? v.v[i] : 0.f;
        return v;
    };
    Col8 w[TAPS], hist[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
        w[j] = dn_ldh<true>(a.conv_w + (int64_t)j * a.wp + c, 8);
        hist[j] = dn_zero();
    }
    int s = a.seq_of[r0], qs = a.q_start[s], qe = a.q_start[s + 1];
    int64_t sin = min(max((int64_t)a.state_in[s], (int64_t)0), a.n_state - 1);
    auto history = [&](int64_t r) {   // inputs of the tokens in front of row r
        const int p = a.pos[r];
#pragma unroll
        for (int k = 1; k < TAPS; ++k) {
            hist[k - 1] = dn_zero();
            if (p - k < 0) continue;
            if (r - k >= qs) hist[k - 1] = load(xs + (r - k) * a.ld + c);
            else hist[k - 1] = load(a.state + (sin * HALO + (HALO - (qs - (r - k)))) * a.wp + c);
        }
    };
    history(r0);
    Col8 x = load(xs + r0 * a.ld + c), xn = dn_zero();
    for (int64_t r = r0; r < r1; ++r) {
        if (r + 1 < r1) xn = load(xs + (r + 1) * a.ld + c);
        if (r == qe) {  // the next sequence's portion begins
            s = a.seq_of[r];
            qs = a.q_start[s];
            qe = a.q_start[s + 1];
            sin = min(max((int64_t)a.state_in[s], (int64_t)0), a.n_state - 1);
            history(r);
        }
        Col8 acc = dn_zero(), h;
#pragma unroll
        for (int k = HALO; k >= 1; --k)
#pragma unroll
            for (int i = 0; i < 8; ++i) acc.v[i] = acc.v[i] + w[TAPS - 1 - k].v[i] * hist[k - 1].v[i];
#pragma unroll
        for (int i = 0; i < 8; ++i) h.v[i] = x.v[i] + (acc.v[i] + w[TAPS - 1].v[i] * x.v[i]);
        dn_st<true>(a.h, r * a.ldh + c, a.act_f32, h, 8);
        const int64_t so = a.state_out[s];
        const int e = qe - 1 - (int)r;  // tokens of the portion behind this one
        if (e < HALO && so >= 0 && so < a.n_state && a.pos[r] >= 0) {
            dn_stf<true>(a.state + (so * HALO + (HALO - 1 - e)) * a.wp + c, x, 8);
            if (e == 0)  // a portion shorter than the history: the older inputs move up
                for (int i = 0; i < HALO - (qe - qs); ++i)
                    dn_stf<true>(a.state + (so * HALO + i) * a.wp + c, dn_ldf<true>(a.state + (sin * HALO + i + (qe - qs)) * a.wp + c, 8), 8);
        }
#pragma unroll
        for (int k = HALO; k >= 2; --k) hist[k - 1] = hist[k - 2];
        hist[0] = x;
        x = xn;
    }
}

constexpr int64_t DN_SPLIT_ROWS = 512;   // rows from which norm and convolution are launches of their own

template <int TAPS>
int launch_depth_conv(const DepthArgs& a, const float* xs, hipStream_t st) {
    const int tr = 32;
    hipLaunchKernelGGL(depth_conv_kernel<TAPS>, dim3((unsigned)((a.T + tr - 1) / tr), (unsigned)((a.wp + 2047) / 2048)), dim3(256), 0, st, a, xs, tr);
    GLM_CHECK_LAUNCH("glm_depth_norm(convolution)");
    return GLM_OK;
}

template <int TAPS>
int launch_depth_norm(const DepthArgs& a, int nt, bool vec, hipStream_t st) {
    if constexpr (TAPS > 1) {
        const float* xs = a.depth ? a.x_next : a.y ? a.x_out : a.x_in;
        if (a.T > DN_SPLIT_ROWS && xs) {
            if (a.y || a.depth || a.x_cast || a.x_out) {
                DepthArgs b = a;
                b.h = nullptr;
                const int rc = launch_depth_norm<1>(b, nt, vec, st);
                if (rc != GLM_OK) return rc;
            }
            return launch_depth_conv<TAPS>(a, xs, st);
        }
    }
    if (vec) hipLaunchKernelGGL((depth_norm_kernel<TAPS, true>), dim3((unsigned)a.T), dim3(nt), 0, st, a);
    else hipLaunchKernelGGL((depth_norm_kernel<TAPS, false>), dim3((unsigned)a.T), dim3(nt), 0, st, a);
    GLM_CHECK_LAUNCH("glm_depth_norm");
    return GLM_OK;
}

}  // namespace

extern "C" int glm_depth_norm_taps(int taps) {
    for (int t : {1, 2, 3, 4, 6, 8, 16, 32})
        if (taps >= 1 && taps <= t) return t;
    return -1;
}

extern "C" int glm_depth_norm(const float* x_in, const int32_t* row_index, int64_t ld, const void* y, int64_t ldy, const int32_t* pair_pos, const float* pair_w, int k, int64_t n_rows,
                              const float* g_post, float* x_out, void* x_cast, int64_t ldc, const float* depth, int64_t depth_stride, int n_depth, const float* coef, float* x_next,
                              const float* g_pre, const void* conv_w, int taps, float* state, int64_t n_state, const int32_t* pos, const int32_t* seq_of, const int32_t* q_start,
                              const int32_t* state_in, const int32_t* state_out, void* h, int64_t ldh, int act_f32, int64_t T, int width, int wp, int groups, float eps,
                              glm_stream_t stream) {
    GLM_CHECK_ARG(x_in && T >= 0 && width > 0 && wp >= width && wp % 8 == 0 && wp - width < 8 && ld >= wp && ld % 4 == 0 && groups > 0 && width % groups == 0, GLM_ERR_INVALID,
                  "glm_depth_norm: bad shape T=%ld width=%d wp=%d groups=%d ld=%ld", (long)T, width, wp, groups, (long)ld);
    GLM_CHECK_ARG(!y || (g_post && ldy >= wp && ldy % 8 == 0), GLM_ERR_INVALID, "glm_depth_norm: bad sublayer output (ldy=%ld)", (long)ldy);
    GLM_CHECK_ARG(!pair_pos || (y && pair_w && k > 0 && n_rows > 0), GLM_ERR_INVALID, "glm_depth_norm: bad expert rows (k=%d rows=%ld)", k, (long)n_rows);
    GLM_CHECK_ARG((!h || (ldh >= wp && ldh % 8 == 0)) && (!x_cast || (ldc >= wp && ldc % 8 == 0)), GLM_ERR_INVALID, "glm_depth_norm: bad output (ldh=%ld ldc=%ld)", (long)ldh, (long)ldc);
    GLM_CHECK_ARG(!depth || (coef && n_depth >= 0 && depth_stride >= 0 && depth_stride % 4 == 0), GLM_ERR_INVALID, "glm_depth_norm: bad depth rows (n=%d)", n_depth);
    GLM_CHECK_ARG(taps == 1 || (conv_w && h && !g_pre && state && n_state > 0 && pos && seq_of && q_start && state_in && state_out && !row_index && x_out != x_in && x_next != x_in),
                  GLM_ERR_INVALID, "glm_depth_norm: the convolution needs weights, state, positions and outputs apart from x_in");
    GLM_CHECK_ARG(taps >= 1 && glm_depth_norm_taps(taps) == taps, GLM_ERR_UNSUPPORTED, "glm_depth_norm: %d taps (see glm_depth_norm_taps)", taps);
    GLM_CHECK_ARG(T < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_depth_norm: too many rows");
    DepthArgs a = {x_in, row_index, ld, y, ldy, pair_pos, pair_w, k, n_rows, g_post, x_out, x_cast, ldc, depth, depth_stride, n_depth, coef, x_next, g_pre, (const bf16_t*)conv_w, state,
                   pos, seq_of, q_start, state_in, state_out, n_state, h, ldh, act_f32, T, width, wp, groups, width / groups, 64, 1, 1, 0, eps};
    int waves;
    if (a.gs > 512) {  // whole waves per part
        a.wpg = (a.gs + 511) / 512;
        a.cpw = ((a.gs + a.wpg - 1) / a.wpg + 7) / 8 * 8;
        waves = groups * a.wpg;
    } else {           // a power of two of lanes per part
        a.lpg = 1;
        while (a.lpg * 8 < a.gs) a.lpg *= 2;
        a.gpw = 64 / a.lpg;
        waves = (groups + a.gpw - 1) / a.gpw;
    }
    GLM_CHECK_ARG(waves <= 16, GLM_ERR_UNSUPPORTED, "glm_depth_norm: %d parts of %d columns need %d waves (16 at most)", groups, a.gs, waves);
    if (T == 0) return GLM_OK;
    const bool vec = a.gs % 8 == 0 && glm_aligned16(x_in) && glm_aligned16(y) && glm_aligned16(h) && glm_aligned16(x_cast) && glm_aligned16(depth);
    const int nt = waves * 64;
    hipStream_t st = glm_s(stream);
    switch (taps) {
        case 1: return launch_depth_norm<1>(a, nt, vec, st);
        case 2: return launch_depth_norm<2>(a, nt, vec, st);
        case 3: return launch_depth_norm<3>(a, nt, vec, st);
        case 4: return launch_depth_norm<4>(a, nt, vec, st);
        case 6: return launch_depth_norm<6>(a, nt, vec, st);
        case 8: return launch_depth_norm<8>(a, nt, vec, st);
        case 16: return launch_depth_norm<16>(a, nt, vec, st);
        default: return launch_depth_norm<32>(a, nt, vec, st);
    }
}
