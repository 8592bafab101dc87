// seq_norm.hip — what happens between two sublayers of a decoder with a 32-bit residual stream, norms in front of and behind
// every sublayer and a short causal convolution over time on what a sublayer reads:
//
//     x_out = x_in + rms(y) * g_post          (y: the finished sublayer's output, optional)
//     h     = rms(x_out) * g_pre              (optional)
//     h     = h + conv(h)                     (optional; depthwise, causal, TAPS taps)
//
// in ONE launch.  gfx950 only.  Roofline: HBM — x_in and y are read once, x_out and h written once (seq_norm_stream_kernel; the
// two-pass seq_norm_kernel, which reads a row again, is for very wide rows and very long convolutions).
//
// The convolution needs the h of the TAPS-1 tokens before.  Inside a step's rows they are RECOMPUTED from x_in and y (a halo
// of TAPS-1 rows per workgroup: no hand-off between workgroups, x_out goes to another buffer than x_in); for tokens of
// earlier steps they come from the sequence's state rows.  The state is double-buffered per sequence (a step reads row set
// state_in and writes row set state_out), because the workgroup that writes a portion's last inputs is not the one that reads
// the previous portion's.  Everything is fp32 up to the store of h, and a token's h is the same arithmetic whether it was
// computed in this step or kept from an earlier one: cutting a sequence differently gives the same bits here.
#include "common.h"

namespace {

struct SeqNormArgs {
    const float* x_in;        // [T, ldx], row r or row_index[r]
    const int32_t* row_index; // optional gather of x_in / y rows (no convolution then)
    int64_t ldx;
    float* x_out;             // [T, ldx] or nullptr
    void* x_cast;             // [T, ldc] x_out in the activation dtype, or nullptr
    int64_t ldc;
    const void* y;            // [T, ldy] or nullptr
    int64_t ldy;
    int y_f32, n_slabs;       // fp32 y: sum of n_slabs slabs (K-slice partial sums)
    int64_t slab_stride;
    const float* g_post;      // [wp]
    const float* g_pre;       // [wp] or nullptr
    const bf16_t* conv_w;     // [TAPS][wp] or nullptr (bf16 in either activation dtype: the checkpoint's values)
    float* state;             // [state rows][TAPS-1][wp]
    const int32_t* pos;       // [T] position of the row in its sequence (< 0: unused row)
    const int32_t* seq_of;    // [T]
    const int32_t* q_start;   // [S+1] first row of every sequence's portion
    const int32_t* state_in;  // [S]
    const int32_t* state_out; // [S] (< 0: keep nothing)
    int64_t n_state;          // state rows
    void* h;                  // [T, ldh]
    int64_t ldh;
    int act_f32;              // activation dtype: 0 bf16, 1 fp32
    int64_t T;
    int width, wp;            // true width (the mean's divisor), padded width (multiple of 8, zero padding)
    float eps;
};

constexpr int SN_NT = 256;

__device__ __forceinline__ f32x4_t sn_load_y(const SeqNormArgs& a, int64_t row, int col) {
    if (!a.y_f32) {
        const u32x2_t u = *reinterpret_cast<const u32x2_t*>(reinterpret_cast<const bf16_t*>(a.y) + row * a.ldy + col);
        return f32x4_t{bflo(u[0]), bfhi(u[0]), bflo(u[1]), bfhi(u[1])};
    }
    const float* p = reinterpret_cast<const float*>(a.y) + row * a.ldy + col;
    f32x4_t v = *reinterpret_cast<const f32x4_t*>(p);
    for (int s = 1; s < a.n_slabs; ++s) v += *reinterpret_cast<const f32x4_t*>(p + s * a.slab_stride);
    return v;
}

__device__ __forceinline__ float sn_sumsq(const f32x4_t& v) { return v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3]; }

// x_out of one row at four columns
__device__ __forceinline__ f32x4_t sn_x(const SeqNormArgs& a, int64_t row, int col, float ry) {
    f32x4_t x = *reinterpret_cast<const f32x4_t*>(a.x_in + row * a.ldx + col);
    if (a.y) {
        const f32x4_t y = sn_load_y(a, row, col), g = *reinterpret_cast<const f32x4_t*>(a.g_post + col);
#pragma unroll
        for (int i = 0; i < 4; ++i) x[i] = x[i] + y[i] * ry * g[i];
    }
    return x;
}

__device__ __forceinline__ void sn_store(void* base, int64_t off, int f32, const f32x4_t& v) {
    if (f32) *reinterpret_cast<f32x4_t*>(reinterpret_cast<float*>(base) + off) = v;
    else *reinterpret_cast<u32x2_t*>(reinterpret_cast<bf16_t*>(base) + off) = u32x2_t{pack2bf(v[0], v[1]), pack2bf(v[2], v[3])};
}

// TR rows per workgroup; TAPS = 1: no convolution
template <int TAPS, int TR>
__global__ __launch_bounds__(SN_NT) void seq_norm_kernel(const SeqNormArgs a) {
    constexpr int HALO = TAPS - 1, NR = TR + HALO;
    __shared__ float s_ry[NR], s_rx[NR], s_red[2][SN_NT / 64];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int64_t r0 = (int64_t)blockIdx.x * TR;
    const int64_t r1 = min(r0 + TR, a.T);  // rows [r0, r1) belong to this workgroup
    const float inv_w = 1.0f / (float)a.width;
    int64_t lo = r0;  // first halo row that is needed: rows of the same sequence only
    if constexpr (TAPS > 1) lo = max(r0 - HALO, (int64_t)a.q_start[a.seq_of[r0]]);
    auto src = [&](int64_t r) -> int64_t { return a.row_index ? a.row_index[r] : r; };

    // ---- pass 1: the two reciprocal root mean squares of every row ----
    if constexpr (TR == 1) {  // the whole workgroup on one row at a time
        for (int64_t r = lo; r < r1; ++r) {
            const int64_t row = src(r);
            float ry = 0.f, s = 0.f;
            if (a.y) {
                for (int c = tid * 4; c < a.wp; c += SN_NT * 4) s += sn_sumsq(sn_load_y(a, row, c));
                s = wave_sum(s);
                if (lane == 0) s_red[0][wid] = s;
                __syncthreads();
                s = 0.f;
#pragma unroll
                for (int w = 0; w < SN_NT / 64; ++w) s += s_red[0][w];
                ry = 1.0f / sqrtf(s * inv_w + a.eps);
            }
            if (a.g_pre) {
                s = 0.f;
                for (int c = tid * 4; c < a.wp; c += SN_NT * 4) s += sn_sumsq(sn_x(a, row, c, ry));
                s = wave_sum(s);
                if (lane == 0) s_red[1][wid] = s;
                __syncthreads();
                s = 0.f;
#pragma unroll
                for (int w = 0; w < SN_NT / 64; ++w) s += s_red[1][w];
            }
            if (tid == 0) {
                s_ry[r - r0 + HALO] = ry;
                s_rx[r - r0 + HALO] = 1.0f / sqrtf(s * inv_w + a.eps);
            }
            __syncthreads();
        }
    } else {
        for (int64_t r = lo + wid; r < r1; r += SN_NT / 64) {
            const int64_t row = src(r);
            float ry = 0.f, s = 0.f;
            if (a.y) {
                for (int c = lane * 4; c < a.wp; c += 256) s += sn_sumsq(sn_load_y(a, row, c));
                ry = 1.0f / sqrtf(wave_sum(s) * inv_w + a.eps);
            }
            if (a.g_pre) {
                s = 0.f;
                for (int c = lane * 4; c < a.wp; c += 256) s += sn_sumsq(sn_x(a, row, c, ry));
                s = wave_sum(s);
            }
            if (lane == 0) {
                s_ry[r - r0 + HALO] = ry;
                s_rx[r - r0 + HALO] = 1.0f / sqrtf(s * inv_w + a.eps);
            }
        }
        __syncthreads();
    }

    // ---- pass 2: four columns per thread, down the rows; the last HALO inputs of the convolution ride in registers ----
    for (int c = tid * 4; c < a.wp; c += SN_NT * 4) {
        f32x4_t gp = {0.f, 0.f, 0.f, 0.f};
        if (a.g_pre) gp = *reinterpret_cast<const f32x4_t*>(a.g_pre + c);
        f32x4_t w[TAPS], hist[TAPS];  // hist[k-1]: h of k tokens ago
        if constexpr (TAPS > 1) {
#pragma unroll
            for (int j = 0; j < TAPS; ++j) {
                const u32x2_t u = *reinterpret_cast<const u32x2_t*>(a.conv_w + (int64_t)j * a.wp + c);
                w[j] = f32x4_t{bflo(u[0]), bfhi(u[0]), bflo(u[1]), bfhi(u[1])};
            }
        }
        auto pre = [&](int64_t r, const f32x4_t& x) {
            const float rx = s_rx[r - r0 + HALO];
            f32x4_t h;
#pragma unroll
            for (int i = 0; i < 4; ++i) h[i] = x[i] * rx * gp[i];
            return h;
        };
        int cur = -1;  // sequence whose history `hist` holds
        for (int64_t r = r0; r < r1; ++r) {
            const f32x4_t x = sn_x(a, src(r), c, s_ry[r - r0 + HALO]);
            if (a.x_out) *reinterpret_cast<f32x4_t*>(a.x_out + r * a.ldx + c) = x;
            if (a.x_cast) sn_store(a.x_cast, r * a.ldc + c, a.act_f32, x);
            if (!a.g_pre) continue;
            const f32x4_t h = pre(r, x);
            f32x4_t o = h;
            if constexpr (TAPS > 1) {
                const int s = a.seq_of[r], p = a.pos[r], qs = a.q_start[s];
                if (s != cur) {
                    cur = s;
                    const int64_t sin = min(max((int64_t)a.state_in[s], (int64_t)0), a.n_state - 1);
#pragma unroll
                    for (int k = 1; k < TAPS; ++k) {
                        f32x4_t v = {0.f, 0.f, 0.f, 0.f};
                        if (p - k >= 0) {
                            if (r - k >= qs) v = pre(r - k, sn_x(a, r - k, c, s_ry[r - k - r0 + HALO]));
                            else v = *reinterpret_cast<const f32x4_t*>(a.state + (sin * HALO + (HALO - (qs - (r - k)))) * a.wp + c);
                        }
                        hist[k - 1] = v;
                    }
                }
                f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int k = HALO; k >= 1; --k)
#pragma unroll
                    for (int i = 0; i < 4; ++i) acc[i] = acc[i] + w[TAPS - 1 - k][i] * hist[k - 1][i];
#pragma unroll
                for (int i = 0; i < 4; ++i) o[i] = h[i] + (acc[i] + w[TAPS - 1][i] * h[i]);
#pragma unroll
                for (int k = HALO; k >= 2; --k) hist[k - 1] = hist[k - 2];
                hist[0] = h;
                const int qe = a.q_start[s + 1];
                const int64_t so = a.state_out[s];
                if (so >= 0 && so < a.n_state && p >= 0) {
                    const int e = qe - 1 - (int)r;  // tokens of the portion behind this one
                    if (e < HALO) *reinterpret_cast<f32x4_t*>(a.state + (so * HALO + (HALO - 1 - e)) * a.wp + c) = h;
                    if (e == 0 && qe - qs < HALO) {  // a portion shorter than the history: the older inputs move up
                        const int64_t sin = min(max((int64_t)a.state_in[s], (int64_t)0), a.n_state - 1);
                        for (int i = 0; i < HALO - (qe - qs); ++i)
                            *reinterpret_cast<f32x4_t*>(a.state + (so * HALO + i) * a.wp + c) =
                                *reinterpret_cast<const f32x4_t*>(a.state + (sin * HALO + i + (qe - qs)) * a.wp + c);
                    }
                }
            }
            sn_store(a.h, r * a.ldh + c, a.act_f32, o);
        }
    }
}

// ---- one pass: every thread owns eight columns and keeps its gains, taps and the convolution's history in registers; the rows of
// the workgroup's run go by one after the other, the next row's loads in flight.  The reduction over a row's x_out^2 and the one
// over the next row's y^2 share a barrier. ----
template <int CTRL, int ROWS>
__device__ __forceinline__ float sn_dpp_add(float v) {
    return v + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, ROWS, 0xf, false));
}
__device__ __forceinline__ float sn_wave_sum(float v) {  // the sum over the wave, in lane 63
    v = sn_dpp_add<0x111, 0xf>(v);  // row_shr:1
    v = sn_dpp_add<0x112, 0xf>(v);
    v = sn_dpp_add<0x114, 0xf>(v);
    v = sn_dpp_add<0x118, 0xf>(v);
    v = sn_dpp_add<0x142, 0xa>(v);  // row_bcast:15
    v = sn_dpp_add<0x143, 0xc>(v);  // row_bcast:31
    return v;
}

struct Row8 {
    f32x4_t a, b;
};
__device__ __forceinline__ Row8 sn_ld8f(const float* p) { return {*reinterpret_cast<const f32x4_t*>(p), *reinterpret_cast<const f32x4_t*>(p + 4)}; }
__device__ __forceinline__ void sn_st8f(float* p, const Row8& v) {
    *reinterpret_cast<f32x4_t*>(p) = v.a;
    *reinterpret_cast<f32x4_t*>(p + 4) = v.b;
}
__device__ __forceinline__ void sn_st8(void* base, int64_t off, int f32, const Row8& v) {
    if (f32) sn_st8f(reinterpret_cast<float*>(base) + off, v);
    else
        *reinterpret_cast<u32x4_t*>(reinterpret_cast<bf16_t*>(base) + off) =
            u32x4_t{pack2bf(v.a[0], v.a[1]), pack2bf(v.a[2], v.a[3]), pack2bf(v.b[0], v.b[1]), pack2bf(v.b[2], v.b[3])};
}
__device__ __forceinline__ float sn_sumsq8(const Row8& v) { return sn_sumsq(v.a) + sn_sumsq(v.b); }

template <int TAPS, int NT>
__global__ __launch_bounds__(NT, (TAPS <= 4 && NT <= 512 ? 4 : 1)) void seq_norm_stream_kernel(const SeqNormArgs a, int tr) {
    constexpr int HALO = TAPS - 1, NW = NT / 64;
    __shared__ float s_red[2][2][NW];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int c = tid * 8;
    const bool on = c < a.wp;
    const int64_t r0 = (int64_t)blockIdx.x * tr, r1 = min(r0 + tr, a.T);
    const float inv_w = 1.0f / (float)a.width;
    int s = 0, qs = 0, qe = 0;
    int64_t lo = r0;
    if constexpr (TAPS > 1) {
        s = a.seq_of[r0];
        qs = a.q_start[s];
        qe = a.q_start[s + 1];
        lo = max(r0 - HALO, (int64_t)qs);
    }
    const Row8 zero = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    Row8 gq = zero, gp = zero, hist[TAPS];
    u32x4_t w[TAPS];  // eight taps packed
    if (on) {
        if (a.y) gq = sn_ld8f(a.g_post + c);
        if (a.g_pre) gp = sn_ld8f(a.g_pre + c);
        if constexpr (TAPS > 1) {
#pragma unroll
            for (int j = 0; j < TAPS; ++j) w[j] = *reinterpret_cast<const u32x4_t*>(a.conv_w + (int64_t)j * a.wp + c);
        }
    }
    if (TAPS > 1 && !on) {
#pragma unroll
        for (int j = 0; j < TAPS; ++j) w[j] = u32x4_t{0, 0, 0, 0};
    }
#pragma unroll
    for (int j = 0; j < TAPS; ++j) hist[j] = zero;
    auto tap = [](const u32x4_t& p, int i) { return (i & 1) ? bfhi(p[i >> 1]) : bflo(p[i >> 1]); };
    auto load_row = [&](int64_t r, Row8& x, Row8& y) {
        if (!on) return;
        const int64_t row = a.row_index ? a.row_index[r] : r;
        x = sn_ld8f(a.x_in + row * a.ldx + c);
        if (!a.y) return;
        if (!a.y_f32) {
            const u32x4_t u = *reinterpret_cast<const u32x4_t*>(reinterpret_cast<const bf16_t*>(a.y) + row * a.ldy + c);
            y.a = f32x4_t{bflo(u[0]), bfhi(u[0]), bflo(u[1]), bfhi(u[1])};
            y.b = f32x4_t{bflo(u[2]), bfhi(u[2]), bflo(u[3]), bfhi(u[3])};
        } else {
            y.a = sn_load_y(a, row, c);
            y.b = sn_load_y(a, row, c + 4);
        }
    };
    // sums over the workgroup of two values per thread
    auto reduce2 = [&](float u, float v, int par, float& su, float& sv) {
        u = sn_wave_sum(u);
        v = sn_wave_sum(v);
        if (lane == 63) {
            s_red[par][0][wid] = u;
            s_red[par][1][wid] = v;
        }
        __syncthreads();
        su = sv = 0.f;
#pragma unroll
        for (int i = 0; i < NW; ++i) {
            su += s_red[par][0][i];
            sv += s_red[par][1][i];
        }
    };
    Row8 x = zero, y = zero, xn = zero, yn = zero;
    load_row(lo, x, y);
    float ry = 0.f, su, sv;
    int par = 0;
    if (a.y) {
        reduce2(sn_sumsq8(y), 0.f, par, su, sv);
        ry = 1.0f / sqrtf(su * inv_w + a.eps);
        par ^= 1;
    }
    for (int64_t r = lo; r < r1; ++r) {
        const bool more = r + 1 < r1;
        if constexpr (TAPS > 1) {  // opaque: unpacked outside the loop the taps would take twice the registers
#pragma unroll
            for (int j = 0; j < TAPS; ++j) asm volatile("" : "+v"(w[j]));
        }
        if (more) load_row(r + 1, xn, yn);
        if (a.y) {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                x.a[i] = x.a[i] + y.a[i] * ry * gq.a[i];
                x.b[i] = x.b[i] + y.b[i] * ry * gq.b[i];
            }
        }
        if (r >= r0 && on) {
            if (a.x_out) sn_st8f(a.x_out + r * a.ldx + c, x);
            if (a.x_cast) sn_st8(a.x_cast, r * a.ldc + c, a.act_f32, x);
        }
        reduce2(sn_sumsq8(x), more ? sn_sumsq8(yn) : 0.f, par, su, sv);
        par ^= 1;
        if (a.g_pre) {
            const float rx = 1.0f / sqrtf(su * inv_w + a.eps);
            Row8 h, o;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                h.a[i] = x.a[i] * rx * gp.a[i];
                h.b[i] = x.b[i] * rx * gp.b[i];
            }
            o = h;
            if constexpr (TAPS > 1) {
                if (r == qe) {  // the next sequence's portion begins
                    s = a.seq_of[r];
                    qs = a.q_start[s];
                    qe = a.q_start[s + 1];
                }
                const int64_t sin = min(max((int64_t)a.state_in[s], (int64_t)0), a.n_state - 1);
                if (r == qs) {
                    const int p = a.pos[r];
#pragma unroll
                    for (int k = 1; k < TAPS; ++k) {
                        hist[k - 1] = zero;
                        if (on && p - k >= 0) hist[k - 1] = sn_ld8f(a.state + (sin * HALO + (HALO - k)) * a.wp + c);
                    }
                }
                Row8 acc = zero;
#pragma unroll
                for (int k = HALO; k >= 1; --k)
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        acc.a[i] = acc.a[i] + tap(w[TAPS - 1 - k], i) * hist[k - 1].a[i];
                        acc.b[i] = acc.b[i] + tap(w[TAPS - 1 - k], 4 + i) * hist[k - 1].b[i];
                    }
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    o.a[i] = h.a[i] + (acc.a[i] + tap(w[TAPS - 1], i) * h.a[i]);
                    o.b[i] = h.b[i] + (acc.b[i] + tap(w[TAPS - 1], 4 + i) * h.b[i]);
                }
                const int64_t so = a.state_out[s];
                const int e = qe - 1 - (int)r;  // tokens of the portion behind this one
                if (r >= r0 && e < HALO && on && so >= 0 && so < a.n_state && a.pos[r] >= 0) {
                    sn_st8f(a.state + (so * HALO + (HALO - 1 - e)) * a.wp + c, h);
                    if (e == 0)  // a portion shorter than the history: the older inputs move up
                        for (int i = 0; i < HALO - (qe - qs); ++i)
                            sn_st8f(a.state + (so * HALO + i) * a.wp + c, sn_ld8f(a.state + (sin * HALO + i + (qe - qs)) * a.wp + c));
                }
#pragma unroll
                for (int k = HALO; k >= 2; --k) hist[k - 1] = hist[k - 2];
                hist[0] = h;
            }
            if (r >= r0 && on) sn_st8(a.h, r * a.ldh + c, a.act_f32, o);
        }
        if (a.y) ry = 1.0f / sqrtf(sv * inv_w + a.eps);
        x = xn;
        y = yn;
    }
}

template <int TAPS, int NT>
int launch_seq_norm_stream(const SeqNormArgs& a, hipStream_t st) {
    // decode: one row per workgroup; else runs of rows long enough to spread the halo and the register setup, short enough
    // to fill the chip
    int tr = a.T <= 512 ? 1 : (int)((a.T + 511) / 512);
    if (tr > 1) tr = tr < 8 ? 8 : tr > 32 ? 32 : tr;
    hipLaunchKernelGGL((seq_norm_stream_kernel<TAPS, NT>), dim3((unsigned)((a.T + tr - 1) / tr)), dim3(NT), 0, st, a, tr);
    GLM_CHECK_LAUNCH("glm_seq_norm");
    return GLM_OK;
}

template <int TAPS>
int launch_seq_norm(const SeqNormArgs& a, hipStream_t st) {
    if constexpr (TAPS <= 8) {
        if (a.wp <= 512) return launch_seq_norm_stream<TAPS, 64>(a, st);
        if (a.wp <= 1024) return launch_seq_norm_stream<TAPS, 128>(a, st);
        if (a.wp <= 2048) return launch_seq_norm_stream<TAPS, 256>(a, st);
        if (a.wp <= 4096) return launch_seq_norm_stream<TAPS, 512>(a, st);
        if (TAPS <= 4 && a.wp <= 8192) return launch_seq_norm_stream<TAPS, (TAPS <= 4 ? 1024 : 512)>(a, st);
    }
    // few rows (decode): one row per workgroup; many: 16 rows share a halo
    if (a.T <= 512) hipLaunchKernelGGL((seq_norm_kernel<TAPS, 1>), dim3((unsigned)a.T), dim3(SN_NT), 0, st, a);
    else hipLaunchKernelGGL((seq_norm_kernel<TAPS, 16>), dim3((unsigned)((a.T + 15) / 16)), dim3(SN_NT), 0, st, a);
    GLM_CHECK_LAUNCH("glm_seq_norm");
    return GLM_OK;
}

// one workgroup per token row: fp32 residual row (the table's row times `scale`) and (optionally) the row in the activation dtype.  freq: a sinusoidal position
// vector is added, sin(p f_i) at the even columns 2i and cos(p f_i) at the odd ones; the angle is taken in double and brought into
// one turn before it is rounded, so far positions are as exact as near ones.
__global__ __launch_bounds__(SN_NT) void embed_rows_kernel(const int64_t* ids, const void* table, int64_t ldw, int64_t vocab, const int32_t* pos,
                                                           const double* freq, float* x, int64_t ldx, void* cast, int64_t ldc, int act_f32, int width, int wp, int vec, float scale) {
    const int64_t t = blockIdx.x;
    const int64_t id = ids[t];
    const bool ok = id >= 0 && id < vocab;  // (an id outside the table gives a row of zeros)
    for (int c = threadIdx.x * 4; c < wp; c += SN_NT * 4) {
        f32x4_t v = {0.f, 0.f, 0.f, 0.f};
        if (ok) {
            if (vec) {  // whole rows of the table, padding included
                if (act_f32) v = *reinterpret_cast<const f32x4_t*>(reinterpret_cast<const float*>(table) + id * ldw + c);
                else {
                    const u32x2_t u = *reinterpret_cast<const u32x2_t*>(reinterpret_cast<const bf16_t*>(table) + id * ldw + c);
                    v = f32x4_t{bflo(u[0]), bfhi(u[0]), bflo(u[1]), bfhi(u[1])};
                }
            } else {
                for (int i = 0; i < 4; ++i)
                    if (c + i < width) v[i] = act_f32 ? reinterpret_cast<const float*>(table)[id * ldw + c + i] : bf2f(reinterpret_cast<const bf16_t*>(table)[id * ldw + c + i]);
            }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] *= scale;
        if (freq) {
            const double p = (double)max(pos[t], 0);
#pragma unroll
            for (int i = 0; i < 4; i += 2) {
                if (c + i >= width) break;
                const double turns = p * freq[(c + i) >> 1] * 0.15915494309189533577;
                const float ang = (float)((turns - rint(turns)) * 6.28318530717958647693);
                v[i] += sinf(ang);
                if (c + i + 1 < width) v[i + 1] += cosf(ang);
            }
        }
        *reinterpret_cast<f32x4_t*>(x + t * ldx + c) = v;
        if (cast) sn_store(cast, t * ldc + c, act_f32, v);
    }
}

}  // namespace

extern "C" int glm_seq_norm_taps(int taps) {
    for (int t : {1, 2, 3, 4, 6, 8, 16, 32})
        if (taps >= 1 && taps <= t) return t;
    return -1;
}

extern "C" int glm_seq_norm(const float* x_in, const int32_t* row_index, int64_t ldx, float* x_out, void* x_cast, int64_t ldc,
                            const void* y, int64_t ldy, int y_f32, int n_slabs, int64_t slab_stride, const float* g_post,
                            const float* g_pre, const void* conv_w, int taps, float* state, int64_t n_state, const int32_t* pos,
                            const int32_t* seq_of, const int32_t* q_start, const int32_t* state_in, const int32_t* state_out,
                            void* h, int64_t ldh, int act_f32, int64_t T, int width, int wp, float eps, glm_stream_t stream) {
    GLM_CHECK_ARG(x_in && T >= 0 && width > 0 && wp >= width && wp % 8 == 0 && ldx >= wp && ldx % 4 == 0, GLM_ERR_INVALID,
                  "glm_seq_norm: bad shape T=%ld width=%d wp=%d ldx=%ld", (long)T, width, wp, (long)ldx);
    GLM_CHECK_ARG(!y || (g_post && ldy >= wp && ldy % 4 == 0 && n_slabs >= 1 && (y_f32 || n_slabs == 1)), GLM_ERR_INVALID,
                  "glm_seq_norm: bad sublayer output (ldy=%ld slabs=%d)", (long)ldy, n_slabs);
    GLM_CHECK_ARG((!g_pre) == (!h) && (!h || (ldh >= wp && ldh % 4 == 0)) && (!x_cast || (ldc >= wp && ldc % 4 == 0)), GLM_ERR_INVALID,
                  "glm_seq_norm: bad output (ldh=%ld ldc=%ld)", (long)ldh, (long)ldc);
    GLM_CHECK_ARG(taps == 1 || (conv_w && g_pre && state && n_state > 0 && pos && seq_of && q_start && state_in && state_out && !row_index && x_out != x_in),
                  GLM_ERR_INVALID, "glm_seq_norm: the convolution needs weights, state, positions and x_out apart from x_in");
    GLM_CHECK_ARG(taps >= 1 && glm_seq_norm_taps(taps) == taps, GLM_ERR_UNSUPPORTED, "glm_seq_norm: %d taps (see glm_seq_norm_taps)", taps);
    GLM_CHECK_ARG(T < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_seq_norm: too many rows");
    if (T == 0) return GLM_OK;
    SeqNormArgs a = {x_in, row_index, ldx, x_out, x_cast, ldc, y, ldy, y_f32, n_slabs, slab_stride, g_post, g_pre, (const bf16_t*)conv_w, state,
                     pos, seq_of, q_start, state_in, state_out, n_state, h, ldh, act_f32, T, width, wp, eps};
    hipStream_t st = glm_s(stream);
    switch (taps) {
        case 1: return launch_seq_norm<1>(a, st);
        case 2: return launch_seq_norm<2>(a, st);
        case 3: return launch_seq_norm<3>(a, st);
        case 4: return launch_seq_norm<4>(a, st);
        case 6: return launch_seq_norm<6>(a, st);
        case 8: return launch_seq_norm<8>(a, st);
        case 16: return launch_seq_norm<16>(a, st);
        default: return launch_seq_norm<32>(a, st);
    }
}

extern "C" int glm_embed_rows(const int64_t* ids, const void* table, int64_t ldw, int64_t vocab, const int32_t* pos, const double* freq,
                              float* x, int64_t ldx, void* cast, int64_t ldc, int act_f32, int64_t T, int width, int wp, float scale,
                              glm_stream_t stream) {
    GLM_CHECK_ARG(ids && table && x && T >= 0 && width > 0 && wp >= width && wp % 8 == 0 && ldw >= width && ldx >= wp && ldx % 4 == 0 &&
                      (!cast || (ldc >= wp && ldc % 4 == 0)) && (!freq || pos), GLM_ERR_INVALID, "glm_embed_rows: bad shape T=%ld width=%d wp=%d", (long)T, width, wp);
    if (T == 0) return GLM_OK;
    const int vec = width == wp && ldw % 8 == 0 && glm_aligned16(table);
    hipLaunchKernelGGL(embed_rows_kernel, dim3((unsigned)T), dim3(SN_NT), 0, glm_s(stream), ids, table, ldw, vocab, pos, freq, x, ldx, cast, ldc, act_f32, width, wp, vec, scale);
    GLM_CHECK_LAUNCH("glm_embed_rows");
    return GLM_OK;
}
