// stream_norm.hip — what happens between two sublayers of a decoder whose residual is several parallel streams ("hyper-
// connections", fp32 throughout).  With the finished sublayer's output y and its matrices
//
//     x'_t = sum_s mix[s, t] x_s + out[t] * (scale . y)      all streams at once from the old ones     (optional: y)
//     u    = sum_s in[s] x'_s                                 what the next sublayer's norm reads
//     h    = u / rms(u) * gain                                RMS norm with ONE gain                     (optional: h)
//     h    = h + (h_prev - h) . shift                         token shift; h_prev: the previous token's h, zero for the first
//
// in ONE launch.  gfx950 only.  Roofline: HBM — the streams are read once and written once, y read once, h written once.
//
// A workgroup takes a run of rows one after the other; a thread owns VC columns of every stream, the next row's loads are in
// flight while a row is worked on, and one barrier per row carries the reduction.  The token shift needs the h of the row in
// front of the run: it is RECOMPUTED from x_in and y (no hand-off between workgroups, so x_out is another buffer than x_in), or
// read from the sequence's state row where the portion begins.  A step reads state row state_in and writes row state_out,
// because the workgroup that writes a portion's last h is not the one that reads the previous portion's.  A token's h is the
// same arithmetic whether it was computed in this step or kept from an earlier one.
#include "common.h"

namespace {

struct StreamNormArgs {
    const float* x_in;        // element (row r, stream s, column c) at r*ldx + s*sx + c; sx = 0: all streams are the same row
    int64_t ldx, sx;
    const int32_t* row_index; // optional gather of x_in / y rows (no token shift, no x_out then)
    float* x_out;             // [T][S][wp] or nullptr
    const void* y;            // [T, ldy] or nullptr
    int64_t ldy;
    int y_f32;
    const float* y_scale;     // [wp]
    const float* mix_out;     // [S*S] mix[from*S + to], then [S] out
    const float* w_in;        // [S]
    float gain;
    const float* shift;       // [wp] or nullptr
    float* state;             // [n_state][wp]
    int64_t n_state;
    const int32_t* pos;       // [T] position of the row in its sequence (< 0: unused row)
    const int32_t* seq_of;    // [T]
    const int32_t* q_start;   // [n_seq+1]
    const int32_t *state_in, *state_out;  // [n_seq] (state_out < 0: keep nothing)
    void* h;                  // [T, ldh] or nullptr
    int64_t ldh;
    int h_f32;
    int64_t T;
    int S, width, wp;         // streams, true width (the mean's divisor), padded width (multiple of 8, zero padding)
    float eps;
};

__device__ __forceinline__ f32x4_t st_load4(const void* base, int64_t off, int f32) {
    if (f32) return *reinterpret_cast<const f32x4_t*>(reinterpret_cast<const float*>(base) + off);
    const u32x2_t u = *reinterpret_cast<const u32x2_t*>(reinterpret_cast<const bf16_t*>(base) + off);
    return f32x4_t{bflo(u[0]), bfhi(u[0]), bflo(u[1]), bfhi(u[1])};
}
__device__ __forceinline__ void st_store4(void* base, int64_t off, int f32, const f32x4_t& v) {
    if (f32) *reinterpret_cast<f32x4_t*>(reinterpret_cast<float*>(base) + off) = v;
    else *reinterpret_cast<u32x2_t*>(reinterpret_cast<bf16_t*>(base) + off) = u32x2_t{pack2bf(v[0], v[1]), pack2bf(v[2], v[3])};
}
__device__ __forceinline__ float st_sumsq(const f32x4_t& v) { return v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3]; }

// S streams, NV vectors of four columns per thread, NT threads: wp <= 4 NV NT
template <int S, int NV, int NT>
__global__ __launch_bounds__(NT) void stream_norm_kernel(const StreamNormArgs a, int tr) {
    constexpr int NW = NT / 64;
    __shared__ float s_red[2][NW];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
    const int64_t r0 = (int64_t)blockIdx.x * tr, r1 = min(r0 + tr, a.T);
    const float inv_w = 1.0f / (float)a.width;
    const bool shifted = a.shift != nullptr;
    int s = 0, qs = 0, qe = 0;
    int64_t lo = r0;
    if (shifted) {
        s = a.seq_of[r0];
        qs = a.q_start[s];
        qe = a.q_start[s + 1];
        if (r0 > qs) lo = r0 - 1;
    }
    // vector j of this thread: columns 4 (tid + j NT) .. + 3
    int col[NV];
    bool on[NV];
    f32x4_t ys[NV], sh[NV], hist[NV];
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        col[j] = 4 * (tid + j * NT);
        on[j] = col[j] < a.wp;
        ys[j] = (on[j] && a.y) ? *reinterpret_cast<const f32x4_t*>(a.y_scale + col[j]) : zero;
        sh[j] = (on[j] && shifted) ? *reinterpret_cast<const f32x4_t*>(a.shift + col[j]) : zero;
        hist[j] = zero;
    }
    float mix[S][S], wo[S], wi[S];
#pragma unroll
    for (int f = 0; f < S; ++f) {
        wi[f] = a.w_in ? a.w_in[f] : 0.f;
        wo[f] = a.y ? a.mix_out[S * S + f] : 0.f;
#pragma unroll
        for (int t = 0; t < S; ++t) mix[f][t] = a.y ? a.mix_out[f * S + t] : 0.f;
    }
    auto load_row = [&](int64_t r, f32x4_t (&x)[S][NV], f32x4_t (&y)[NV]) {
        const int64_t row = a.row_index ? a.row_index[r] : r;
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            if (!on[j]) continue;
#pragma unroll
            for (int t = 0; t < S; ++t) x[t][j] = __builtin_nontemporal_load(reinterpret_cast<const f32x4_t*>(a.x_in + row * a.ldx + t * a.sx + col[j]));
            if (a.y) y[j] = st_load4(a.y, row * a.ldy + col[j], a.y_f32);
        }
    };
    f32x4_t x[S][NV], y[NV], xn[S][NV], yn[NV];
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        y[j] = yn[j] = zero;
#pragma unroll
        for (int t = 0; t < S; ++t) x[t][j] = xn[t][j] = zero;
    }
    load_row(lo, x, y);
    int par = 0;
    for (int64_t r = lo; r < r1; ++r) {
        if (r + 1 < r1) load_row(r + 1, xn, yn);
        float sq = 0.f;
        f32x4_t u[NV];
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            if (a.y) {
                f32x4_t v[S];
#pragma unroll
                for (int t = 0; t < S; ++t) {
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        float acc = wo[t] * (ys[j][i] * y[j][i]);
#pragma unroll
                        for (int f = 0; f < S; ++f) acc = fmaf(mix[f][t], x[f][j][i], acc);
                        v[t][i] = acc;
                    }
                }
#pragma unroll
                for (int t = 0; t < S; ++t) x[t][j] = v[t];
            }
            if (a.x_out && r >= r0 && on[j]) {
#pragma unroll
                for (int t = 0; t < S; ++t) __builtin_nontemporal_store(x[t][j], reinterpret_cast<f32x4_t*>(a.x_out + (r * S + t) * a.wp + col[j]));
            }
            u[j] = zero;
#pragma unroll
            for (int t = 0; t < S; ++t)
#pragma unroll
                for (int i = 0; i < 4; ++i) u[j][i] = fmaf(wi[t], x[t][j][i], u[j][i]);
            sq += st_sumsq(u[j]);
        }
        if (a.h) {
            sq = wave_sum(sq);
            if constexpr (NW > 1) {
                if (lane == 0) s_red[par][wid] = sq;
                __syncthreads();
                sq = 0.f;
#pragma unroll
                for (int w = 0; w < NW; ++w) sq += s_red[par][w];
                par ^= 1;
            }
            const float rms = sqrtf(sq * inv_w + a.eps), f = a.gain / rms;
            int64_t so = -1;
            bool first = false;
            int64_t sin = 0;
            if (shifted) {
                if (r == qe) {  // the next sequence's portion begins
                    s = a.seq_of[r];
                    qs = a.q_start[s];
                    qe = a.q_start[s + 1];
                }
                first = r == qs;
                sin = min(max((int64_t)a.state_in[s], (int64_t)0), a.n_state - 1);
                if (r == qe - 1 && r >= r0 && a.pos[r] >= 0) so = a.state_out[s];
                if (so >= a.n_state) so = -1;
            }
            const bool fresh = first && a.pos[r] <= 0;  // first token of its sequence: whatever the state row holds is not its
#pragma unroll
            for (int j = 0; j < NV; ++j) {
                f32x4_t o;
#pragma unroll
                for (int i = 0; i < 4; ++i) o[i] = u[j][i] * f;
                if (shifted && on[j]) {
                    const f32x4_t hv = o;
                    if (first) hist[j] = fresh ? zero : *reinterpret_cast<const f32x4_t*>(a.state + sin * a.wp + col[j]);
#pragma unroll
                    for (int i = 0; i < 4; ++i) o[i] = fmaf(hist[j][i] - hv[i], sh[j][i], hv[i]);
                    hist[j] = hv;
                    if (so >= 0) *reinterpret_cast<f32x4_t*>(a.state + so * a.wp + col[j]) = hv;
                }
                if (r >= r0 && on[j]) st_store4(a.h, r * a.ldh + col[j], a.h_f32, o);
            }
        }
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            y[j] = yn[j];
#pragma unroll
            for (int t = 0; t < S; ++t) x[t][j] = xn[t][j];
        }
    }
}

// any number of streams and any width: one row per workgroup, rows read again for every use
constexpr int SW_NT = 256;
__global__ __launch_bounds__(SW_NT) void stream_norm_any_kernel(const StreamNormArgs a) {
    __shared__ float s_red[SW_NT / 64];
    const int tid = threadIdx.x, S = a.S;
    const int64_t r = blockIdx.x;
    const float inv_w = 1.0f / (float)a.width;
    auto stream = [&](int64_t row, int t, int c) {  // x'_t at column c
        float v = 0.f;
        if (!a.y) return a.x_in[row * a.ldx + t * a.sx + c];
        const float yv = a.y_f32 ? reinterpret_cast<const float*>(a.y)[row * a.ldy + c] : bf2f(reinterpret_cast<const bf16_t*>(a.y)[row * a.ldy + c]);
        v = a.mix_out[S * S + t] * (a.y_scale[c] * yv);
        for (int f = 0; f < S; ++f) v = fmaf(a.mix_out[f * S + t], a.x_in[row * a.ldx + f * a.sx + c], v);
        return v;
    };
    auto collapsed = [&](int64_t row, int c) {
        float u = 0.f;
        for (int t = 0; t < S; ++t) u = fmaf(a.w_in[t], stream(row, t, c), u);
        return u;
    };
    auto factor = [&](int64_t row) {
        float sq = 0.f;
        for (int c = tid; c < a.wp; c += SW_NT) {
            const float u = collapsed(row, c);
            sq += u * u;
        }
        sq = wave_sum(sq);
        __syncthreads();
        if ((tid & 63) == 0) s_red[tid >> 6] = sq;
        __syncthreads();
        sq = 0.f;
        for (int w = 0; w < SW_NT / 64; ++w) sq += s_red[w];
        return a.gain / sqrtf(sq * inv_w + a.eps);
    };
    const int64_t row = a.row_index ? a.row_index[r] : r;
    if (a.x_out)
        for (int c = tid; c < a.wp; c += SW_NT)
            for (int t = 0; t < S; ++t) a.x_out[(r * S + t) * a.wp + c] = stream(row, t, c);
    if (!a.h) return;
    int s = 0;
    bool from_row = false, from_state = false;
    int64_t so = -1, sin = 0;
    if (a.shift) {
        s = a.seq_of[r];
        from_row = r > a.q_start[s];
        from_state = !from_row && a.pos[r] > 0;
        sin = min(max((int64_t)a.state_in[s], (int64_t)0), a.n_state - 1);
        if (r == a.q_start[s + 1] - 1 && a.pos[r] >= 0) so = a.state_out[s];
    }
    const float f = factor(row), fp = from_row ? factor(row - 1) : 0.f;
    for (int c = tid; c < a.wp; c += SW_NT) {
        const float hv = collapsed(row, c) * f;
        float o = hv;
        if (a.shift) {
            const float prev = from_row ? collapsed(row - 1, c) * fp : from_state ? a.state[sin * a.wp + c] : 0.f;
            o = fmaf(prev - hv, a.shift[c], hv);
            if (so >= 0 && so < a.n_state) a.state[so * a.wp + c] = hv;
        }
        if (a.h_f32) reinterpret_cast<float*>(a.h)[r * a.ldh + c] = o;
        else reinterpret_cast<bf16_t*>(a.h)[r * a.ldh + c] = f2bf(o);
    }
}

template <int S, int NV, int NT>
int launch_stream(const StreamNormArgs& a, hipStream_t st) {
    // decode: one row per workgroup; else runs of rows long enough to spread the halo, short enough to fill the chip
    constexpr int WGS = NT >= 512 ? 512 : 4096 / (NT / 64) > 2048 ? 2048 : 4096 / (NT / 64);   // four waves on every SIMD
    int tr = a.T <= 512 ? 1 : (int)((a.T + WGS - 1) / WGS);
    if (tr > 1) tr = tr < 8 ? 8 : tr > 32 ? 32 : tr;
    hipLaunchKernelGGL((stream_norm_kernel<S, NV, NT>), dim3((unsigned)((a.T + tr - 1) / tr)), dim3(NT), 0, st, a, tr);
    GLM_CHECK_LAUNCH("glm_stream_norm");
    return GLM_OK;
}

template <int S>
int launch_stream_width(const StreamNormArgs& a, hipStream_t st) {
    constexpr int NV = S <= 3 ? 2 : 1;
    constexpr int PER = 4 * NV;
    if (a.wp <= 64 * PER) return launch_stream<S, NV, 64>(a, st);
    if (a.wp <= 128 * PER) return launch_stream<S, NV, 128>(a, st);
    if (a.wp <= 256 * PER) return launch_stream<S, NV, 256>(a, st);
    if (a.wp <= 512 * PER) return launch_stream<S, NV, 512>(a, st);
    if (a.wp <= 1024 * PER) return launch_stream<S, NV, 1024>(a, st);
    hipLaunchKernelGGL(stream_norm_any_kernel, dim3((unsigned)a.T), dim3(SW_NT), 0, st, a);
    GLM_CHECK_LAUNCH("glm_stream_norm");
    return GLM_OK;
}

}  // namespace

extern "C" int glm_stream_norm(const float* x_in, int64_t ldx, int64_t sx, const int32_t* row_index, float* x_out, const void* y, int64_t ldy, int y_f32,
                               const float* y_scale, const float* mix_out, const float* w_in, float gain, const float* shift, float* state, int64_t n_state,
                               const int32_t* pos, const int32_t* seq_of, const int32_t* q_start, const int32_t* state_in, const int32_t* state_out, void* h,
                               int64_t ldh, int h_f32, int64_t T, int S, int width, int wp, float eps, glm_stream_t stream) {
    GLM_CHECK_ARG(x_in && T >= 0 && T < (1ll << 31) && S >= 1 && width > 0 && wp >= width && wp % 8 == 0 && ldx >= wp && ldx % 4 == 0 && sx >= 0 && sx % 4 == 0 &&
                      (sx == 0 || (sx >= wp && ldx >= S * sx)), GLM_ERR_INVALID,
                  "glm_stream_norm: bad shape T=%ld S=%d width=%d wp=%d ldx=%ld sx=%ld", (long)T, S, width, wp, (long)ldx, (long)sx);
    GLM_CHECK_ARG(!y || (y_scale && mix_out && ldy >= wp && ldy % 4 == 0), GLM_ERR_INVALID, "glm_stream_norm: bad sublayer output (ldy=%ld)", (long)ldy);
    GLM_CHECK_ARG((x_out || h) && (!h || (w_in && ldh >= wp && ldh % 4 == 0)), GLM_ERR_INVALID, "glm_stream_norm: bad output (ldh=%ld)", (long)ldh);
    GLM_CHECK_ARG(x_out != x_in && !(row_index && x_out), GLM_ERR_INVALID, "glm_stream_norm: x_out must be apart from x_in, and gathered rows have none");
    GLM_CHECK_ARG(!shift || (h && state && n_state > 0 && pos && seq_of && q_start && state_in && state_out && !row_index), GLM_ERR_INVALID,
                  "glm_stream_norm: the token shift needs h, state and positions");
    if (T == 0) return GLM_OK;
    StreamNormArgs a = {x_in, ldx, sx, row_index, x_out, y, ldy, y_f32, y_scale, mix_out, w_in, gain, shift, state, n_state, pos, seq_of, q_start, state_in, state_out,
                        h, ldh, h_f32, T, S, width, wp, eps};
    hipStream_t st = glm_s(stream);
    switch (S) {
        case 1: return launch_stream_width<1>(a, st);
        case 2: return launch_stream_width<2>(a, st);
        case 3: return launch_stream_width<3>(a, st);
        case 4: return launch_stream_width<4>(a, st);
        case 5: return launch_stream_width<5>(a, st);
        case 6: return launch_stream_width<6>(a, st);
        case 8: return launch_stream_width<8>(a, st);
        default: break;
    }
    hipLaunchKernelGGL(stream_norm_any_kernel, dim3((unsigned)T), dim3(SW_NT), 0, st, a);
    GLM_CHECK_LAUNCH("glm_stream_norm");
    return GLM_OK;
}
