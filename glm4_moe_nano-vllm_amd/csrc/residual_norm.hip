// residual_norm.hip — what lies between two layers whose sublayers are not normed behind: the 32-bit residual takes up what it is given
// and the next norm reads it,
//
//     x_out = x_in + y + e        (y: output of the layer, bf16, or the sum of fp32 slabs; e: rows of the embedding table; each optional)
//     h     = x_out / sqrt(mean(x_out^2) + eps) * g        (optional)
//
// in one launch.  gfx950 only.  Roofline: HBM — every operand is touched once, the row stays in registers between its sum and its store
// (rows beyond 8192 columns are read again).  One wave per row up to 1024 columns, four above: no row waits for another.
#include "common.h"

namespace {

struct ResArgs {
    const float* x_in;       // [.., wp] or nullptr
    const int32_t* rows;     // gather of x_in / y / ids rows, or nullptr
    const void* y;           // [.., ldy] or nullptr
    int64_t ldy;
    int y_f32, n_slabs;
    int64_t slab_stride;
    const void* table;       // [vocab, ldt] in the activation dtype, or nullptr
    int64_t ldt, vocab;
    const int64_t* ids;
    float* x_out;            // [T, wp] or nullptr
    const float* g;          // [wp] or nullptr
    void* h;                 // [T, ldh]
    int64_t ldh;
    int act_f32;
    int64_t T;
    int width, wp;
    float eps;
};

struct Cols8 {
    f32x4_t a, b;
};
__device__ __forceinline__ float rn_sumsq(const Cols8& v) {
    return v.a[0] * v.a[0] + v.a[1] * v.a[1] + v.a[2] * v.a[2] + v.a[3] * v.a[3] + v.b[0] * v.b[0] + v.b[1] * v.b[1] + v.b[2] * v.b[2] + v.b[3] * v.b[3];
}
template <bool NT>
__device__ __forceinline__ Cols8 rn_ldf(const float* p) {
    const f32x4_t* q = reinterpret_cast<const f32x4_t*>(p);
    if constexpr (NT) return {__builtin_nontemporal_load(q), __builtin_nontemporal_load(q + 1)};
    else return {q[0], q[1]};
}
// eight columns of a row in bf16 or fp32
template <bool NT>
__device__ __forceinline__ Cols8 rn_ld(const void* base, int64_t off, int f32) {
    if (f32) return rn_ldf<NT>(reinterpret_cast<const float*>(base) + off);
    const u32x4_t* q = reinterpret_cast<const u32x4_t*>(reinterpret_cast<const bf16_t*>(base) + off);
    const u32x4_t u = NT ? __builtin_nontemporal_load(q) : *q;
    return {{bflo(u[0]), bfhi(u[0]), bflo(u[1]), bfhi(u[1])}, {bflo(u[2]), bfhi(u[2]), bflo(u[3]), bfhi(u[3])}};
}
__device__ __forceinline__ void rn_add(Cols8& v, const Cols8& w) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        v.a[i] = v.a[i] + w.a[i];
        v.b[i] = v.b[i] + w.b[i];
    }
}
template <bool NT>
__device__ __forceinline__ Cols8 rn_sum(const ResArgs& a, int64_t src, int64_t id, int c) {
    Cols8 v = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    if (a.x_in) v = rn_ldf<NT>(a.x_in + src * a.wp + c);
    if (a.y) {
        Cols8 y = rn_ld<NT>(a.y, src * a.ldy + c, a.y_f32);
        for (int s = 1; s < a.n_slabs; ++s) rn_add(y, rn_ld<NT>(a.y, s * a.slab_stride + src * a.ldy + c, 1));
        rn_add(v, y);
    }
    if (a.table) rn_add(v, rn_ld<false>(a.table, id * a.ldt + c, a.act_f32));
    return v;
}
template <bool NT>
__device__ __forceinline__ void rn_store_x(const ResArgs& a, int64_t r, int c, const Cols8& v) {
    f32x4_t* q = reinterpret_cast<f32x4_t*>(a.x_out + r * a.wp + c);
    if constexpr (NT) {
        __builtin_nontemporal_store(v.a, q);
        __builtin_nontemporal_store(v.b, q + 1);
    } else {
        q[0] = v.a;
        q[1] = v.b;
    }
}
__device__ __forceinline__ void rn_store_h(const ResArgs& a, int64_t r, int c, const Cols8& v, float rinv) {
    const f32x4_t g0 = *reinterpret_cast<const f32x4_t*>(a.g + c), g1 = *reinterpret_cast<const f32x4_t*>(a.g + c + 4);
    Cols8 o;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        o.a[i] = v.a[i] * rinv * g0[i];
        o.b[i] = v.b[i] * rinv * g1[i];
    }
    if (a.act_f32) {
        f32x4_t* q = reinterpret_cast<f32x4_t*>(reinterpret_cast<float*>(a.h) + r * a.ldh + c);
        q[0] = o.a;
        q[1] = o.b;
    } else {
        *reinterpret_cast<u32x4_t*>(reinterpret_cast<bf16_t*>(a.h) + r * a.ldh + c) =
            u32x4_t{pack2bf(o.a[0], o.a[1]), pack2bf(o.a[2], o.a[3]), pack2bf(o.b[0], o.b[1]), pack2bf(o.b[2], o.b[3])};
    }
}

// TPR threads per row (64 or 256), CH pieces of eight columns per thread (0: as many as it takes, read twice)
template <int TPR, int CH, bool NT>
__global__ __launch_bounds__(256) void residual_norm_kernel(const ResArgs a) {
    __shared__ float red[4];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int64_t r = TPR == 64 ? (int64_t)blockIdx.x * 4 + wid : (int64_t)blockIdx.x;
    if (TPR == 64 && r >= a.T) return;
    const int t = TPR == 64 ? lane : tid;
    const int64_t src = a.rows ? a.rows[r] : r;
    int64_t id = 0;
    if (a.table) id = min(max(a.ids[src], (int64_t)0), a.vocab - 1);
    constexpr int N = CH > 0 ? CH : 1;
    Cols8 v[N];
    float s = 0.f;
    if constexpr (CH > 0) {
#pragma unroll
        for (int k = 0; k < CH; ++k) {
            const int c = (t + k * TPR) * 8;
            if (c < a.wp) v[k] = rn_sum<NT>(a, src, id, c);
        }
#pragma unroll
        for (int k = 0; k < CH; ++k) {
            const int c = (t + k * TPR) * 8;
            if (c >= a.wp) continue;
            if (a.x_out) rn_store_x<NT>(a, r, c, v[k]);
            s += rn_sumsq(v[k]);
        }
    } else {
        for (int c = t * 8; c < a.wp; c += TPR * 8) s += rn_sumsq(rn_sum<false>(a, src, id, c));
    }
    if (CH > 0 && !a.g) return;
    s = wave_sum(s);
    if constexpr (TPR == 256) {
        if (lane == 0) red[wid] = s;
        __syncthreads();
        s = red[0] + red[1] + red[2] + red[3];
    }
    const float rinv = 1.0f / sqrtf(s / (float)a.width + a.eps);
    if constexpr (CH > 0) {
#pragma unroll
        for (int k = 0; k < CH; ++k) {
            const int c = (t + k * TPR) * 8;
            if (c < a.wp) rn_store_h(a, r, c, v[k], rinv);
        }
    } else {
        for (int c = t * 8; c < a.wp; c += TPR * 8) {
            const Cols8 w = rn_sum<false>(a, src, id, c);
            if (a.x_out) rn_store_x<false>(a, r, c, w);
            if (a.g) rn_store_h(a, r, c, w, rinv);
        }
    }
}

template <int TPR, int CH>
void launch(const ResArgs& a, hipStream_t st) {
    const dim3 grid((unsigned)(TPR == 64 ? (a.T + 3) / 4 : a.T));
    // many rows: the residual passes the caches by, h stays for the projection that reads it
    if (CH > 0 && a.T >= 2048) hipLaunchKernelGGL((residual_norm_kernel<TPR, CH, true>), grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((residual_norm_kernel<TPR, CH, false>), grid, dim3(256), 0, st, a);
}

}  // namespace

extern "C" int glm_residual_norm(const float* x_in, const int32_t* rows, const void* y, int64_t ldy, int y_f32, int n_slabs, int64_t slab_stride, const void* table, int64_t ldt,
                                 int64_t vocab, const int64_t* ids, float* x_out, const float* g, void* h, int64_t ldh, int act_f32, int64_t T, int width, int wp, float eps,
                                 glm_stream_t stream) {
    GLM_CHECK_ARG((x_in || table) && (x_out || g) && (!g || h) && (!table || ids), GLM_ERR_INVALID, "glm_residual_norm: null pointer");
    GLM_CHECK_ARG(T >= 0 && width > 0 && wp >= width && wp % 8 == 0 && n_slabs >= 1 && (n_slabs == 1 || (y_f32 && slab_stride >= 0)) && (!y || (ldy >= wp && ldy % 8 == 0)) &&
                      (!table || (ldt >= wp && ldt % 8 == 0 && vocab > 0)) && (!g || (ldh >= wp && ldh % 8 == 0)) && T < (1ll << 31), GLM_ERR_INVALID,
                  "glm_residual_norm: bad shape T=%ld width=%d wp=%d ldy=%ld ldt=%ld ldh=%ld", (long)T, width, wp, (long)ldy, (long)ldt, (long)ldh);
    GLM_CHECK_ARG((!x_in || glm_aligned16(x_in)) && (!y || glm_aligned16(y)) && (!table || glm_aligned16(table)) && (!x_out || glm_aligned16(x_out)) && (!g || (glm_aligned16(g) && glm_aligned16(h))),
                  GLM_ERR_UNSUPPORTED, "glm_residual_norm: operands need 16-byte alignment");
    if (T == 0) return GLM_OK;
    const ResArgs a = {x_in, rows, y, ldy, y_f32, n_slabs, slab_stride, table, ldt, vocab, ids, x_out, g, h, ldh, act_f32, T, width, wp, eps};
    hipStream_t st = glm_s(stream);
    if (wp <= 512) launch<64, 1>(a, st);
    else if (wp <= 1024) launch<64, 2>(a, st);
    else if (wp <= 2048) launch<256, 1>(a, st);
    else if (wp <= 4096) launch<256, 2>(a, st);
    else if (wp <= 8192) launch<256, 4>(a, st);
    else launch<256, 0>(a, st);
    GLM_CHECK_LAUNCH("glm_residual_norm");
    return GLM_OK;
}
