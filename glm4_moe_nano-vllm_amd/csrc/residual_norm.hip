// residual_norm.hip — what lies between two layers whose sublayers are not normed behind: the 32-bit residual takes up what it is given
// and the next norm reads it,
//
//     x_out = x_in + y + e        (y: output of the layer, bf16, or the sum of fp32 slabs; e: rows of the embedding table; each optional)
//     h     = x_out / sqrt(mean(x_out^2) + eps) * g        (optional)
//
// in one launch.  gfx950 only.  Roofline: HBM — every operand is touched once, the row stays in registers between its sum and its store
// (rows beyond 8192 columns are read again).  One wave per row up to 1024 columns, four above, and sixteen where rows are few: no row
// waits for another.
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

__device__ __forceinline__ float rn_sumsq(const f32x4_t& v) { return v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3]; }
template <bool NT>
__device__ __forceinline__ f32x4_t rn_ldf(const float* p) {
    const f32x4_t* q = reinterpret_cast<const f32x4_t*>(p);
    return NT ? __builtin_nontemporal_load(q) : *q;
}
// four columns of a row in bf16 or fp32
__device__ __forceinline__ f32x4_t rn_ld(const void* base, int64_t off, int f32) {
    if (f32) return rn_ldf<false>(reinterpret_cast<const float*>(base) + off);
    const u32x2_t u = *reinterpret_cast<const u32x2_t*>(reinterpret_cast<const bf16_t*>(base) + off);
    return f32x4_t{bflo(u[0]), bfhi(u[0]), bflo(u[1]), bfhi(u[1])};
}
template <bool NT>
__device__ __forceinline__ f32x4_t rn_sum(const ResArgs& a, int64_t src, int64_t id, int c) {
    f32x4_t v = {0.f, 0.f, 0.f, 0.f};
    if (a.x_in) v = rn_ldf<NT>(a.x_in + src * a.wp + c);
    if (a.y) {
        f32x4_t y = rn_ld(a.y, src * a.ldy + c, a.y_f32);
        for (int s = 1; s < a.n_slabs; s += 8) {  // eight slabs in flight
            f32x4_t t[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) t[j] = rn_ldf<false>(reinterpret_cast<const float*>(a.y) + (int64_t)min(s + j, a.n_slabs - 1) * a.slab_stride + src * a.ldy + c);
#pragma unroll
            for (int j = 0; j < 8; ++j)
                if (s + j < a.n_slabs) y += t[j];
        }
        v += y;
    }
    if (a.table) v += rn_ld(a.table, id * a.ldt + c, a.act_f32);
    return v;
}
template <bool NT>
__device__ __forceinline__ void rn_store_x(const ResArgs& a, int64_t r, int c, const f32x4_t& v) {
    f32x4_t* q = reinterpret_cast<f32x4_t*>(a.x_out + r * a.wp + c);
    if constexpr (NT) __builtin_nontemporal_store(v, q);
    else *q = v;
}
__device__ __forceinline__ void rn_store_h(const ResArgs& a, int64_t r, int c, const f32x4_t& v, float rinv) {
    const f32x4_t o = v * rinv * *reinterpret_cast<const f32x4_t*>(a.g + c);
    if (a.act_f32) *reinterpret_cast<f32x4_t*>(reinterpret_cast<float*>(a.h) + r * a.ldh + c) = o;
    else *reinterpret_cast<u32x2_t*>(reinterpret_cast<bf16_t*>(a.h) + r * a.ldh + c) = u32x2_t{pack2bf(o[0], o[1]), pack2bf(o[2], o[3])};
}

// TPR threads per row (64, 256 or 1024), CH pieces of four columns per thread (0: as many as it takes, read twice)
template <int TPR, int CH, bool NT>
__global__ __launch_bounds__(TPR == 1024 ? 1024 : 256) void residual_norm_kernel(const ResArgs a) {
    __shared__ float red[TPR == 64 ? 1 : TPR / 64];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int64_t r = TPR == 64 ? (int64_t)blockIdx.x * 4 + wid : (int64_t)blockIdx.x;
    if (TPR == 64 && r >= a.T) return;
    const int t = TPR == 64 ? lane : tid;
    const int64_t src = a.rows ? a.rows[r] : r;
    int64_t id = 0;
    if (a.table) id = min(max(a.ids[src], (int64_t)0), a.vocab - 1);
    constexpr int N = CH > 0 ? CH : 1;
    f32x4_t v[N];
    float s = 0.f;
    if constexpr (CH > 0) {
#pragma unroll
        for (int k = 0; k < CH; ++k) {
            const int c = (t + k * TPR) * 4;
            if (c < a.wp) v[k] = rn_sum<NT>(a, src, id, c);
        }
#pragma unroll
        for (int k = 0; k < CH; ++k) {
            const int c = (t + k * TPR) * 4;
            if (c >= a.wp) continue;
            if (a.x_out) rn_store_x<NT>(a, r, c, v[k]);
            s += rn_sumsq(v[k]);
        }
    } else {
        for (int c = t * 4; c < a.wp; c += TPR * 4) s += rn_sumsq(rn_sum<false>(a, src, id, c));
    }
    if (CH > 0 && !a.g) return;
    s = wave_sum(s);
    if constexpr (TPR > 64) {
        if (lane == 0) red[wid] = s;
        __syncthreads();
        s = 0.f;
#pragma unroll
        for (int k = 0; k < TPR / 64; ++k) s += red[k];
    }
    const float rinv = 1.0f / sqrtf(s / (float)a.width + a.eps);
    if constexpr (CH > 0) {
#pragma unroll
        for (int k = 0; k < CH; ++k) {
            const int c = (t + k * TPR) * 4;
            if (c < a.wp) rn_store_h(a, r, c, v[k], rinv);
        }
    } else {
        for (int c = t * 4; c < a.wp; c += TPR * 4) {
            const f32x4_t w = rn_sum<false>(a, src, id, c);
            if (a.x_out) rn_store_x<false>(a, r, c, w);
            if (a.g) rn_store_h(a, r, c, w, rinv);
        }
    }
}

template <int TPR, int CH>
void launch(const ResArgs& a, hipStream_t st) {
    const dim3 grid((unsigned)(TPR == 64 ? (a.T + 3) / 4 : a.T)), block(TPR == 1024 ? 1024 : 256);
    // many rows: the residual passes the caches by, h stays for the projection that reads it
    if (CH > 0 && TPR < 1024 && a.T >= 2048) hipLaunchKernelGGL((residual_norm_kernel<TPR, CH, TPR < 1024>), grid, block, 0, st, a);
    else hipLaunchKernelGGL((residual_norm_kernel<TPR, CH, false>), grid, block, 0, st, a);
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
    const bool few = T <= 512;
    if (few && wp > 1024 && wp <= 4096) launch<1024, 1>(a, st);
    else if (few && wp > 4096 && wp <= 8192) launch<1024, 2>(a, st);
    else if (wp <= 512) launch<64, 2>(a, st);
    else if (wp <= 1024) launch<64, 4>(a, st);
    else if (wp <= 2048) launch<256, 2>(a, st);
    else if (wp <= 4096) launch<256, 4>(a, st);
    else if (wp <= 8192) launch<256, 8>(a, st);
    else launch<256, 0>(a, st);
    GLM_CHECK_LAUNCH("glm_residual_norm");
    return GLM_OK;
}
