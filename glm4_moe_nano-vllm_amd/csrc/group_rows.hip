// group_rows.hip — what happens to the projection's rows of an attention with grouped heads (group_attn.hip) before it attends, when
// that is more than storing them: rotation, norms, a temperature.  gfx950 only.
//
//   group_rotate_store   queries are rotated where they are, rotated keys and plain values go to the pages.  Column i of a head's (or,
//                        with two maps per head, of each map's) first `dims` columns turns with column i + dims / 2
//   group_norm_store     queries and keys are normed over the whole projection.  The values are the raw keys, and only they are stored,
//                        with one number per token: 1 / rms of its key row.  Norm gains of the keys are put on the queries (they meet in
//                        the score's products), so a score is (q gq gk / rms_q) . k_raw times that number
//
// Roofline: HBM, every column read and written once; a thread owns both columns of its pairs, so queries can stay in place.  fp32 whatever
// the rows' dtype.
#include "common.h"

namespace {

template <typename T>
__device__ __forceinline__ void gr_ld8(const T* p, float (&v)[8]) {
    if constexpr (sizeof(T) == 4) {
#pragma unroll
        for (int i = 0; i < 8; i += 4) {
            const f32x4_t x = *reinterpret_cast<const f32x4_t*>(p + i);
#pragma unroll
            for (int j = 0; j < 4; ++j) v[i + j] = x[j];
        }
    } else {
        const u32x4_t u = *reinterpret_cast<const u32x4_t*>(p);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            v[2 * i] = bflo(u[i]);
            v[2 * i + 1] = bfhi(u[i]);
        }
    }
}
template <typename T>
__device__ __forceinline__ void gr_st8(T* p, const float (&v)[8]) {
    if constexpr (sizeof(T) == 4) {
#pragma unroll
        for (int i = 0; i < 8; i += 4) *reinterpret_cast<f32x4_t*>(p + i) = f32x4_t{v[i], v[i + 1], v[i + 2], v[i + 3]};
    } else {
        *reinterpret_cast<u32x4_t*>(p) = u32x4_t{pack2bf(v[0], v[1]), pack2bf(v[2], v[3]), pack2bf(v[4], v[5]), pack2bf(v[6], v[7])};
    }
}
template <typename T>
__device__ __forceinline__ float gr_f(T v) {
    if constexpr (sizeof(T) == 4) return v;
    else return bf2f(v);
}
template <typename T>
__device__ __forceinline__ T gr_t(float v) {
    if constexpr (sizeof(T) == 4) return v;
    else return f2bf(v);
}

struct RotArgs {
    void* x;               // row r at r*ld: queries at q_off, keys at k_off, values at v_off
    int64_t ld;
    int q_off, k_off, v_off, nq, G, maps, dm, dv, dims;  // nq: query heads x maps; dm, dv: columns of a map / of a value head
    const float* cs;       // [rows, pairs, 2] of glm_rope_pairs
    int pairs;
    const int32_t* slots;
    void *kc, *vc;         // [n_slots / bs][G][bs][maps * dm], [..][dv]
    int n_slots, bs, log2_bs;
    int T;
    int per;               // items of a row
};

// cache row (in units of a head's columns) of slot, head 0; the heads are bs rows apart
__device__ __forceinline__ int64_t gr_base(int slot, int bs, int log2_bs, int G) {
    const int blk = log2_bs >= 0 ? slot >> log2_bs : slot / bs;
    return (int64_t)blk * G * bs + (slot - blk * bs);
}

// UNIT 8: half of the rotated columns is a multiple of eight, pieces of eight; 1: column by column (the values still by eight).  An item is
// eight pairs (or one), eight columns of a key that do not turn (or one), eight columns of a value; workgroup (row, part of its items)
template <typename T, int UNIT>
__global__ __launch_bounds__(512) void group_rotate_store_kernel(const RotArgs a) {
    const int half = a.dims / 2, pi = half / UNIT, ri = (a.dm - a.dims) / UNIT, nk = a.G * a.maps;
    const int n_q = a.nq * pi, n_k = nk * pi, n_r = nk * ri;
    const int64_t r = blockIdx.x;
    int i = blockIdx.y * blockDim.x + threadIdx.x;
    if (i >= a.per) return;
    const int slot = a.slots[r];
    T* row = reinterpret_cast<T*>(a.x) + r * a.ld;
    // every item: load, then look where it goes (the slot's load is on its way meanwhile)
    if (i < n_q + n_k) {
        const bool key = i >= n_q;
        if (key) i -= n_q;
        const int hm = i / pi, p = (i - hm * pi) * UNIT;
        T* src = row + (key ? a.k_off : a.q_off) + hm * a.dm + p;
        const float* cs = a.cs + (r * a.pairs + p) * 2;
        float x[UNIT], y[UNIT];
        if constexpr (UNIT == 8) {
            float u[8], v[8];
            f32x4_t t[4];
            gr_ld8(src, u);
            gr_ld8(src + half, v);
#pragma unroll
            for (int j = 0; j < 4; ++j) t[j] = *reinterpret_cast<const f32x4_t*>(cs + 4 * j);
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const float c = t[j >> 1][2 * (j & 1)], s = t[j >> 1][2 * (j & 1) + 1];
                x[j] = u[j] * c - v[j] * s;
                y[j] = v[j] * c + u[j] * s;
            }
        } else {
            const float u = gr_f(src[0]), v = gr_f(src[half]), c = cs[0], s = cs[1];
            x[0] = u * c - v * s;
            y[0] = v * c + u * s;
        }
        T* dst = src;
        if (key) {
            if (slot < 0 || slot >= a.n_slots) return;
            const int g = a.maps == 2 ? hm >> 1 : hm;
            dst = reinterpret_cast<T*>(a.kc) + (gr_base(slot, a.bs, a.log2_bs, a.G) + (int64_t)g * a.bs) * (a.maps * a.dm) + (hm - g * a.maps) * a.dm + p;
        }
        if constexpr (UNIT == 8) {
            gr_st8(dst, x);
            gr_st8(dst + half, y);
        } else {
            dst[0] = gr_t<T>(x[0]);
            dst[half] = gr_t<T>(y[0]);
        }
        return;
    }
    i -= n_q + n_k;
    if (i < n_r) {
        const int hm = i / ri, col = a.dims + (i - hm * ri) * UNIT, g = a.maps == 2 ? hm >> 1 : hm;
        const T* src = row + a.k_off + hm * a.dm + col;
        float u[8];
        T one;
        if constexpr (UNIT == 8) gr_ld8(src, u);
        else one = src[0];
        if (slot < 0 || slot >= a.n_slots) return;
        T* dst = reinterpret_cast<T*>(a.kc) + (gr_base(slot, a.bs, a.log2_bs, a.G) + (int64_t)g * a.bs) * (a.maps * a.dm) + (hm - g * a.maps) * a.dm + col;
        if constexpr (UNIT == 8) gr_st8(dst, u);
        else dst[0] = one;
        return;
    }
    i -= n_r;
    const int w = a.dv / 8, g = i / w, col = (i - g * w) * 8;
    float u[8];
    gr_ld8(row + a.v_off + g * a.dv + col, u);
    if (slot < 0 || slot >= a.n_slots) return;
    gr_st8(reinterpret_cast<T*>(a.vc) + (gr_base(slot, a.bs, a.log2_bs, a.G) + (int64_t)g * a.bs) * a.dv + col, u);
}

struct NormArgs {
    void* x;               // row r at r*ld: queries at q_off, keys at k_off
    int64_t ld;
    int q_off, nq, q_n, k_off, nk, k_n;  // padded columns, true columns (the mean's divisor)
    const float* gq;       // [nq] gains of queries and keys, multiplied
    int dm, g0, G;         // columns of a head; key heads g0 .. g0 + G of the row are stored
    float eps, coef;
    int every;             // temperature 1 + coef ln(floor((p + 1) / every) + 1); 0: none
    const int32_t *pos, *slots;
    void* kc;              // [n_slots / bs][G][bs][dm]
    float* kscale;         // [n_slots]
    int n_slots, bs, log2_bs;
};

// one row per workgroup; CH pieces of eight query columns per thread in registers (0: read twice)
template <typename T, int CH>
__global__ __launch_bounds__(256) void group_norm_store_kernel(const NormArgs a) {
    __shared__ float red[2][4];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int64_t r = blockIdx.x;
    const int slot = a.slots[r], pos = a.every > 0 ? max(a.pos[r], 0) : 0;
    const bool kept = slot >= 0 && slot < a.n_slots;
    T* q = reinterpret_cast<T*>(a.x) + r * a.ld + a.q_off;
    const T* k = reinterpret_cast<const T*>(a.x) + r * a.ld + a.k_off;
    constexpr int N = CH > 0 ? CH : 1;
    float v[N][8], sq = 0.f, sk = 0.f;
    if constexpr (CH > 0) {
#pragma unroll
        for (int j = 0; j < CH; ++j) {
            const int c = (tid + j * 256) * 8;
            if (c < a.nq) gr_ld8(q + c, v[j]);
        }
    }
    const int64_t base = kept ? gr_base(slot, a.bs, a.log2_bs, a.G) : 0;
    for (int c = tid * 8; c < a.nk; c += 2048) {
        float u[8];
        gr_ld8(k + c, u);
#pragma unroll
        for (int e = 0; e < 8; ++e) sk = fmaf(u[e], u[e], sk);
        const int g = c / a.dm - a.g0;
        if (kept && g >= 0 && g < a.G) gr_st8(reinterpret_cast<T*>(a.kc) + (base + (int64_t)g * a.bs) * a.dm + c % a.dm, u);
    }
    if constexpr (CH > 0) {
#pragma unroll
        for (int j = 0; j < CH; ++j) {
            if ((tid + j * 256) * 8 >= a.nq) continue;
#pragma unroll
            for (int e = 0; e < 8; ++e) sq = fmaf(v[j][e], v[j][e], sq);
        }
    } else {
        for (int c = tid * 8; c < a.nq; c += 2048) {
            gr_ld8(q + c, v[0]);
#pragma unroll
            for (int e = 0; e < 8; ++e) sq = fmaf(v[0][e], v[0][e], sq);
        }
    }
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if (lane == 0) {
        red[0][wid] = sq;
        red[1][wid] = sk;
    }
    __syncthreads();
    sq = red[0][0] + red[0][1] + red[0][2] + red[0][3];
    sk = red[1][0] + red[1][1] + red[1][2] + red[1][3];
    if (tid == 0 && kept) a.kscale[slot] = 1.0f / sqrtf(sk / (float)a.k_n + a.eps);
    float f = 1.0f / sqrtf(sq / (float)a.q_n + a.eps);
    if (a.every > 0) f *= 1.0f + a.coef * logf((float)((pos + 1) / a.every) + 1.0f);
    auto put = [&](int c, float (&u)[8]) {
#pragma unroll
        for (int e = 0; e < 8; ++e) u[e] = u[e] * f * a.gq[c + e];
        gr_st8(q + c, u);
    };
    if constexpr (CH > 0) {
#pragma unroll
        for (int j = 0; j < CH; ++j) {
            const int c = (tid + j * 256) * 8;
            if (c < a.nq) put(c, v[j]);
        }
    } else {
        for (int c = tid * 8; c < a.nq; c += 2048) {
            gr_ld8(q + c, v[0]);
            put(c, v[0]);
        }
    }
}

int log2_of(int n) {
    for (int i = 0; i < 30; ++i)
        if (n == 1 << i) return i;
    return -1;
}

template <typename T>
void launch_rotate(RotArgs a, hipStream_t st) {
    const int unit = a.dims % 16 == 0 ? 8 : 1, half = a.dims / 2, nk = a.G * a.maps;
    a.per = (a.nq + nk) * (half / unit) + nk * ((a.dm - a.dims) / unit) + a.G * (a.dv / 8);
    const int parts = (a.per + 511) / 512, size = ((a.per + parts - 1) / parts + 63) / 64 * 64;  // equal parts of whole waves
    const dim3 grid((unsigned)a.T, (unsigned)parts);
    if (unit == 8) hipLaunchKernelGGL((group_rotate_store_kernel<T, 8>), grid, dim3(size), 0, st, a);
    else hipLaunchKernelGGL((group_rotate_store_kernel<T, 1>), grid, dim3(size), 0, st, a);
}
template <typename T>
void launch_norm(const NormArgs& a, int64_t rows, hipStream_t st) {
    const dim3 grid((unsigned)rows);
    if (a.nq <= 2048) hipLaunchKernelGGL((group_norm_store_kernel<T, 1>), grid, dim3(256), 0, st, a);
    else if (a.nq <= 4096) hipLaunchKernelGGL((group_norm_store_kernel<T, 2>), grid, dim3(256), 0, st, a);
    else if (a.nq <= 8192) hipLaunchKernelGGL((group_norm_store_kernel<T, 4>), grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((group_norm_store_kernel<T, 0>), grid, dim3(256), 0, st, a);
}

}  // namespace

extern "C" int glm_group_rotate_store(void* x, int64_t ld, int q_off, int k_off, int v_off, int f32, int H, int G, int maps, int dm, int dv, int dims, const float* cs, int pairs,
                                      const int32_t* slots, int64_t T, void* kc, void* vc, int64_t n_slots, int bs, glm_stream_t stream) {
    GLM_CHECK_ARG(x && cs && slots && kc && vc, GLM_ERR_INVALID, "glm_group_rotate_store: null pointer");
    GLM_CHECK_ARG(T >= 0 && H > 0 && G > 0 && (maps == 1 || maps == 2) && dm > 0 && dv > 0 && dm % 8 == 0 && dv % 8 == 0 && dims > 0 && dims % 2 == 0 && dims <= dm && pairs >= dims / 2 && (dims % 16 != 0 || (pairs % 2 == 0 && glm_aligned16(cs))) && bs > 0 &&
                      n_slots > 0 && n_slots < (1ll << 31) && n_slots % bs == 0 && q_off >= 0 && k_off >= 0 && v_off >= 0 && q_off % 8 == 0 && k_off % 8 == 0 && v_off % 8 == 0 && ld % 8 == 0 &&
                      ld >= q_off + (int64_t)H * maps * dm && ld >= k_off + (int64_t)G * maps * dm && ld >= v_off + (int64_t)G * dv && glm_aligned16(x) && glm_aligned16(kc) && glm_aligned16(vc) &&
                      T < (1ll << 31), GLM_ERR_INVALID, "glm_group_rotate_store: bad shape T=%ld H=%d G=%d dm=%d dv=%d dims=%d ld=%ld", (long)T, H, G, dm, dv, dims, (long)ld);
    if (T == 0) return GLM_OK;
    const RotArgs a = {x, ld, q_off, k_off, v_off, H * maps, G, maps, dm, dv, dims, cs, pairs, slots, kc, vc, (int)n_slots, bs, log2_of(bs), (int)T, 0};
    if (f32) launch_rotate<float>(a, glm_s(stream));
    else launch_rotate<bf16_t>(a, glm_s(stream));
    GLM_CHECK_LAUNCH("glm_group_rotate_store");
    return GLM_OK;
}

extern "C" int glm_group_norm_store(void* x, int64_t ld, int q_off, int nq, int q_n, int k_off, int nk, int k_n, int f32, const float* gq, int dm, int g0, int G, float eps, float coef,
                                    int every, const int32_t* pos, const int32_t* slots, int64_t T, void* kc, float* kscale, int64_t n_slots, int bs, glm_stream_t stream) {
    GLM_CHECK_ARG(x && gq && pos && slots && kc && kscale, GLM_ERR_INVALID, "glm_group_norm_store: null pointer");
    GLM_CHECK_ARG(T >= 0 && nq > 0 && nk > 0 && q_n > 0 && k_n > 0 && q_n <= nq && k_n <= nk && dm > 0 && dm % 8 == 0 && nq % dm == 0 && nk % dm == 0 && g0 >= 0 && G > 0 && (g0 + G) * dm <= nk &&
                      q_off >= 0 && k_off >= 0 && q_off % 8 == 0 && k_off % 8 == 0 && ld % 8 == 0 && ld >= (int64_t)q_off + nq && ld >= (int64_t)k_off + nk && every >= 0 && bs > 0 && n_slots > 0 && n_slots < (1ll << 31) &&
                      n_slots % bs == 0 && glm_aligned16(x) && glm_aligned16(kc) && T < (1ll << 31), GLM_ERR_INVALID,
                  "glm_group_norm_store: bad shape T=%ld nq=%d nk=%d dm=%d G=%d+%d ld=%ld", (long)T, nq, nk, dm, g0, G, (long)ld);
    if (T == 0) return GLM_OK;
    const NormArgs a = {x, ld, q_off, nq, q_n, k_off, nk, k_n, gq, dm, g0, G, eps, coef, every, pos, slots, kc, kscale, (int)n_slots, bs, log2_of(bs)};
    if (f32) launch_norm<float>(a, T, glm_s(stream));
    else launch_norm<bf16_t>(a, T, glm_s(stream));
    GLM_CHECK_LAUNCH("glm_group_norm_store");
    return GLM_OK;
}
