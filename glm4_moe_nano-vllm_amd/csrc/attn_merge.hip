// attn_merge.hip — sum of the KV splits of a decode attention: per (token, head) row the splits' unnormalised outputs, their maxima and
// masses (in log2 units) and the head's sink make the finished row; splits of weights that are not normalised are added up; of two maps per
// head the second's result, times lam, is taken off the first's and the difference normed.  A gate on the result is optional.  gfx950 only.
#include "common.h"

namespace {

constexpr float LOG2E = 1.4426950408889634f;

// ---------------------------------------------------------------------------------------------------------------------------
struct MergeArgs {
    const float *part_o, *part_ml, *sink;  // sink: [H] or nullptr
    int nsplit, plain_sum;                 // plain_sum: the weights are not normalised
    bf16_t* out;                           // [tokens, ldo], head h at h*cols
    int64_t ldo, rows;                     // (token, head) rows
    int H, cols, nchunk;
    const bf16_t* gate;                    // as in glm_group_form
    int64_t ldg;
    int gate_cols;
    float lam, post, eps;
    int vn;
};

// The splits of one row, N in flight: this wave adds up splits w, w + WPR, ... of the row's columns k .. k + 4, each weighed with its
// share of the row's mass (brought to the common maximum, over the mass of all and the sink's)
template <int WPR, int N>
__device__ __forceinline__ f32x4_t merge_row(const MergeArgs& a, int64_t prow, int h, int k, int lane, int w) {
    const float* p = a.part_o + prow * a.nsplit * a.cols + k;
    float m = -INFINITY, l = 0.f;
    if (lane < a.nsplit) {
        m = a.part_ml[(prow * a.nsplit + lane) * 2];
        l = a.part_ml[(prow * a.nsplit + lane) * 2 + 1];
    }
    f32x4_t o = {0.f, 0.f, 0.f, 0.f};
    float f = 0.f;
    for (int s0 = 0; s0 < a.nsplit; s0 += N * WPR) {
        f32x4_t x[N];
#pragma unroll
        for (int j = 0; j < N; ++j) x[j] = *reinterpret_cast<const f32x4_t*>(p + (int64_t)min(s0 + j * WPR + w, a.nsplit - 1) * a.cols);
        if (s0 == 0) {
            const float sk = a.sink ? a.sink[h] * LOG2E : -INFINITY;
            const float M = fmaxf(wave_max(m), sk);
            const float e = l > 0.f ? __builtin_amdgcn_exp2f(m - M) : 0.f;
            const float mass = wave_sum(l * e) + (a.sink ? __builtin_amdgcn_exp2f(sk - M) : 0.f);
            f = a.plain_sum ? (l > 0.f ? 1.0f : 0.f) : mass > 0.f ? e / mass : 0.f;  // 0: an empty split, its sums were never written
        }
#pragma unroll
        for (int j = 0; j < N; ++j) {
            const int s = s0 + j * WPR + w;
            const float fs = s < a.nsplit ? __shfl(f, s, 64) : 0.f;
            if (fs != 0.f) {
#pragma unroll
                for (int i = 0; i < 4; ++i) o[i] += fs * x[j][i];
            }
        }
    }
    return o;
}

// WPR waves (1 or 4) per (token, head) and 256 columns; two maps: all columns of a head together
template <bool TWO, int WPR, int N>
__global__ __launch_bounds__(256) void attn_merge_kernel(const MergeArgs a) {
    __shared__ f32x4_t sums[WPR == 1 ? 1 : (TWO ? 2 : 1) * (WPR - 1)][64];
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
    const int64_t item = WPR == 1 ? (int64_t)blockIdx.x * 4 + w : (int64_t)blockIdx.x;
    const int64_t grow = item / a.nchunk, t = grow / a.H;
    if (grow >= a.rows) return;
    const int k = (int)(item % a.nchunk) * 256 + lane * 4, h = (int)(grow - t * a.H), kk = k < a.cols ? k : 0;
    const bool on = k < a.cols;
    f32x4_t o, y;
    if constexpr (TWO) {
        o = merge_row<WPR, N>(a, grow * 2, h, kk, lane, WPR == 1 ? 0 : w);
        y = merge_row<WPR, N>(a, grow * 2 + 1, h, kk, lane, WPR == 1 ? 0 : w);
    } else {
        o = merge_row<WPR, N>(a, grow, h, kk, lane, WPR == 1 ? 0 : w);
    }
    if constexpr (WPR > 1) {
        if (w > 0) {
            sums[w - 1][lane] = o;
            if constexpr (TWO) sums[WPR - 1 + w - 1][lane] = y;
        }
        __syncthreads();
        if (w > 0) return;
#pragma unroll
        for (int i = 0; i < WPR - 1; ++i) {
            o += sums[i][lane];
            if constexpr (TWO) y += sums[WPR - 1 + i][lane];
        }
    }
    if constexpr (TWO) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            o[i] = o[i] - a.lam * y[i];
            ss += on ? o[i] * o[i] : 0.f;
        }
        o *= a.post / sqrtf(wave_sum(ss) / (float)a.vn + a.eps);
    }
    if (!on) return;
    if (a.gate) {
        const bf16_t* g = a.gate + t * a.ldg + (a.gate_cols ? (int64_t)h * a.cols + k : h);
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] *= bf2f(a.gate_cols ? g[i] : g[0]);
    }
    *reinterpret_cast<u32x2_t*>(a.out + t * a.ldo + (int64_t)h * a.cols + k) = u32x2_t{pack2bf(o[0], o[1]), pack2bf(o[2], o[3])};
}

template <int WPR, int N>
void launch(const MergeArgs& a, int maps, hipStream_t st) {
    const int64_t items = a.rows * a.nchunk;
    const dim3 grid((unsigned)(WPR == 1 ? (items + 3) / 4 : items));
    if (maps == 2) hipLaunchKernelGGL((attn_merge_kernel<true, WPR, N>), grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((attn_merge_kernel<false, WPR, N>), grid, dim3(256), 0, st, a);
}

}  // namespace

extern "C" int glm_attn_merge(const float* part_o, const float* part_ml, const float* sink, int nsplit, void* out, int64_t ldo, int64_t Ta, int H, int cols,
                              const glm_group_form* form, glm_stream_t stream) {
    const int maps = form ? form->maps : 1;
    GLM_CHECK_ARG(part_o && part_ml && out && nsplit >= 1 && nsplit <= 64 && Ta >= 0 && H > 0 && cols > 0 && cols % 8 == 0 && ldo >= (int64_t)H * cols && ldo % 4 == 0 &&
                      (((uintptr_t)out) & 7) == 0 && (maps == 1 || (maps == 2 && cols <= 256 && form->vn > 0)), GLM_ERR_INVALID,
                  "glm_attn_merge: bad shape Ta=%ld H=%d cols=%d splits=%d", (long)Ta, H, cols, nsplit);
    GLM_CHECK_ARG(Ta * H < (1ll << 26), GLM_ERR_UNSUPPORTED, "glm_attn_merge: too many rows");
    if (Ta == 0) return GLM_OK;
    MergeArgs a = {part_o, part_ml, sink, nsplit, 0, (bf16_t*)out, ldo, Ta * H, H, cols, (cols + 255) / 256, nullptr, 0, 0, 0.f, 0.f, 0.f, 0};
    if (form) {
        a.plain_sum = form->sigmoid;
        a.gate = (const bf16_t*)form->gate; a.ldg = form->ldg; a.gate_cols = form->gate_cols;
        a.lam = form->lam; a.post = form->post; a.eps = form->eps; a.vn = form->vn;
    }
    if (nsplit <= 4) launch<1, 4>(a, maps, glm_s(stream));
    else if (a.rows * a.nchunk <= 2048) launch<4, 8>(a, maps, glm_s(stream));
    else launch<1, 16>(a, maps, glm_s(stream));
    GLM_CHECK_LAUNCH("glm_attn_merge");
    return GLM_OK;
}
