// attn_merge.hip — sum of the KV splits of a decode attention: per (token, head) row the splits' unnormalised outputs, their maxima and
// masses (in log2 units) and the head's sink make the finished row.  gfx950 only.
#include "common.h"

namespace {

constexpr float LOG2E = 1.4426950408889634f;

// ---------------------------------------------------------------------------------------------------------------------------
// ctx = (sum over the KV splits, each brought to the common maximum) / (mass of the splits + the sink's): one wave per (token,
// head) and 256 columns, sixteen splits in flight
__global__ __launch_bounds__(256) void attn_merge_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml, const float* __restrict__ sink,
                                                         int nsplit, bf16_t* __restrict__ ctx, int64_t rows, int H, int cols, int nchunk) {
    const int lane = threadIdx.x & 63;
    const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    const int64_t grow = item / nchunk;
    if (grow >= rows) return;
    const int k = (int)(item % nchunk) * 256 + lane * 4;
    const bool on = k < cols;
    const float* p = part_o + grow * nsplit * cols + (on ? k : 0);
    float m = -INFINITY, l = 0.f;
    if (lane < nsplit) {
        m = part_ml[(grow * nsplit + lane) * 2];
        l = part_ml[(grow * nsplit + lane) * 2 + 1];
    }
    f32x4_t o = {0.f, 0.f, 0.f, 0.f};
    float f = 0.f;
    for (int s0 = 0; s0 < nsplit; s0 += 16) {
        f32x4_t x[16];
#pragma unroll
        for (int j = 0; j < 16; ++j) x[j] = *reinterpret_cast<const f32x4_t*>(p + (int64_t)min(s0 + j, nsplit - 1) * cols);
        if (s0 == 0) {
            const float sk = sink[grow % H] * LOG2E;
            const float M = fmaxf(wave_max(m), sk);
            const float e = l > 0.f ? __builtin_amdgcn_exp2f(m - M) : 0.f;
            f = e / (wave_sum(l * e) + __builtin_amdgcn_exp2f(sk - M));  // 0: an empty split, its sums were never written
        }
#pragma unroll
        for (int j = 0; j < 16; ++j) {
            const float fs = s0 + j < nsplit ? __shfl(f, s0 + j, 64) : 0.f;
            if (fs != 0.f) {
#pragma unroll
                for (int i = 0; i < 4; ++i) o[i] += fs * x[j][i];
            }
        }
    }
    if (on) *reinterpret_cast<u32x2_t*>(ctx + grow * cols + k) = u32x2_t{pack2bf(o[0], o[1]), pack2bf(o[2], o[3])};
}

}  // namespace

extern "C" int glm_attn_merge(const float* part_o, const float* part_ml, const float* sink, int nsplit, void* ctx, int64_t Ta, int H, int cols,
                                glm_stream_t stream) {
    GLM_CHECK_ARG(part_o && part_ml && sink && ctx && nsplit >= 1 && nsplit <= 64 && Ta >= 0 && H > 0 && cols > 0 && cols % 8 == 0, GLM_ERR_INVALID,
                  "glm_attn_merge: bad shape Ta=%ld H=%d cols=%d splits=%d", (long)Ta, H, cols, nsplit);
    GLM_CHECK_ARG(Ta * H < (1ll << 26), GLM_ERR_UNSUPPORTED, "glm_attn_merge: too many rows");
    if (Ta == 0) return GLM_OK;
    const int nchunk = (cols + 255) / 256;
    hipLaunchKernelGGL(attn_merge_kernel, dim3((unsigned)((Ta * H * nchunk + 3) / 4)), dim3(256), 0, glm_s(stream), part_o, part_ml, sink, nsplit, (bf16_t*)ctx,
                       Ta * H, H, cols, nchunk);
    GLM_CHECK_LAUNCH("glm_attn_merge");
    return GLM_OK;
}
