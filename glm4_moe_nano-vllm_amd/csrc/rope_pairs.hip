// rope_pairs.hip — the rotation table of a step: cos and sin of every pair of rotated columns at the positions of its rows, shared by all
// layers with the same rotation.  gfx950 only.
#include "common.h"

namespace {

// cos and sin of every pair of rotated columns at the positions of a step, times mscale; the angle is taken in double and brought into
// one turn before it is rounded, so far positions are as exact as near ones.  Pairs behind the last frequency do not turn.
__global__ __launch_bounds__(256) void rope_pairs_kernel(const int32_t* pos, const double* freq, int n_freq, float mscale, float* cs, int64_t T, int pairs) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x, t = i / pairs;
    const int j = (int)(i % pairs);
    if (t >= T) return;
    float c = 1.f, s = 0.f;
    if (j < n_freq) {
        const double turns = (double)max(pos[t], 0) * freq[j] * 0.15915494309189533577;
        const float ang = (float)((turns - rint(turns)) * 6.28318530717958647693);
        c = cosf(ang) * mscale;
        s = sinf(ang) * mscale;
    }
    cs[i * 2] = c;
    cs[i * 2 + 1] = s;
}

}  // namespace

extern "C" int glm_rope_pairs(const int32_t* pos, const double* freq, int n_freq, float mscale, float* cs, int64_t T, int pairs, glm_stream_t stream) {
    GLM_CHECK_ARG(pos && cs && (freq || n_freq == 0) && T >= 0 && pairs > 0 && n_freq >= 0 && n_freq <= pairs && (T * pairs + 255) / 256 < (1ll << 31), GLM_ERR_INVALID,
                  "glm_rope_pairs: bad shape T=%ld pairs=%d freq=%d", (long)T, pairs, n_freq);
    if (T == 0) return GLM_OK;
    hipLaunchKernelGGL(rope_pairs_kernel, dim3((unsigned)((T * pairs + 255) / 256)), dim3(256), 0, glm_s(stream), pos, freq, n_freq, mscale, cs, T, pairs);
    GLM_CHECK_LAUNCH("glm_rope_pairs");
    return GLM_OK;
}
