// gemm_f32.hip — y = act(x · W^T + bias) in true fp32 (vector FMAs, no reduced-precision matrix mode), optionally batched.
// gfx950 only.  For models that are served in 32-bit: exactness first; a 64 x 64 tile per workgroup, 4 x 4 outputs per
// thread, 16-wide K slabs through LDS.  Every output is one fixed-order sum over K, whatever the number of rows.
#include "gemm_internal.h"

namespace {

constexpr int GF_B = 64, GF_K = 16, GF_PAD = 4;

struct GemmF32Args {
    const float *x, *w, *bias;
    float* y;
    int64_t ldx, xb, ldw, wb, ldy, yb, M;
    int N, K;
    GlmAct act;
    const int32_t *offs, *src;  // grouped: [G+1] row offsets of the groups (their weights wb apart), source row of row r (or nullptr)
    int G;
};

template <bool GROUPED>
__global__ __launch_bounds__(256) void gemm_f32_kernel(const GemmF32Args a) {
    __shared__ __attribute__((aligned(16))) float sx[GF_K][GF_B + GF_PAD], sw[GF_K][GF_B + GF_PAD];
    const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
    int64_t m0 = (int64_t)blockIdx.y * GF_B, m1 = a.M;
    const int n0 = blockIdx.x * GF_B;
    const float* x = a.x + blockIdx.z * a.xb;
    const float* w = a.w + blockIdx.z * a.wb;
    if constexpr (GROUPED) {
        __shared__ int s_blk[3];
        glm_locate_block(a.offs, a.G, a.M, GF_B, blockIdx.y, s_blk);
        __syncthreads();
        if (s_blk[0] < 0) return;
        m0 = s_blk[1];
        m1 = min(a.M, m0 + s_blk[2]);
        w = a.w + s_blk[0] * a.wb;
    }
    float acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = 0.f;
    const int lr = tid >> 2, lk = (tid & 3) * 4;  // row and K offset this thread stages
    int64_t xr = m0 + lr;
    if constexpr (GROUPED) {
        if (a.src && xr < m1) xr = a.src[xr];
    }
    for (int k0 = 0; k0 < a.K; k0 += GF_K) {
        f32x4_t vx = {0.f, 0.f, 0.f, 0.f}, vw = {0.f, 0.f, 0.f, 0.f};
        if (k0 + lk < a.K) {  // K is a multiple of 4
            if (m0 + lr < m1) vx = *reinterpret_cast<const f32x4_t*>(x + xr * a.ldx + k0 + lk);
            if (n0 + lr < a.N) vw = *reinterpret_cast<const f32x4_t*>(w + (int64_t)(n0 + lr) * a.ldw + k0 + lk);
        }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            sx[lk + i][lr] = vx[i];
            sw[lk + i][lr] = vw[i];
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < GF_K; ++k) {
            const f32x4_t xv = *reinterpret_cast<const f32x4_t*>(&sx[k][ty * 4]);
            const f32x4_t wv = *reinterpret_cast<const f32x4_t*>(&sw[k][tx * 4]);
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(xv[i], wv[j], acc[i][j]);
        }
    }
    float* y = a.y + blockIdx.z * a.yb;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int64_t m = m0 + ty * 4 + i;
        if (m >= m1) continue;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int n = n0 + tx * 4 + j;
            if (n >= a.N) continue;
            float v = acc[i][j];
            if (a.bias) v += a.bias[n];
            y[m * a.ldy + n] = glm_act_precise(a.act, v, n);
        }
    }
}

// y = clamped gated unit of fp32 rows gate | up (bf16: the epilogue of glm_gemm_bf16_glu)
__global__ __launch_bounds__(256) void glu_f32_kernel(const float* x, int64_t ldx, float* y, int64_t ldy, int64_t M, int N, GlmAct act) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x, r = i / N;
    const int c = (int)(i - r * N);
    if (r < M) y[r * ldy + c] = glm_glu_precise(act, x[r * ldx + c], x[r * ldx + N + c]);
}

// y = silu(gate) up of fp32 rows gate | up (bf16: the epilogue of glm_grouped_gemm_gateup_silu)
__global__ __launch_bounds__(256) void swiglu_f32_kernel(const float* x, int64_t ldx, float* y, int64_t ldy, int64_t M, int N) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x, r = i / N;
    const int c = (int)(i - r * N);
    if (r >= M) return;
    const float g = x[r * ldx + c];
    y[r * ldy + c] = g / (1.0f + expf(-g)) * x[r * ldx + N + c];
}

// y *= g (a gate that is through its sigmoid)
__global__ __launch_bounds__(256) void mul_f32_kernel(float* y, int64_t ldy, const float* g, int64_t ldg, int64_t M, int N) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x, r = i / N;
    const int c = (int)(i - r * N);
    if (r < M) y[r * ldy + c] *= g[r * ldg + c];
}

}  // namespace

extern "C" int glm_swiglu_f32(const float* x, int64_t ldx, float* y, int64_t ldy, int64_t M, int N, glm_stream_t stream) {
    GLM_CHECK_ARG(x && y && M >= 0 && N > 0 && ldx >= 2 * (int64_t)N && ldy >= N && (M * N + 255) / 256 < (1ll << 31), GLM_ERR_INVALID, "glm_swiglu_f32: bad shape M=%ld N=%d", (long)M, N);
    if (M == 0) return GLM_OK;
    hipLaunchKernelGGL(swiglu_f32_kernel, dim3((unsigned)((M * N + 255) / 256)), dim3(256), 0, glm_s(stream), x, ldx, y, ldy, M, N);
    GLM_CHECK_LAUNCH("glm_swiglu_f32");
    return GLM_OK;
}

extern "C" int glm_mul_f32(float* y, int64_t ldy, const float* g, int64_t ldg, int64_t M, int N, glm_stream_t stream) {
    GLM_CHECK_ARG(y && g && M >= 0 && N > 0 && ldy >= N && ldg >= N && (M * N + 255) / 256 < (1ll << 31), GLM_ERR_INVALID, "glm_mul_f32: bad shape M=%ld N=%d", (long)M, N);
    if (M == 0) return GLM_OK;
    hipLaunchKernelGGL(mul_f32_kernel, dim3((unsigned)((M * N + 255) / 256)), dim3(256), 0, glm_s(stream), y, ldy, g, ldg, M, N);
    GLM_CHECK_LAUNCH("glm_mul_f32");
    return GLM_OK;
}

extern "C" int glm_grouped_gemm_f32(const float* x, int64_t ldx, const float* w, int64_t w_group_stride, int64_t ldw, const int32_t* offsets, const int32_t* src,
                                    float* y, int64_t ldy, int64_t R, int N, int K, int G, glm_stream_t stream) {
    GLM_CHECK_ARG(x && w && y && offsets && R >= 0 && N > 0 && K > 0 && G > 0 && ldx >= K && ldw >= K && ldy >= N && w_group_stride >= (int64_t)N * ldw, GLM_ERR_INVALID,
                  "glm_grouped_gemm_f32: bad shape R=%ld N=%d K=%d G=%d", (long)R, N, K, G);
    GLM_CHECK_ARG(K % 4 == 0 && ldx % 4 == 0 && ldw % 4 == 0 && w_group_stride % 4 == 0 && glm_aligned16(x) && glm_aligned16(w), GLM_ERR_UNSUPPORTED,
                  "glm_grouped_gemm_f32: needs K, pitches %% 4 == 0 and 16-byte aligned operands (K=%d)", K);
    const int64_t gy = R / GF_B + G;
    GLM_CHECK_ARG(gy <= 65535, GLM_ERR_UNSUPPORTED, "glm_grouped_gemm_f32: too many rows (%ld)", (long)R);
    if (R == 0) return GLM_OK;
    GemmF32Args a = {x, w, nullptr, y, ldx, 0, ldw, w_group_stride, ldy, 0, R, N, K, {GLM_ACT_NONE, 0.f, 0.f}, offsets, src, G};
    hipLaunchKernelGGL(gemm_f32_kernel<true>, dim3((unsigned)((N + GF_B - 1) / GF_B), (unsigned)gy), dim3(256), 0, glm_s(stream), a);
    GLM_CHECK_LAUNCH("glm_grouped_gemm_f32");
    return GLM_OK;
}

extern "C" int glm_glu_f32(const float* x, int64_t ldx, float* y, int64_t ldy, int64_t M, int N, float limit, float slope, glm_stream_t stream) {
    GLM_CHECK_ARG(x && y && M >= 0 && N > 0 && ldx >= 2 * (int64_t)N && ldy >= N && (M * N + 255) / 256 < (1ll << 31), GLM_ERR_INVALID, "glm_glu_f32: bad shape M=%ld N=%d", (long)M, N);
    if (M == 0) return GLM_OK;
    hipLaunchKernelGGL(glu_f32_kernel, dim3((unsigned)((M * N + 255) / 256)), dim3(256), 0, glm_s(stream), x, ldx, y, ldy, M, N, GlmAct{GLM_ACT_GLU_CLAMP, limit, slope});
    GLM_CHECK_LAUNCH("glm_glu_f32");
    return GLM_OK;
}

extern "C" int glm_gemm_f32(const float* x, int64_t ldx, int64_t xb, const float* w, int64_t ldw, int64_t wb, const float* bias, float* y,
                            int64_t ldy, int64_t yb, int64_t M, int N, int K, int batch, int act, float act_a, float act_b, glm_stream_t stream) {
    GLM_CHECK_ARG(x && w && y && M >= 0 && N > 0 && K > 0 && batch > 0 && ldx >= K && ldw >= K && ldy >= N, GLM_ERR_INVALID,
                  "glm_gemm_f32: bad shape M=%ld N=%d K=%d", (long)M, N, K);
    GLM_CHECK_ARG(K % 4 == 0 && ldx % 4 == 0 && ldw % 4 == 0 && xb % 4 == 0 && wb % 4 == 0 && glm_aligned16(x) && glm_aligned16(w), GLM_ERR_UNSUPPORTED,
                  "glm_gemm_f32: needs K, ldx, ldw, batch strides %% 4 == 0 and 16-byte aligned operands (K=%d)", K);
    GLM_CHECK_ARG(act >= GLM_ACT_NONE && act <= GLM_ACT_RELU2_GATE && act != GLM_ACT_GLU_CLAMP, GLM_ERR_INVALID, "glm_gemm_f32: unknown activation %d", act);
    const int64_t gy = (M + GF_B - 1) / GF_B;
    GLM_CHECK_ARG(gy <= 65535 && batch <= 65535, GLM_ERR_UNSUPPORTED, "glm_gemm_f32: too many rows (%ld)", (long)M);
    if (M == 0) return GLM_OK;
    GemmF32Args a = {x, w, bias, y, ldx, xb, ldw, wb, ldy, yb, M, N, K, {act, act_a, act_b}, nullptr, nullptr, 1};
    hipLaunchKernelGGL(gemm_f32_kernel<false>, dim3((unsigned)((N + GF_B - 1) / GF_B), (unsigned)gy, (unsigned)batch), dim3(256), 0, glm_s(stream), a);
    GLM_CHECK_LAUNCH("glm_gemm_f32");
    return GLM_OK;
}
