// window_attn.hip — varlen causal attention with a sliding window and a learned sink per head for prompts and long portions of
// prompts: q rows of the step against expanded k / v rows (the portion's own tokens and the part of the sequence's history that
// the window still reaches).  Head sizes of keys and values are independent, multiples of 8.  gfx950 only.
//
// Roofline: MFMA.  A workgroup owns 128 query rows of one (sequence, head); each of its 4 waves two 16-row query tiles, so
// that every K / V fragment read from LDS feeds two tiles.  64-key tiles are staged by LDS-DMA, double-buffered, one barrier per
// tile, only over the keys the rows can see: [first row - window + 1, last row].  S^T = K . Q^T, fp32 online softmax per lane
// column in log2 units, O^T += V^T . P^T straight from registers.  Tiles that all rows of a wave see in full take a path
// without masks; the running maximum is raised only when a score exceeds it by more than 2^8 (the sums stay exact:
// the reference point cancels).  The sink joins the denominator once, at the end.
#include "common.h"
#include "attn_lds.h"

namespace {

constexpr float WA_LOG2E = 1.4426950408889634f;
__device__ const u32x4_t wa_zero_page[4] = {};

struct WinArgs {
    const bf16_t* q;   // [rows, ldq], head h at h*dk
    int64_t ldq;
    const bf16_t *k, *v;  // [Tk, ldkv], head h at h*dkn / h*dv
    int64_t ldkv;
    const bf16_t* kr;  // [Tk, ldr] the last dk - dkn key columns, shared by all heads
    int64_t ldr;
    const float* cs;   // [rows, (dk - dkn) / 2, 2] rotation of those query columns, pairs (2i, 2i+1)
    const bf16_t* gate;  // [rows, ldg] factors of the output, laid out like out, or nullptr
    int64_t ldg;
    bf16_t* out;       // [rows, ldo], head h at h*dv
    int64_t ldo;
    const int32_t *q_start;  // [S+1] first q / out row of every sequence's portion
    const int32_t *k_start;  // [S+1] first k / v row
    const int32_t *tile_seq, *tile_off;  // [n_tiles]
    const float* sink;
    int S, n_tiles, H, dk, dkn, dv, window;
    int64_t Tq, Tk;
    float scale;
};

// DK, DV: multiples of 64
template <int DK, int DV>
__global__ __launch_bounds__(256, (DK + DV) <= 320 ? 2 : 1) void window_attn_kernel(const WinArgs a) {
    constexpr int KS = DK / 32, VT = DV / 16;
    constexpr bool VEARLY = DK + DV <= 256;                      // V fragments requested in front of the score products
    constexpr int KG = KS < 4 ? KS : 4, VG = VEARLY ? VT : 4;    // fragments per request group
    constexpr int KB = DK * 2, VB = DV * 2, KTILE = 64 * KB, VTILE = 64 * VB, STAGE = KTILE + VTILE;
    constexpr int KCPR = DK / 8, VCPR = DV / 8, KDMA = DK / 32, VDMA = DV / 32;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    const int tid = threadIdx.x, lane = tid & 63;
    const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4;
    // XCD-aware order: workgroups with equal id % 8 share an XCD and take one contiguous run of (head, tile) items
    const int total = a.n_tiles * a.H, per = (total + 7) >> 3;
    const int item = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per || item >= total) return;
    const int h = item / a.n_tiles, tile = item % a.n_tiles;
    const int seq = a.tile_seq[tile], qo = a.tile_off[tile];
    const int qs = a.q_start[seq], nq = a.q_start[seq + 1] - qs;
    const int ks0 = a.k_start[seq], nk = a.k_start[seq + 1] - ks0;
    const int hist = nk - nq;  // keys in front of the portion's first token
    if (qo >= nq || hist < 0) return;
    const int qlast = min(qo + 127, nq - 1);
    const int jlo = max(0, hist + qo - a.window + 1), jhi = hist + qlast;
    const int n = (jhi - jlo + 64) >> 6;
    // this wave's rows: tile t holds rows qo + 64 t + 16 w + c (the two half-dead tiles of the causal edge cost all waves the same)
    int rq[2];   // key index of the row itself; -1: no row
    u32x4_t qf[2][KS];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        const int r = qo + 64 * t + 16 * w + c;
        rq[t] = r < nq ? hist + r : -1;
        const bf16_t* qp = a.q + (int64_t)(qs + min(r, nq - 1)) * a.ldq + (int64_t)h * a.dk;
#pragma unroll
        for (int i = 0; i < KS; ++i) {
            const int k = 32 * i + 8 * g;
            qf[t][i] = u32x4_t{0, 0, 0, 0};
            if (k < a.dk) qf[t][i] = *reinterpret_cast<const u32x4_t*>(qp + k);
            if (k >= a.dkn && k < a.dk) {  // rotated here: a lane holds whole pairs
                const float* cs = a.cs + (int64_t)(qs + min(r, nq - 1)) * (a.dk - a.dkn) + (k - a.dkn);
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const float u = bflo(qf[t][i][j]), v = bfhi(qf[t][i][j]), co = cs[2 * j], si = cs[2 * j + 1];
                    qf[t][i][j] = pack2bf(u * co - v * si, v * co + u * si);
                }
            }
        }
    }
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int i = 0; i < KS; ++i) asm volatile("" : "+v"(qf[t][i]));
    const unsigned base = lds_addr(smem);
    const bf16_t* kbase = a.k + (int64_t)(ks0 + jlo) * a.ldkv + (int64_t)h * a.dkn;
    const bf16_t* rbase = a.kr ? a.kr + (int64_t)(ks0 + jlo) * a.ldr : kbase;
    const bf16_t* vbase = a.v + (int64_t)(ks0 + jlo) * a.ldkv + (int64_t)h * a.dv;
    const int nkeys = jhi - jlo + 1;
    // per-lane source offsets of the DMA pieces: constant over the tiles
    unsigned koff[KDMA], voff[VDMA];
    int krow[KDMA], vrow_[VDMA];
    bool kpad[KDMA], krot[KDMA], vpad[VDMA];
#pragma unroll
    for (int i = 0; i < KDMA; ++i) {
        const int q = (w * KDMA + i) * 64 + lane, row = q / KCPR, ch = (q % KCPR) ^ attn_swz(row);
        krow[i] = row;
        kpad[i] = ch * 8 >= a.dk;
        krot[i] = ch * 8 >= a.dkn;
        koff[i] = (unsigned)(krot[i] ? row * (int)a.ldr + ch * 8 - a.dkn : row * (int)a.ldkv + ch * 8);
    }
#pragma unroll
    for (int i = 0; i < VDMA; ++i) {
        const int q = (w * VDMA + i) * 64 + lane, row = q / VCPR, ch = (q % VCPR) ^ attn_swz(row);
        vrow_[i] = row;
        vpad[i] = ch * 8 >= a.dv;
        voff[i] = (unsigned)(row * (int)a.ldkv + ch * 8);
    }
    auto issue = [&](int it) {
        const int64_t adv = (int64_t)it * 64 * a.ldkv, advr = (int64_t)it * 64 * a.ldr;
        const int left = nkeys - it * 64;
        char* st = smem + (it & 1) * STAGE;
#pragma unroll
        for (int i = 0; i < KDMA; ++i) {
            const void* s = (kpad[i] || krow[i] >= left) ? (const void*)wa_zero_page : (const void*)((krot[i] ? rbase + advr : kbase + adv) + koff[i]);
            lds_dma16(s, st + (w * KDMA + i) * 1024);
        }
#pragma unroll
        for (int i = 0; i < VDMA; ++i) {
            const void* s = (vpad[i] || vrow_[i] >= left) ? (const void*)wa_zero_page : (const void*)(vbase + adv + voff[i]);
            lds_dma16(s, st + KTILE + (w * VDMA + i) * 1024);
        }
    };
    f32x4_t acc[2][VT];
    float m_run[2] = {-INFINITY, -INFINITY}, l_run[2] = {0.f, 0.f};
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int d = 0; d < VT; ++d) acc[t][d] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    // fragment offsets: K row 16 kt + c, chunk 4 i + g (its low three bits depend on the parity of i only); V row 4 g + qq
    unsigned k_rel[2], v_rel[4];
#pragma unroll
    for (int e = 0; e < 2; ++e) k_rel[e] = c * KB + (((4 * e + g) ^ attn_swz(c)) << 4);
    const int qq = (lane >> 2) & 3, pp = lane & 3, vr = 4 * g + qq;
#pragma unroll
    for (int e = 0; e < 4; ++e) v_rel[e] = vr * VB + (((2 * e + (pp >> 1)) ^ attn_swz(vr)) << 4) + ((pp & 1) << 3);
    const float sc = a.scale * WA_LOG2E;
    // key range every row of the wave's tile t sees in full / at all
    int full_lo[2], full_hi[2], any_lo[2], any_hi[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        const int r0 = qo + 64 * t + 16 * w;
        const bool some = r0 < nq;
        const int a0 = hist + r0, a1 = hist + min(r0 + 15, nq - 1);
        any_lo[t] = some ? a0 - a.window + 1 : 1 << 30;
        any_hi[t] = some ? a1 : -1;
        full_lo[t] = some ? a1 - a.window + 1 : 1 << 30;
        full_hi[t] = some ? a0 : -1;
    }
    issue(0);
    for (int it = 0; it < n; ++it) {
        wait_vm<0>();
        __builtin_amdgcn_s_barrier();
        if (it + 1 < n) issue(it + 1);
        const unsigned kst = base + (it & 1) * STAGE, vst = kst + KTILE;
#pragma unroll
        for (int sl = 0; sl < 2; ++sl) {  // 32-key slabs
            const int j0 = jlo + it * 64 + sl * 32;
            const bool live0 = j0 <= any_hi[0] && j0 + 31 >= any_lo[0], live1 = j0 <= any_hi[1] && j0 + 31 >= any_lo[1];
            if (!live0 && !live1) continue;
            u32x2_t vf[VG][2];
            auto read_v = [&](auto D0) {
                static_for<VG>([&](auto I) {
                    constexpr int i = decltype(I)::value, d = decltype(D0)::value + i;
                    lds_read_tr16_b64<(d >> 2) * 128>(vf[i][0], vst + sl * 32 * VB + v_rel[d & 3]);
                    lds_read_tr16_b64<(d >> 2) * 128 + 16 * VB>(vf[i][1], vst + sl * 32 * VB + v_rel[d & 3]);
                });
            };
            f32x4_t s[2][2];
#pragma unroll
            for (int t = 0; t < 2; ++t)
#pragma unroll
                for (int kt = 0; kt < 2; ++kt) s[t][kt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
            static_for<(KS + KG - 1) / KG>([&](auto G) {
                constexpr int k0 = decltype(G)::value * KG, kn = KS - k0 < KG ? KS - k0 : KG;
                constexpr bool last = k0 + KG >= KS;
                u32x4_t kf[2][KG];
                static_for<kn>([&](auto I) {
                    constexpr int i = k0 + decltype(I)::value;
                    lds_read_b128<(i >> 1) * 128>(kf[0][i - k0], kst + sl * 32 * KB + k_rel[i & 1]);
                    lds_read_b128<(i >> 1) * 128 + 16 * KB>(kf[1][i - k0], kst + sl * 32 * KB + k_rel[i & 1]);
                });
                if constexpr (last && VEARLY) {
                    read_v(std::integral_constant<int, 0>{});
                    // the K fragments are in; the V fragments (issued last) may still be on their way
                    asm volatile("s_waitcnt lgkmcnt(%0)" ::"i"(2 * VG <= 15 ? 2 * VG : 15) : "memory");
                } else {
                    wait_lds();
                }
#pragma unroll
                for (int i = 0; i < kn; ++i) asm volatile("" : "+v"(kf[0][i]), "+v"(kf[1][i]));
#pragma unroll
                for (int i = 0; i < kn; ++i)
#pragma unroll
                    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                        for (int t = 0; t < 2; ++t)
                            s[t][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kf[kt][i]), __builtin_bit_cast(bf16x8_t, qf[t][k0 + i]), s[t][kt], 0, 0, 0);
            });
            bf16x8_t pf[2];
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                if (!(t == 0 ? live0 : live1)) {
#pragma unroll
                    for (int i = 0; i < 8; ++i) pf[t][i] = (__bf16)0.f;
                    continue;
                }
                float mx = -INFINITY;
                if (j0 >= full_lo[t] && j0 + 31 <= full_hi[t]) {
#pragma unroll
                    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            s[t][kt][r] *= sc;
                            mx = fmaxf(mx, s[t][kt][r]);
                        }
                } else {
                    const int d0 = rq[t] - (j0 + 4 * g);
#pragma unroll
                    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            const int d = d0 - 16 * kt - r;
                            s[t][kt][r] = (rq[t] >= 0 && d >= 0 && d < a.window) ? s[t][kt][r] * sc : -INFINITY;
                            mx = fmaxf(mx, s[t][kt][r]);
                        }
                }
                if (__any(mx > m_run[t] + 8.0f || (m_run[t] == -INFINITY && mx > -INFINITY))) {
                    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
                    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
                    const float m_new = fmaxf(m_run[t], mx);
                    const float alpha = m_new == -INFINITY ? 1.0f : __builtin_amdgcn_exp2f(m_run[t] - m_new);
                    l_run[t] *= alpha;
#pragma unroll
                    for (int d = 0; d < VT; ++d) acc[t][d] *= alpha;
                    m_run[t] = m_new;
                }
                const float m_use = m_run[t] == -INFINITY ? 0.f : m_run[t];
#pragma unroll
                for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        const float p = __builtin_amdgcn_exp2f(s[t][kt][r] - m_use);
                        l_run[t] += p;
                        pf[t][4 * kt + r] = (__bf16)p;
                    }
            }
            static_for<VT / VG>([&](auto G) {
                constexpr int d0 = decltype(G)::value * VG;
                if constexpr (!VEARLY) read_v(std::integral_constant<int, d0>{});
                wait_lds();
#pragma unroll
                for (int i = 0; i < VG; ++i) asm volatile("" : "+v"(vf[i][0]), "+v"(vf[i][1]));
#pragma unroll
                for (int i = 0; i < VG; ++i) {
                    const u32x4_t vv = {vf[i][0][0], vf[i][0][1], vf[i][1][0], vf[i][1][1]};
#pragma unroll
                    for (int t = 0; t < 2; ++t)
                        acc[t][d0 + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, vv), pf[t], acc[t][d0 + i], 0, 0, 0);
                }
            });
        }
    }
    const float sk = a.sink[h] * WA_LOG2E;
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        float l = l_run[t];
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);
        const int r = qo + 64 * t + 16 * w + c;
        if (r >= nq) continue;
        const float M = fmaxf(m_run[t], sk), f = __builtin_amdgcn_exp2f(m_run[t] - M);
        const float inv = f / (l * f + __builtin_amdgcn_exp2f(sk - M));
        bf16_t* o = a.out + (int64_t)(qs + r) * a.ldo + (int64_t)h * a.dv;
#pragma unroll
        for (int d = 0; d < VT; ++d) {
            const int dim = 16 * d + 4 * g;
            if (a.gate && dim < a.dv) {
                const u32x2_t gt = *reinterpret_cast<const u32x2_t*>(a.gate + (int64_t)(qs + r) * a.ldg + (int64_t)h * a.dv + dim);
                acc[t][d] *= f32x4_t{bflo(gt[0]), bfhi(gt[0]), bflo(gt[1]), bfhi(gt[1])};
            }
            if (dim < a.dv) *reinterpret_cast<u32x2_t*>(o + dim) = u32x2_t{pack2bf(acc[t][d][0] * inv, acc[t][d][1] * inv), pack2bf(acc[t][d][2] * inv, acc[t][d][3] * inv)};
        }
    }
}

template <int DK, int DV>
int launch_window(const WinArgs& a, hipStream_t st) {
    constexpr int LDS = 2 * 64 * (DK + DV) * 2;
    static_assert(LDS <= 160 * 1024, "LDS of a CU");
    auto kern = window_attn_kernel<DK, DV>;
    GLM_SET_MAX_LDS(kern, LDS, "glm_window_attn_prefill");
    const int64_t per = ((int64_t)a.n_tiles * a.H + 7) / 8;
    GLM_CHECK_ARG(per * 8 < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_window_attn_prefill: grid too large");
    hipLaunchKernelGGL(kern, dim3((unsigned)(per * 8)), dim3(256), LDS, st, a);
    GLM_CHECK_LAUNCH("glm_window_attn_prefill");
    return GLM_OK;
}

template <int DK>
int launch_window_dv(const WinArgs& a, hipStream_t st) {
    if (a.dv <= 64) return launch_window<DK, 64>(a, st);
    if (a.dv <= 128) return launch_window<DK, 128>(a, st);
    if (a.dv <= 192) return launch_window<DK, 192>(a, st);
    return launch_window<DK, 256>(a, st);
}

}  // namespace

extern "C" int glm_window_attn_prefill(const void* q, int64_t ldq, const void* k, const void* v, int64_t ldkv, const void* kr, int64_t ldr, int rotp, const float* cs,
                                       const void* gate, int64_t ldg, void* out, int64_t ldo,
                                       const int32_t* q_start, const int32_t* k_start, const int32_t* tile_seq, const int32_t* tile_off, int n_tiles, int S,
                                       int64_t Tq, int64_t Tk, int H, int dk, int dv, int window, float scale, const float* sink, glm_stream_t stream) {
    GLM_CHECK_ARG(q && k && v && out && q_start && k_start && tile_seq && tile_off && sink, GLM_ERR_INVALID, "glm_window_attn_prefill: null pointer");
    GLM_CHECK_ARG(H > 0 && dk > 0 && dv > 0 && dk % 8 == 0 && dv % 8 == 0 && ldq >= (int64_t)H * dk && ldkv >= (int64_t)H * (dk - rotp > dv ? dk - rotp : dv) && ldo >= (int64_t)H * dv &&
                      ldq % 8 == 0 && ldkv % 8 == 0 && ldo % 4 == 0 && window > 0 && S > 0 && n_tiles >= 0 && Tq >= 0 && Tk >= Tq && ldkv < (1 << 24) &&
                      glm_aligned16(q) && glm_aligned16(k) && glm_aligned16(v), GLM_ERR_INVALID,
                  "glm_window_attn_prefill: bad shape H=%d dk=%d dv=%d ldq=%ld ldkv=%ld window=%d", H, dk, dv, (long)ldq, (long)ldkv, window);
    GLM_CHECK_ARG(dk <= 256 && dv <= 256, GLM_ERR_UNSUPPORTED, "glm_window_attn_prefill: head sizes up to 256 (dk=%d dv=%d)", dk, dv);
    GLM_CHECK_ARG(rotp >= 0 && rotp < dk && rotp % 8 == 0 && (rotp == 0 || (kr && cs && ldr >= rotp && ldr % 8 == 0 && ldr < (1 << 24) && glm_aligned16(kr))) &&
                      (!gate || (ldg >= (int64_t)H * dv && ldg % 4 == 0)), GLM_ERR_INVALID, "glm_window_attn_prefill: bad rotated part of %d columns or gate", rotp);
    if (n_tiles == 0) return GLM_OK;
    WinArgs a = {(const bf16_t*)q, ldq, (const bf16_t*)k, (const bf16_t*)v, ldkv, rotp ? (const bf16_t*)kr : nullptr, ldr, cs, (const bf16_t*)gate, ldg, (bf16_t*)out, ldo,
                 q_start, k_start, tile_seq, tile_off, sink, S, n_tiles, H, dk, dk - rotp, dv, window, Tq, Tk, scale};
    hipStream_t st = glm_s(stream);
    if (dk <= 64) return launch_window_dv<64>(a, st);
    if (dk <= 128) return launch_window_dv<128>(a, st);
    if (dk <= 192) return launch_window_dv<192>(a, st);
    return launch_window_dv<256>(a, st);
}
