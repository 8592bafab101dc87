// matrix_memory.hip — the gated matrix memory of a recurrent mixer (mLSTM of xLSTM).  Per head, with S [dim, vdim], n [dim] and a running
// maximum m that all start at zero, log gates i and f,
//
//     i_t = cap tanh(a_t / cap)             f_t = log sigmoid(cap tanh(b_t / cap))         a, b: projections with their biases
//     m_t = max(f_t + m_(t-1), i_t)
//     S_t = e^(f_t + m_(t-1) - m_t) S_(t-1) + e^(i_t - m_t) k_t v_t^T                      n_t likewise with k_t alone
//     o_t = S_t^T q_t dim^-1/2 / (max(|n_t . q_t| dim^-1/2, e^(-m_t)) + 1e-6)
//     y_t = o_t / rms(o_t) . norm . sigmoid(g_t)
//
// State, gates and everything between the projections and y in fp32.  gfx950 only.
//
// And its plain relative, the linear memory of attention with a constant decay per head (GATED = false):
//
//     S_t = decay S_(t-1) + k_t v_t^T        o_t = S_t^T q_t        y_t = o_t / rms(o_t) . norm . gate_t      the norm over all heads together
//
//   memory_recurrent   token by token, state in registers (decoded tokens, short portions, fp32): one (sequence, head) per workgroup, gate
//                      projections and the output norm included; memory_recurrent_any for head sizes beyond its registers
//   memory_gates       gate projections of long portions and the part of the gates' scan that stays inside a chunk of 64 tokens
//   memory_chunkwise   long portions: 64 tokens at a time on the matrix cores, one (sequence, head, 64 value columns) per workgroup
//   memory_output      norm and output gate of memory_chunkwise's rows
//   row_norm_gate      the linear memory's norm and gate, for rows of either form
//
// Rooflines: the recurrent form is HBM-bound (the state is read once and written once per step), the chunkwise form is bound by the chain
// of its chunks (the state of one is the input of the next).
//
// The chunkwise form, with b_t the running sum of f inside the chunk: m_t = b_t + max(m_in, max_(s<=t) (i_s - b_s)) is a scan over 64
// lanes; with D_ts = e^(b_t - m_t + i_s - b_s) for s <= t and c_t = e^(b_t + m_in - m_t),
//
//     S_t^T q_t = c_t S_in^T q_t + sum_s D_ts (k_s . q_t) v_s            S_out = c_L S_in + sum_s e^(b_L - m_L + i_s - b_s) k_s v_s^T
//
// (the linear memory: D_ts = decay^(t-s), c_t = decay^(t+1), from a table of powers; they are the same in every chunk and stay in registers)
//
// q, k and v are bf16 as the projection left them; the weights D (k . q), the decayed values and the state enter the matrix cores as a
// bf16 pair hi + lo each, so the products keep about 16 bits of their fp32 operand.
#include "common.h"
#include "attn_lds.h"

namespace {

constexpr float MM_LOG2E = 1.4426950408889634f;
__device__ const u32x4_t mm_zero_page[4] = {};

__device__ __forceinline__ float mm_log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float mm_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float mm_cap(float z, float cap) { return cap * tanhf(z / cap); }

struct RecArgs {
    const void* x;        // projection rows: q at h*dimp, k at k_off + h*dimp, v at v_off + h*vdimp, g at g_off + h*vdimp
    int64_t ldx, k_off, v_off, g_off;
    const void* hrow;     // [T, ldh] what the gates are projected from
    int64_t ldh;
    const void* wif;      // [2 H, ldw] rows i then f
    int64_t ldw;
    int wk;               // columns of hrow / wif
    const float* bif;     // [2 H]
    const float* norm;    // [H * vdimp]
    void* y;              // [T, ldy] head h at h*vdimp
    int64_t ldy;
    float *S, *n, *m;     // [rows][H][dimp][vdimp], [rows][H][dimp], [rows][H]
    int64_t n_state;
    const int32_t *pos, *q_start, *state_in, *state_out;
    int seqs, H, dim, dimp, vdim, vdimp;
    float cap, eps;
    const float* decay;   // [H]: the linear memory; y is then fp32 and holds o as it is
};

template <typename T>
__device__ __forceinline__ float mm_ld(const void* p, int64_t i) {
    if constexpr (sizeof(T) == 4) return reinterpret_cast<const float*>(p)[i];
    else return bf2f(reinterpret_cast<const bf16_t*>(p)[i]);
}
template <typename T>
__device__ __forceinline__ void mm_st(void* p, int64_t i, float v) {
    if constexpr (sizeof(T) == 4) reinterpret_cast<float*>(p)[i] = v;
    else reinterpret_cast<bf16_t*>(p)[i] = f2bf(v);
}
template <typename T>
__device__ __forceinline__ f32x4_t mm_ld4(const void* p, int64_t i) {
    if constexpr (sizeof(T) == 4) return *reinterpret_cast<const f32x4_t*>(reinterpret_cast<const float*>(p) + i);
    else {
        const u32x2_t u = *reinterpret_cast<const u32x2_t*>(reinterpret_cast<const bf16_t*>(p) + i);
        return f32x4_t{bflo(u[0]), bfhi(u[0]), bflo(u[1]), bfhi(u[1])};
    }
}
// this thread's share of the two gate projections of row r, head h
template <typename T>
__device__ __forceinline__ void mm_gate_parts(const RecArgs& a, int64_t r, int h, int tid, int nt, float& gi, float& gf) {
    gi = gf = 0.f;
    for (int c = tid * 4; c < a.wk; c += nt * 4) {
        const f32x4_t x = mm_ld4<T>(a.hrow, r * a.ldh + c), wi = mm_ld4<T>(a.wif, (int64_t)h * a.ldw + c), wf = mm_ld4<T>(a.wif, (int64_t)(a.H + h) * a.ldw + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            gi = fmaf(x[e], wi[e], gi);
            gf = fmaf(x[e], wf[e], gf);
        }
    }
}

__device__ __forceinline__ void mm_st_o(const RecArgs& a, int64_t r, int h, int c, float v) { reinterpret_cast<float*>(a.y)[r * a.ldy + (int64_t)h * a.vdimp + c] = v; }

// dimp <= 16 KD, vdimp <= 64 NW.  256 NW threads: column block tid / 256 (64 columns), thread (rg, cq) of a block holds rows rg + 16 k of the
// four columns cq.
template <typename T, int KD, int NW, bool GATED>
__global__ __launch_bounds__(256 * NW, GATED ? 1 : KD <= 8 ? 6 : 4) void memory_recurrent_kernel(const RecArgs a) {
    constexpr int NT = 256 * NW, NWV = 4 * NW;
    __shared__ float s_q[16 * KD], s_k[16 * KD], s_g[2][NWV], s_nq[NWV], s_ss[NWV];
    __shared__ __attribute__((aligned(16))) float s_o[NW][4][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int cb = tid >> 8, cq = tid & 15, rg = (tid >> 4) & 15, wv = (tid >> 6) & 3;
    const int seq = blockIdx.x / a.H, h = blockIdx.x % a.H;
    const int r0 = a.q_start[seq], r1 = a.q_start[seq + 1];
    const int c0 = GATED ? 0 : blockIdx.y * 64 * NW;   // (no sum over a head's value columns: they are shared out)
    const int col = c0 + cb * 64 + cq * 4;
    const bool con = col < a.vdimp;
    if (r1 <= r0) return;
    if (a.pos[r0] < 0) {  // unused rows of a padded batch
        for (int r = r0; r < r1; ++r) {
            if constexpr (GATED) {
                for (int c = tid; c < a.vdimp; c += NT) mm_st<T>(a.y, (int64_t)r * a.ldy + (int64_t)h * a.vdimp + c, 0.f);
            } else if (tid < 64 * NW && c0 + tid < a.vdimp) {
                mm_st_o(a, r, h, c0 + tid, 0.f);
            }
        }
        return;
    }
    f32x4_t S[KD];
    float n = 0.f, m = 0.f;
    const bool fresh = a.pos[r0] == 0;
    const int64_t sin = min(max((int64_t)a.state_in[seq], (int64_t)0), a.n_state - 1) * a.H + h;
#pragma unroll
    for (int k = 0; k < KD; ++k) {
        const int d = rg + 16 * k;
        S[k] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        if (!fresh && con && d < a.dimp) S[k] = *reinterpret_cast<const f32x4_t*>(a.S + (sin * a.dimp + d) * a.vdimp + col);
    }
    if (GATED && !fresh) {
        if (tid < a.dimp) n = a.n[sin * a.dimp + tid];
        m = a.m[sin];
    }
    const float scale = GATED ? 1.0f / sqrtf((float)a.dim) : 1.0f, bi = GATED ? a.bif[h] : 0.f, bf = GATED ? a.bif[a.H + h] : 0.f, inv_v = 1.0f / (float)a.vdim;
    float keep = GATED ? 0.f : a.decay[h], add = 1.0f;
    for (int r = r0; r < r1; ++r) {
        if constexpr (GATED) {
            float gi, gf;
            mm_gate_parts<T>(a, r, h, tid, NT, gi, gf);
            gi = wave_sum(gi);
            gf = wave_sum(gf);
            if (lane == 0) {
                s_g[0][wave] = gi;
                s_g[1][wave] = gf;
            }
        }
        const int64_t base = (int64_t)r * a.ldx;
        float kd = 0.f, qd = 0.f;
        if (tid < 16 * KD) {
            if (tid < a.dimp) {
                qd = mm_ld<T>(a.x, base + (int64_t)h * a.dimp + tid) * scale;
                kd = mm_ld<T>(a.x, base + a.k_off + (int64_t)h * a.dimp + tid);
            }
            s_q[tid] = qd;
            s_k[tid] = kd;
        }
        f32x4_t v = {0.f, 0.f, 0.f, 0.f};
        if (con) v = mm_ld4<T>(a.x, base + a.v_off + (int64_t)h * a.vdimp + col);
        __syncthreads();
        if constexpr (GATED) {
            float zi = 0.f, zf = 0.f;
#pragma unroll
            for (int w = 0; w < NWV; ++w) {
                zi += s_g[0][w];
                zf += s_g[1][w];
            }
            const float li = mm_cap(zi + bi, a.cap), lf = mm_log_sigmoid(mm_cap(zf + bf, a.cap));
            const float mn = fmaxf(lf + m, li);
            keep = expf(lf + m - mn);
            add = expf(li - mn);
            m = mn;
            n = keep * n + add * kd;
        }
        f32x4_t o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KD; ++k) {
            const float ak = add * s_k[rg + 16 * k], q = s_q[rg + 16 * k];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                S[k][e] = fmaf(ak, v[e], keep * S[k][e]);
                o[e] = fmaf(S[k][e], q, o[e]);
            }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            o[e] += __shfl_xor(o[e], 16, 64);
            o[e] += __shfl_xor(o[e], 32, 64);
        }
        if (lane < 16) *reinterpret_cast<f32x4_t*>(&s_o[cb][wv][cq * 4]) = o;
        float den = 0.f;
        if constexpr (GATED) {
            const float nq = wave_sum(n * qd);
            if (lane == 0) s_nq[wave] = nq;
        }
        __syncthreads();
        if constexpr (!GATED) {  // (s_o is written again behind the next token's first barrier)
            if (tid < 64 * NW && c0 + tid < a.vdimp) mm_st_o(a, r, h, c0 + tid, (s_o[tid >> 6][0][tid & 63] + s_o[tid >> 6][1][tid & 63]) + (s_o[tid >> 6][2][tid & 63] + s_o[tid >> 6][3][tid & 63]));
            continue;
        }
#pragma unroll
        for (int w = 0; w < NWV; ++w) den += s_nq[w];
        den = fmaxf(fabsf(den), expf(-m)) + 1e-6f;
        float ov = 0.f;  // thread tid owns column tid
        if (tid < a.vdimp) ov = (s_o[tid >> 6][0][tid & 63] + s_o[tid >> 6][1][tid & 63] + s_o[tid >> 6][2][tid & 63] + s_o[tid >> 6][3][tid & 63]) / den;
        const float ss = wave_sum(ov * ov);
        if (lane == 0) s_ss[wave] = ss;
        __syncthreads();
        float sq = 0.f;
#pragma unroll
        for (int w = 0; w < NWV; ++w) sq += s_ss[w];
        if (tid < a.vdimp) {
            const float rms = sqrtf(sq * inv_v + a.eps), g = mm_ld<T>(a.x, base + a.g_off + (int64_t)h * a.vdimp + tid);
            mm_st<T>(a.y, (int64_t)r * a.ldy + (int64_t)h * a.vdimp + tid, ov / rms * a.norm[(int64_t)h * a.vdimp + tid] * mm_sigmoid(g));
        }
    }
    const int64_t so = a.state_out[seq];
    if (so < 0 || so >= a.n_state) return;
    const int64_t sout = so * a.H + h;
#pragma unroll
    for (int k = 0; k < KD; ++k) {
        const int d = rg + 16 * k;
        if (con && d < a.dimp) *reinterpret_cast<f32x4_t*>(a.S + (sout * a.dimp + d) * a.vdimp + col) = S[k];
    }
    if constexpr (GATED) {
        if (tid < a.dimp) a.n[sout * a.dimp + tid] = n;
        if (tid == 0) a.m[sout] = m;
    }
}

// any head size: the state lives in its rows in memory (the row set that the step writes; scratch rows are not needed because a row set that
// nobody keeps is only ever asked for by unused rows)
template <typename T, bool GATED>
__global__ __launch_bounds__(256) void memory_recurrent_any_kernel(const RecArgs a) {
    extern __shared__ __attribute__((aligned(16))) char smem[];
    float* s_q = reinterpret_cast<float*>(smem);  // [dimp]
    float* s_k = s_q + a.dimp;                     // [dimp]
    float* s_o = s_k + a.dimp;                     // [vdimp]
    __shared__ __attribute__((aligned(16))) float s_part[16][64];
    __shared__ float s_red[3][4];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, cq = tid & 15, rg = tid >> 4;
    const int seq = blockIdx.x / a.H, h = blockIdx.x % a.H;
    const int r0 = a.q_start[seq], r1 = a.q_start[seq + 1];
    if (r1 <= r0) return;
    const int64_t so = a.state_out[seq];
    if (a.pos[r0] < 0 || so < 0 || so >= a.n_state) {
        for (int r = r0; r < r1; ++r)
            for (int c = tid; c < a.vdimp; c += 256) {
                if constexpr (GATED) mm_st<T>(a.y, (int64_t)r * a.ldy + (int64_t)h * a.vdimp + c, 0.f);
                else mm_st_o(a, r, h, c, 0.f);
            }
        return;
    }
    const int64_t sin = min(max((int64_t)a.state_in[seq], (int64_t)0), a.n_state - 1) * a.H + h, sout = so * a.H + h;
    const bool fresh = a.pos[r0] == 0;
    const float scale = GATED ? 1.0f / sqrtf((float)a.dim) : 1.0f, bi = GATED ? a.bif[h] : 0.f, bf = GATED ? a.bif[a.H + h] : 0.f, inv_v = 1.0f / (float)a.vdim;
    float m = !GATED || fresh ? 0.f : a.m[sin];
    float keep = GATED ? 0.f : a.decay[h], add = 1.0f;
    for (int r = r0; r < r1; ++r) {
        const bool first = r == r0;
        float gi = 0.f, gf = 0.f;
        if constexpr (GATED) {
            mm_gate_parts<T>(a, r, h, tid, 256, gi, gf);
            gi = wave_sum(gi);
            gf = wave_sum(gf);
        }
        __syncthreads();
        if (lane == 0) {
            s_red[0][wave] = gi;
            s_red[1][wave] = gf;
        }
        const int64_t base = (int64_t)r * a.ldx;
        for (int d = tid; d < a.dimp; d += 256) {
            s_q[d] = mm_ld<T>(a.x, base + (int64_t)h * a.dimp + d) * scale;
            s_k[d] = mm_ld<T>(a.x, base + a.k_off + (int64_t)h * a.dimp + d);
        }
        __syncthreads();
        const float zi = s_red[0][0] + s_red[0][1] + s_red[0][2] + s_red[0][3], zf = s_red[1][0] + s_red[1][1] + s_red[1][2] + s_red[1][3];
        float den = 1.0f;
        if constexpr (GATED) {
            const float li = mm_cap(zi + bi, a.cap), lf = mm_log_sigmoid(mm_cap(zf + bf, a.cap));
            const float mn = fmaxf(lf + m, li);
            keep = expf(lf + m - mn);
            add = expf(li - mn);
            m = mn;
            float nq = 0.f;
            for (int d = tid; d < a.dimp; d += 256) {
                const float old = !first ? a.n[sout * a.dimp + d] : fresh ? 0.f : a.n[sin * a.dimp + d];
                const float nn = keep * old + add * s_k[d];
                a.n[sout * a.dimp + d] = nn;
                nq += nn * s_q[d];
            }
            nq = wave_sum(nq);
            if (lane == 0) s_red[2][wave] = nq;
            __syncthreads();
            den = fmaxf(fabsf(s_red[2][0] + s_red[2][1] + s_red[2][2] + s_red[2][3]), expf(-m)) + 1e-6f;
        }
        float ss = 0.f;
        for (int c0 = 0; c0 < a.vdimp; c0 += 64) {
            const int col = c0 + cq * 4;
            f32x4_t o = {0.f, 0.f, 0.f, 0.f};
            if (col < a.vdimp) {
                const f32x4_t v = mm_ld4<T>(a.x, base + a.v_off + (int64_t)h * a.vdimp + col);
                for (int d = rg; d < a.dimp; d += 16) {
                    f32x4_t s = {0.f, 0.f, 0.f, 0.f};
                    if (!first) s = *reinterpret_cast<const f32x4_t*>(a.S + (sout * a.dimp + d) * a.vdimp + col);
                    else if (!fresh) s = *reinterpret_cast<const f32x4_t*>(a.S + (sin * a.dimp + d) * a.vdimp + col);
                    const float ak = add * s_k[d], q = s_q[d];
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        s[e] = fmaf(ak, v[e], keep * s[e]);
                        o[e] = fmaf(s[e], q, o[e]);
                    }
                    *reinterpret_cast<f32x4_t*>(a.S + (sout * a.dimp + d) * a.vdimp + col) = s;
                }
            }
            *reinterpret_cast<f32x4_t*>(&s_part[rg][cq * 4]) = o;
            __syncthreads();
            if (tid < 64 && c0 + tid < a.vdimp) {
                float ov = 0.f;
                for (int i = 0; i < 16; ++i) ov += s_part[i][tid];
                if constexpr (GATED) ov /= den;
                else mm_st_o(a, r, h, c0 + tid, ov);
                s_o[c0 + tid] = ov;
                ss += ov * ov;
            }
            __syncthreads();
        }
        if constexpr (!GATED) continue;
        if (wave == 0) {
            ss = wave_sum(ss);
            if (lane == 0) s_red[0][0] = ss;
        }
        __syncthreads();
        const float rms = sqrtf(s_red[0][0] * inv_v + a.eps);
        for (int c = tid; c < a.vdimp; c += 256)
            mm_st<T>(a.y, (int64_t)r * a.ldy + (int64_t)h * a.vdimp + c,
                     s_o[c] / rms * a.norm[(int64_t)h * a.vdimp + c] * mm_sigmoid(mm_ld<T>(a.x, base + a.g_off + (int64_t)h * a.vdimp + c)));
    }
    if (GATED && tid == 0) a.m[sout] = m;
}

// ---------------------------------------------------------------------------------------------------------------------------
// Gates of long portions, 64 tokens of a portion and up to 16 heads per workgroup: the two projections on the matrix cores (the four
// waves share K), then everything of a chunk that does not depend on the chunks before it.
struct GateArgs {
    const bf16_t* hrow;   // [rows, ldh]
    int64_t ldh;
    const bf16_t* wif;    // [2 H, ldw] rows i then f
    int64_t ldw;
    int wk;
    const float* bif;     // [2 H]
    float* gates;         // [3][H][rows], log2 units: i_s - b_s; b_s, the sum of f from the chunk's first token; running maximum of the first
    int64_t rows;
    const int32_t *q_start, *tile_seq, *tile_off;  // 128-row tiles
    int H;
    float cap;
};
__global__ __launch_bounds__(256) void memory_gates_kernel(const GateArgs a) {
    __shared__ float s_z[4][32][64];
    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, c = lane & 15, g = lane >> 4;
    const int tile = blockIdx.x >> 1, seq = a.tile_seq[tile], h0 = blockIdx.y * 16;
    const int qs = a.q_start[seq], T = a.q_start[seq + 1] - qs, off = a.tile_off[tile] + (blockIdx.x & 1) * 64;
    if (off >= T) return;
    const int n = min(64, T - off);
    f32x4_t acc[2][4];
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int t = 0; t < 4; ++t) acc[m][t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int wrow = min(h0 + c, a.H - 1);  // (heads behind the last one: computed again, not used)
    const bf16_t* wp[2] = {a.wif + (int64_t)wrow * a.ldw, a.wif + (int64_t)(a.H + wrow) * a.ldw};
    const bf16_t* hp[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) hp[t] = a.hrow + (int64_t)(qs + off + min(16 * t + c, n - 1)) * a.ldh;
    const u32x4_t zero = {0, 0, 0, 0};
#pragma unroll 4
    for (int k = w * 32 + 8 * g; k - 8 * g < a.wk; k += 128) {
        const bool on = k < a.wk;
        u32x4_t x[4], y[2];
#pragma unroll
        for (int m = 0; m < 2; ++m) y[m] = on ? *reinterpret_cast<const u32x4_t*>(wp[m] + k) : zero;
#pragma unroll
        for (int t = 0; t < 4; ++t) x[t] = on ? *reinterpret_cast<const u32x4_t*>(hp[t] + k) : zero;
#pragma unroll
        for (int m = 0; m < 2; ++m)
#pragma unroll
            for (int t = 0; t < 4; ++t)
                acc[m][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, y[m]), __builtin_bit_cast(bf16x8_t, x[t]), acc[m][t], 0, 0, 0);
    }
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) s_z[w][16 * m + 4 * g + r][16 * t + c] = acc[m][t][r];
    __syncthreads();
    for (int hh = w; hh < 16 && h0 + hh < a.H; hh += 4) {
        const int h = h0 + hh;
        float zi = a.bif[h], zf = a.bif[a.H + h];
#pragma unroll
        for (int x = 0; x < 4; ++x) {
            zi += s_z[x][hh][lane];
            zf += s_z[x][16 + hh][lane];
        }
        float b = mm_log_sigmoid(mm_cap(zf, a.cap));
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const float v = __shfl_up(b, o, 64);
            if (lane >= o) b += v;
        }
        const float as = mm_cap(zi, a.cap) - b;
        float mx = as;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const float v = __shfl_up(mx, o, 64);
            if (lane >= o) mx = fmaxf(mx, v);
        }
        if (lane < n) {
            float* o = a.gates + (int64_t)h * a.rows + qs + off + lane;
            const int64_t part = (int64_t)a.H * a.rows;
            o[0] = as * MM_LOG2E;
            o[part] = b * MM_LOG2E;
            o[2 * part] = mx * MM_LOG2E;
        }
    }
}

constexpr int MM_MAX_SEG = 8;
struct ChunkArgs {
    const bf16_t* x;      // projection rows (see RecArgs)
    int64_t ldx, k_off, v_off;
    const float* gates;   // [3][H][rows] of memory_gates
    int64_t rows;
    bf16_t* o;            // [rows, ldo] head h at h*vdimp, before the norm
    int64_t ldo;
    float *S, *n, *m;
    int64_t n_state;
    const int32_t *pos, *q_start, *state_in, *state_out;  // of the long portions; q_start and pos relative to x's first row
    int H, dim, dimp, vdimp, vtiles;
    const float* powers;  // [H][65] decay^j: the linear memory
    float seg[MM_MAX_SEG + 1];  // where its segments begin, as parts of a sequence
};

template <typename T>
__device__ __forceinline__ T mm_lds(const char* p) { return *reinterpret_cast<const T*>(p); }
// four transposed reads, complete when they return: the compiler would drain the LDS-DMA that is in flight in front of its own
template <int O0, int O1, int O2, int O3>
__device__ __forceinline__ void mm_lds_tr4(u32x2_t (&d)[2][2], const char* p) {
    asm volatile("ds_read_b64_tr_b16 %0, %4 offset:%5\n\tds_read_b64_tr_b16 %1, %4 offset:%6\n\tds_read_b64_tr_b16 %2, %4 offset:%7\n\t"
                 "ds_read_b64_tr_b16 %3, %4 offset:%8\n\ts_waitcnt lgkmcnt(0)"
                 : "=&v"(d[0][0]), "=&v"(d[0][1]), "=&v"(d[1][0]), "=&v"(d[1][1]) : "v"(lds_addr(p)), "i"(O0), "i"(O1), "i"(O2), "i"(O3) : "memory");
}
// sixteen of them: rows 0, 16, 32, 48 (pitch RB) at four addresses
template <int RB>
__device__ __forceinline__ void mm_lds_tr16(u32x2_t (&d)[4][2][2], unsigned p0, unsigned p1, unsigned p2, unsigned p3) {
#define MM_TR(D, P, O) "ds_read_b64_tr_b16 " D ", " P " offset:" O "\n\t"
    asm volatile(MM_TR("%0", "%16", "%20") MM_TR("%1", "%16", "%21") MM_TR("%2", "%16", "%22") MM_TR("%3", "%16", "%23")
                 MM_TR("%4", "%17", "%20") MM_TR("%5", "%17", "%21") MM_TR("%6", "%17", "%22") MM_TR("%7", "%17", "%23")
                 MM_TR("%8", "%18", "%20") MM_TR("%9", "%18", "%21") MM_TR("%10", "%18", "%22") MM_TR("%11", "%18", "%23")
                 MM_TR("%12", "%19", "%20") MM_TR("%13", "%19", "%21") MM_TR("%14", "%19", "%22") MM_TR("%15", "%19", "%23") "s_waitcnt lgkmcnt(0)"
                 : "=&v"(d[0][0][0]), "=&v"(d[0][0][1]), "=&v"(d[0][1][0]), "=&v"(d[0][1][1]), "=&v"(d[1][0][0]), "=&v"(d[1][0][1]), "=&v"(d[1][1][0]), "=&v"(d[1][1][1]),
                   "=&v"(d[2][0][0]), "=&v"(d[2][0][1]), "=&v"(d[2][1][0]), "=&v"(d[2][1][1]), "=&v"(d[3][0][0]), "=&v"(d[3][0][1]), "=&v"(d[3][1][0]), "=&v"(d[3][1][1])
                 : "v"(p0), "v"(p1), "v"(p2), "v"(p3), "i"(0), "i"(16 * RB), "i"(32 * RB), "i"(48 * RB) : "memory");
#undef MM_TR
}
// v = hi + lo, two bf16 each
__device__ __forceinline__ void mm_split(const float (&v)[8], bf16x8_t& hi, bf16x8_t& lo) {
    typedef __attribute__((ext_vector_type(2))) float f32x2;
    typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2;
    u32x4_t h, l;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        h[e] = __builtin_bit_cast(unsigned, __builtin_convertvector((f32x2{v[2 * e], v[2 * e + 1]}), bf16x2));
        l[e] = __builtin_bit_cast(unsigned, __builtin_convertvector((f32x2{v[2 * e] - bflo(h[e]), v[2 * e + 1] - bfhi(h[e])}), bf16x2));
    }
    hi = __builtin_bit_cast(bf16x8_t, h);
    lo = __builtin_bit_cast(bf16x8_t, l);
}
// barrier that leaves LDS-DMA in flight
__device__ __forceinline__ void mm_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
}
__device__ __forceinline__ bf16x8_t mm_frag(const u32x2_t& x, const u32x2_t& y) { return __builtin_bit_cast(bf16x8_t, u32x4_t{x[0], x[1], y[0], y[1]}); }
__device__ __forceinline__ f32x4_t mm_f4(const u32x4_t& v) { return __builtin_bit_cast(f32x4_t, v); }
__device__ __forceinline__ f32x4_t mm_mfma(const bf16x8_t& x, const bf16x8_t& y, const f32x4_t& z) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, y, z, 0, 0, 0); }

// D: multiple of 64, dimp <= D <= 256.  Eight waves; wave (v, dh) = (w & 3, w >> 2) computes the scores of query rows 16 v .. + 15 with half dh
// of the keys, and owns the part d in half dh, value columns 16 v .. + 15 of the state.  That part, in the matrix cores' output layout
// (lane (c, g): column c, rows d = 16 i + 4 g + r), is the left operand of the next chunk's readout without leaving the registers.  Of
// the 64 output rows, half 0 finishes row tiles 0 and 3, half 1 tiles 1 and 2 (equal work under the causal mask); the readouts of the
// other half come through LDS.
template <int D, bool GATED>
__global__ __launch_bounds__(512, 2) void memory_chunkwise_kernel(const ChunkArgs a) {
    constexpr int KS = D / 32, DT = D / 16, HT = DT / 2, RB = D * 2, CPR = D / 8, QT = 64 * RB, VTB = 64 * 128, GT = 1024, STAGE = 2 * QT + VTB + GT;
    constexpr int NST = D <= 128 ? 3 : 2;           // LDS stages: chunks on their way are NST - 1
    constexpr int QDMA = D / 64;                    // 1 KiB pieces per wave (of q, of k; one of v, one of the gates)
    // the weights (hi, lo: 16 KiB) and the readouts that change hands (16 KiB) go over the chunk's query rows, which are done by then, as far as
    // these reach
    constexpr bool PALIAS = QT >= 16384, XALIAS = QT >= 32768;
    constexpr int POFF = PALIAS ? 0 : NST * STAGE, XOFF = XALIAS ? 16384 : NST * STAGE + (PALIAS ? 0 : 16384), SMALL = NST * STAGE + (PALIAS ? 0 : 16384) + (XALIAS ? 0 : 16384);
    extern __shared__ __attribute__((aligned(16))) char smem[];
    float* s_a = reinterpret_cast<float*>(smem + SMALL);  // i_s - b_s                   (log2 units)
    float* s_row = s_a + 64;                               // b_t - m_t                   (log2 units)
    float* s_in = s_row + 64;                              // c_t dim^-1/2
    float* s_floor = s_in + 64;                            // e^(-m_t)
    float* s_w = s_floor + 64;                             // e^(b_L - m_L + i_s - b_s)
    float* s_den = s_w + 64;                               // n_t . q_t, two parts [2][64]
    float* s_n = s_den + 128;                              // [D]
    const int tid = threadIdx.x, lane = tid & 63;
    const int w = __builtin_amdgcn_readfirstlane(tid >> 6), v = w & 3, dh = w >> 2;
    const int c = lane & 15, g = lane >> 4;
    const int vt = blockIdx.x % a.vtiles, h = (blockIdx.x / a.vtiles) % a.H, seq = blockIdx.x / (a.vtiles * a.H);
    const int r0 = a.q_start[seq], T = a.q_start[seq + 1] - r0;
    if (T <= 0) return;
    // chunks [ch0, n_chunks) are this workgroup's.  The linear memory's few (sequence, head) pairs are cut into segments: a workgroup brings the
    // state up to its segment by itself, which costs a fraction of a chunk's work (no scores, no readout)
    int n_chunks = (T + 63) >> 6, ch0 = 0;
    const bool keeps = GATED || blockIdx.y + 1 == gridDim.y;
    if constexpr (!GATED) {
        ch0 = (int)((float)n_chunks * a.seg[blockIdx.y]);
        if (!keeps) n_chunks = (int)((float)n_chunks * a.seg[blockIdx.y + 1]);
        if (ch0 >= n_chunks) return;
    }
    const bool fresh = a.pos[r0] <= 0;
    const int64_t sin = min(max((int64_t)a.state_in[seq], (int64_t)0), a.n_state - 1) * a.H + h;
    const int col = vt * 64 + 16 * v + c;  // this lane's value column
    const bool con = col < a.vdimp;
    f32x4_t S[HT];
#pragma unroll
    for (int i = 0; i < HT; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = 16 * (dh * HT + i) + 4 * g + r;
            S[i][r] = (!fresh && con && d < a.dimp) ? a.S[(sin * a.dimp + d) * a.vdimp + col] : 0.f;
        }
    // n of the rows d = 16 (dh HT + i) + c with i = v mod 4 (the same in all four lane groups)
    constexpr int NR = HT > 4 ? HT / 4 : 1;
    float nreg[NR];
#pragma unroll
    for (int i = 0; i < NR; ++i) {
        const int d = 16 * (dh * HT + 4 * i + v) + c;
        nreg[i] = (GATED && !fresh && v < HT && d < a.dimp) ? a.n[sin * a.dimp + d] : 0.f;
        if (GATED && g == 0 && v < HT) s_n[d] = nreg[i];
    }
    float m_in = !GATED || fresh ? 0.f : a.m[sin];
    const float scale = GATED ? 1.0f / sqrtf((float)a.dim) : 1.0f;
    // the linear memory's weights: of this wave's rows and keys, of its output rows, of a token in the state behind a whole chunk
    float dw_c[2][4], wt_c[2][8], inc_a = 0.f, inc_b = 0.f, carry_c = 0.f;
    const float* pw = GATED ? nullptr : a.powers + h * 65;
    if constexpr (!GATED) {
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int d = 16 * v + c - (32 * dh + 16 * u + 4 * g + r);
                dw_c[u][r] = d >= 0 ? pw[d] : 0.f;
            }
#pragma unroll
        for (int sl = 0; sl < 2; ++sl)
#pragma unroll
            for (int e = 0; e < 8; ++e) wt_c[sl][e] = pw[63 - (32 * sl + 4 * g + (e & 3) + (e & 4) * 4)];
        inc_a = pw[16 * (dh ? 1 : 0) + c + 1];
        inc_b = pw[16 * (dh ? 2 : 3) + c + 1];
        carry_c = pw[64];
    }
    const bf16_t* xq = a.x + (int64_t)r0 * a.ldx + (int64_t)h * a.dimp;
    const bf16_t* xv = a.x + (int64_t)r0 * a.ldx + a.v_off + (int64_t)h * a.vdimp + vt * 64;
    const float* gp = GATED ? a.gates + (int64_t)h * a.rows + r0 : nullptr;
    const int64_t gpart = (int64_t)a.H * a.rows;
    // per-lane source offsets of the DMA pieces: constant over the chunks
    unsigned qoff[QDMA];
#pragma unroll
    for (int i = 0; i < QDMA; ++i) {
        const int p = (w * QDMA + i) * 64 + lane, row = p / CPR;
        qoff[i] = (unsigned)(row * (int)a.ldx + ((p % CPR) ^ attn_swz(row)) * 8);
    }
    const int vrow = w * 8 + (lane >> 3), vcc = (lane & 7) ^ attn_swz(vrow);
    const unsigned voff = (unsigned)(vrow * (int)a.ldx + vcc * 8);
    const bool whole = a.dimp == D && vt * 64 + 64 <= a.vdimp;  // no padding columns in this workgroup's tiles
    auto issue = [&](int ch) {
        char* st = smem + (ch % NST) * STAGE;
        const int left = T - ch * 64;
        // gates: i - b, b and the running maximum, 256 bytes each (the other waves' piece is not used)
        if constexpr (GATED) __builtin_amdgcn_global_load_lds((attn_glb_void*)(gp + min(w, 2) * gpart + ch * 64 + min(lane, left - 1)), (attn_lds_void*)(st + 2 * QT + VTB + min(w, 3) * 256), 4, 0, 0);
        const bf16_t *q = xq + (int64_t)ch * 64 * a.ldx, *k = q + a.k_off, *vv = xv + (int64_t)ch * 64 * a.ldx;
        const bool full = GATED || ch >= ch0;
        if (whole && left >= 64) {
#pragma unroll
            for (int i = 0; i < QDMA; ++i) {
                if (full) lds_dma16(q + qoff[i], st + (w * QDMA + i) * 1024);
                lds_dma16(k + qoff[i], st + QT + (w * QDMA + i) * 1024);
            }
            lds_dma16(vv + voff, st + 2 * QT + w * 1024);
            return;
        }
#pragma unroll
        for (int i = 0; i < QDMA; ++i) {
            const int p = (w * QDMA + i) * 64 + lane, row = p / CPR, cc = (p % CPR) ^ attn_swz(row);
            const bool ok = row < left && cc * 8 < a.dimp;
            if (full) lds_dma16(ok ? (const void*)(q + qoff[i]) : (const void*)mm_zero_page, st + (w * QDMA + i) * 1024);
            lds_dma16(ok ? (const void*)(k + qoff[i]) : (const void*)mm_zero_page, st + QT + (w * QDMA + i) * 1024);
        }
        const bool ok = vrow < left && vt * 64 + vcc * 8 < a.vdimp;
        lds_dma16(ok ? (const void*)(vv + voff) : (const void*)mm_zero_page, st + 2 * QT + w * 1024);
    };
    // fragment offsets.  Rows by 16 (lane c), eight columns 32 i + 8 g: the scores.  Rows by 16, columns 32 i + 4 g and + 16: the readout,
    // in the order of the state's registers.  Transposed reads, rows 4 g + qq: k and v over tokens.
    unsigned row_rel[2], half_rel[2][2], tr_rel[4], vt_rel;
#pragma unroll
    for (int e = 0; e < 2; ++e) {
        row_rel[e] = c * RB + (((4 * e + g) ^ attn_swz(c)) << 4);
#pragma unroll
        for (int u = 0; u < 2; ++u) half_rel[e][u] = c * RB + (((4 * e + 2 * u + (g >> 1)) ^ attn_swz(c)) << 4) + ((g & 1) << 3);
    }
    const int qq = (lane >> 2) & 3, pp = lane & 3, tr = 4 * g + qq;
#pragma unroll
    for (int e = 0; e < 4; ++e) tr_rel[e] = tr * RB + (((2 * e + (pp >> 1)) ^ attn_swz(tr)) << 4) + ((pp & 1) << 3);
    vt_rel = tr * 128 + (((2 * v + (pp >> 1)) ^ attn_swz(tr)) << 4) + ((pp & 1) << 3);
    const int rt_a = dh ? 1 : 0, rt_b = dh ? 2 : 3;   // the output row tiles this wave finishes
    m_in *= MM_LOG2E;
#pragma unroll
    for (int i = 0; i < NST - 1; ++i)
        if (i < n_chunks) issue(i);
    const char* sa = smem + SMALL;
    // a chunk's output rows are stored behind the next chunk's first barrier: their way to memory is then not waited for
    u32x2_t rows_out[2];
    const int vc = vt * 64 + 16 * v + 4 * g;
    auto store_rows = [&](int ch) {
        const int left = T - ch * 64;
        bf16_t* o = a.o + (int64_t)(r0 + ch * 64 + c) * a.ldo + (int64_t)h * a.vdimp + vc;
        if (16 * rt_a + c < left && vc < a.vdimp) *reinterpret_cast<u32x2_t*>(o + (int64_t)(16 * rt_a) * a.ldo) = rows_out[0];
        if (16 * rt_b + c < left && vc < a.vdimp) *reinterpret_cast<u32x2_t*>(o + (int64_t)(16 * rt_b) * a.ldo) = rows_out[1];
    };
    for (int ch = 0; ch < n_chunks; ++ch) {
        const int left = T - ch * 64;
        // the chunk is in (what was issued behind it may be on its way): loads return in order
        const bool full = GATED || ch >= ch0;
        if (ch + NST - 2 >= n_chunks) wait_vm<0>();
        else if (GATED || ch + NST - 2 >= ch0) wait_vm<(NST - 2) * (2 * QDMA + (GATED ? 2 : 1))>();
        else wait_vm<(NST - 2) * (QDMA + 1)>();
        mm_barrier();  // ... for every wave, and every wave is past its reads of the chunk before
        if (ch > ch0) store_rows(ch - 1);
        if (ch + NST - 1 < n_chunks) issue(ch + NST - 1);
        const char *qst = smem + (ch % NST) * STAGE, *kst = qst + QT, *vst = kst + QT, *gst = vst + VTB;
        char *pst = smem + (PALIAS ? (ch % NST) * STAGE : POFF), *xst = smem + (XALIAS ? (ch % NST) * STAGE : 0) + XOFF;
        // gates of the chunk, one token per lane, the same in every wave
        const bool tok = GATED && lane < left;
        const float ga = tok ? mm_lds<float>(gst + 4 * lane) : -INFINITY, gb = tok ? mm_lds<float>(gst + 256 + 4 * lane) : 0.f,
                    gm = tok ? mm_lds<float>(gst + 512 + 4 * lane) : 0.f;
        const float mt = gb + fmaxf(m_in, gm);
        const int last = min(left, 64) - 1;
        float bL = 0.f, mL = 0.f, carry;
        if constexpr (GATED) {
            bL = __shfl(gb, last, 64);
            mL = __shfl(mt, last, 64);
            carry = __builtin_amdgcn_exp2f(bL + m_in - mL);
        } else {
            carry = last == 63 ? carry_c : pw[last + 1];
        }
        if (GATED && w == 0) {
            s_a[lane] = ga;
            s_row[lane] = gb - mt;
            s_in[lane] = __builtin_amdgcn_exp2f(gb + m_in - mt) * scale;
            s_floor[lane] = __builtin_amdgcn_exp2f(-mt);
            s_w[lane] = __builtin_amdgcn_exp2f(bL - mL + ga);
        }
        // ---- scores of 16 query rows with 32 keys; n . q of these rows, over this half's d ----
        f32x4_t s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
        float nq = 0.f;
        if (full) static_for<KS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const u32x4_t qf = mm_lds<u32x4_t>(qst + v * 16 * RB + row_rel[i & 1] + (i >> 1) * 128);
            const u32x4_t k0 = mm_lds<u32x4_t>(kst + dh * 32 * RB + row_rel[i & 1] + (i >> 1) * 128), k1 = mm_lds<u32x4_t>(kst + dh * 32 * RB + row_rel[i & 1] + (i >> 1) * 128 + 16 * RB);
            s[0] = mm_mfma(__builtin_bit_cast(bf16x8_t, k0), __builtin_bit_cast(bf16x8_t, qf), s[0]);
            s[1] = mm_mfma(__builtin_bit_cast(bf16x8_t, k1), __builtin_bit_cast(bf16x8_t, qf), s[1]);
            if (GATED && i / (KS / 2) == dh) {
                const f32x4_t n0 = mm_lds<f32x4_t>(sa + 1792 + 128 * i + 32 * g), n1 = mm_lds<f32x4_t>(sa + 1792 + 128 * i + 32 * g + 16);
#pragma unroll
                for (int e = 0; e < 2; ++e) {
                    nq = fmaf(bflo(qf[e]), n0[2 * e], nq);
                    nq = fmaf(bfhi(qf[e]), n0[2 * e + 1], nq);
                    nq = fmaf(bflo(qf[2 + e]), n1[2 * e], nq);
                    nq = fmaf(bfhi(qf[2 + e]), n1[2 * e + 1], nq);
                }
            }
        });
        // ---- what this part of the state gives all 64 rows, in this wave's columns ----
        f32x4_t acc[4];
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) acc[rt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        const char* qh_st = qst + (KS / 2 >= 2 ? dh * (KS / 4) * 128 : 0);   // columns of this half: 128 bytes hold 64 of them
        if (full) static_for<KS / 2>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const unsigned ra = KS / 2 >= 2 ? half_rel[i & 1][0] : (dh ? half_rel[1][0] : half_rel[0][0]), rb = KS / 2 >= 2 ? half_rel[i & 1][1] : (dh ? half_rel[1][1] : half_rel[0][1]);
            const f32x4_t &u = S[2 * i], &x = S[2 * i + 1];
            const float sv[8] = {u[0], u[1], u[2], u[3], x[0], x[1], x[2], x[3]};
            bf16x8_t hi, lo, q[4];
            mm_split(sv, hi, lo);
#pragma unroll
            for (int rt = 0; rt < 4; ++rt) q[rt] = mm_frag(mm_lds<u32x2_t>(qh_st + ra + (i >> 1) * 128 + rt * 16 * RB), mm_lds<u32x2_t>(qh_st + rb + (i >> 1) * 128 + rt * 16 * RB));
#pragma unroll
            for (int rt = 0; rt < 4; ++rt) acc[rt] = mm_mfma(hi, q[rt], acc[rt]);
#pragma unroll
            for (int rt = 0; rt < 4; ++rt) acc[rt] = mm_mfma(lo, q[rt], acc[rt]);
        });
        f32x4_t o_a = dh ? acc[1] : acc[0], o_b = dh ? acc[2] : acc[3];
        const f32x4_t x_a = dh ? acc[0] : acc[1], x_b = dh ? acc[3] : acc[2];   // for the other half
        // ---- operands of the state's update: values over tokens ----
        u32x2_t vf[2][2];
        mm_lds_tr4<0, 16 * 128, 32 * 128, 48 * 128>(vf, vst + vt_rel);
        if (full) mm_barrier();  // query rows read, gate arrays written
        const bf16x8_t vv[2] = {mm_frag(vf[0][0], vf[0][1]), mm_frag(vf[1][0], vf[1][1])};
        // ---- weights of this wave's rows and keys: hi and lo, in the order the second product reads them ----
        const int row = 16 * v + c;
        const float rowc = GATED ? mm_lds<float>(sa + 256 + 4 * row) : 0.f, inc = GATED ? mm_lds<float>(sa + 512 + 4 * row) : 0.f;
        if (full) {
            *reinterpret_cast<f32x4_t*>(xst + (w * 2 * 64 + lane) * 16) = x_a;
            *reinterpret_cast<f32x4_t*>(xst + ((w * 2 + 1) * 64 + lane) * 16) = x_b;
            float p[8], dsum = 0.f;
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const int k0 = 32 * dh + 16 * u + 4 * g;
                f32x4_t ax = {0.f, 0.f, 0.f, 0.f};
                if constexpr (GATED) ax = mm_lds<f32x4_t>(sa + 4 * k0);
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float dw = !GATED ? dw_c[u][r] : k0 + r <= row ? __builtin_amdgcn_exp2f(rowc + ax[r]) * scale : 0.f;
                    p[4 * u + r] = s[u][r] * dw;
                    dsum += p[4 * u + r];
                }
            }
            bf16x8_t hi, lo;
            mm_split(p, hi, lo);
            const int chunk = ((4 * dh + g) ^ (c & 7)) << 4;
            *reinterpret_cast<bf16x8_t*>(pst + row * 128 + chunk) = hi;
            *reinterpret_cast<bf16x8_t*>(pst + 8192 + row * 128 + chunk) = lo;
            if constexpr (GATED) {
                nq = fmaf(nq, inc, dsum);
                nq += __shfl_xor(nq, 16, 64);
                nq += __shfl_xor(nq, 32, 64);
                if (g == 0) s_den[64 * dh + row] = nq;
            }
        }
        // ---- state of the next chunk ----
        bf16x8_t vhi[2], vlo[2];
        float wt[2][8];
#pragma unroll
        for (int sl = 0; sl < 2; ++sl) {
            f32x4_t w0 = {0.f, 0.f, 0.f, 0.f}, w1 = w0;
            if constexpr (GATED) {
                w0 = mm_lds<f32x4_t>(sa + 1024 + 128 * sl + 16 * g);
                w1 = mm_lds<f32x4_t>(sa + 1024 + 128 * sl + 64 + 16 * g);
            }
            float p[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                if constexpr (GATED) {
                    wt[sl][e] = e < 4 ? w0[e & 3] : w1[e & 3];
                } else {
                    wt[sl][e] = wt_c[sl][e];
                    if (last < 63) {  // the portion's last chunk
                        const int d = last - (32 * sl + 4 * g + (e & 3) + (e & 4) * 4);
                        wt[sl][e] = d >= 0 ? pw[d] : 0.f;
                    }
                }
                p[e] = wt[sl][e] * (float)vv[sl][e];
            }
            mm_split(p, vhi[sl], vlo[sl]);
        }
        constexpr int GI = HT >= 4 ? 4 : HT;   // row tiles of the state per group of reads
        static_for<HT / GI>([&](auto I4) {
            constexpr int i0 = GI * decltype(I4)::value;
            u32x2_t kf[GI][2][2];
            if constexpr (GI == 4) {
                const unsigned kb = lds_addr(kst) + (dh * HT / 4 + (i0 >> 2)) * 128;
                mm_lds_tr16<RB>(kf, kb + tr_rel[0], kb + tr_rel[1], kb + tr_rel[2], kb + tr_rel[3]);
            } else {
#pragma unroll
                for (int jj = 0; jj < GI; ++jj) mm_lds_tr4<0, 16 * RB, 32 * RB, 48 * RB>(kf[jj], kst + (dh ? tr_rel[2 + jj] : tr_rel[jj]));
            }
#pragma unroll
            for (int jj = 0; jj < GI; ++jj) S[i0 + jj] *= carry;
#pragma unroll
            for (int sl = 0; sl < 2; ++sl)
#pragma unroll
                for (int x = 0; x < 2; ++x)
#pragma unroll
                    for (int jj = 0; jj < GI; ++jj) S[i0 + jj] = mm_mfma(mm_frag(kf[jj][sl][0], kf[jj][sl][1]), x ? vlo[sl] : vhi[sl], S[i0 + jj]);
            if constexpr (!GATED) return;
            float nn = 0.f;   // n of the rows 16 (dh HT + i0 + v) + c
#pragma unroll
            for (int jj = 0; jj < GI; ++jj) {
                if (jj != v) continue;
#pragma unroll
                for (int sl = 0; sl < 2; ++sl) {
                    const bf16x8_t k = mm_frag(kf[jj][sl][0], kf[jj][sl][1]);
#pragma unroll
                    for (int e = 0; e < 8; ++e) nn = fmaf(wt[sl][e], (float)k[e], nn);
                }
            }
            nn += __shfl_xor(nn, 16, 64);
            nn += __shfl_xor(nn, 32, 64);
            nreg[i0 >> 2] = fmaf(carry, nreg[i0 >> 2], nn);
        });
        if (!full) continue;
        mm_barrier();
        // ---- output rows ----
        if (GATED && g == 0 && v < HT) {
#pragma unroll
            for (int i = 0; i < NR; ++i) s_n[16 * (dh * HT + 4 * i + v) + c] = nreg[i];  // read again behind the next barrier
        }
        const int ow = v + 4 * (1 - dh);       // the wave whose readout of these rows this one finishes
        o_a += mm_lds<f32x4_t>(xst + (ow * 2 * 64 + lane) * 16);
        o_b += mm_lds<f32x4_t>(xst + ((ow * 2 + 1) * 64 + lane) * 16);
        const int ta = 16 * rt_a + c, tb = 16 * rt_b + c;
        o_a *= GATED ? mm_lds<float>(sa + 512 + 4 * ta) : inc_a;
        o_b *= GATED ? mm_lds<float>(sa + 512 + 4 * tb) : inc_b;
        const unsigned ca = (g ^ (c & 7)) << 4, cb = ((4 + g) ^ (c & 7)) << 4;
        const bf16x8_t pa0 = mm_lds<bf16x8_t>(pst + ta * 128 + ca), pa1 = mm_lds<bf16x8_t>(pst + 8192 + ta * 128 + ca);   // tiles 0 and 1: keys 32 .. 63 are all in the future
        const bf16x8_t pb0 = mm_lds<bf16x8_t>(pst + tb * 128 + ca), pb1 = mm_lds<bf16x8_t>(pst + 8192 + tb * 128 + ca);
        const bf16x8_t pb2 = mm_lds<bf16x8_t>(pst + tb * 128 + cb), pb3 = mm_lds<bf16x8_t>(pst + 8192 + tb * 128 + cb);
        o_b = mm_mfma(vv[0], pb0, o_b);
        o_a = mm_mfma(vv[0], pa0, o_a);
        o_b = mm_mfma(vv[0], pb1, o_b);
        o_a = mm_mfma(vv[0], pa1, o_a);
        o_b = mm_mfma(vv[1], pb2, o_b);
        o_b = mm_mfma(vv[1], pb3, o_b);
        float ia = 1.0f, ib = 1.0f;
        if constexpr (GATED) {
            ia = __builtin_amdgcn_rcpf(fmaxf(fabsf(mm_lds<float>(sa + 1280 + 4 * ta) + mm_lds<float>(sa + 1536 + 4 * ta)), mm_lds<float>(sa + 768 + 4 * ta)) + 1e-6f);
            ib = __builtin_amdgcn_rcpf(fmaxf(fabsf(mm_lds<float>(sa + 1280 + 4 * tb) + mm_lds<float>(sa + 1536 + 4 * tb)), mm_lds<float>(sa + 768 + 4 * tb)) + 1e-6f);
        }
        rows_out[0] = u32x2_t{pack2bf(o_a[0] * ia, o_a[1] * ia), pack2bf(o_a[2] * ia, o_a[3] * ia)};
        rows_out[1] = u32x2_t{pack2bf(o_b[0] * ib, o_b[1] * ib), pack2bf(o_b[2] * ib, o_b[3] * ib)};
        m_in = mL;
    }
    store_rows(n_chunks - 1);
    const int64_t so = a.state_out[seq];
    if (!keeps || so < 0 || so >= a.n_state) return;
    const int64_t sout = so * a.H + h;
#pragma unroll
    for (int i = 0; i < HT; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = 16 * (dh * HT + i) + 4 * g + r;
            if (con && d < a.dimp) a.S[(sout * a.dimp + d) * a.vdimp + col] = S[i][r];
        }
    if (GATED && vt == 0) {
#pragma unroll
        for (int i = 0; i < NR; ++i) {
            const int d = 16 * (dh * HT + 4 * i + v) + c;
            if (g == 0 && v < HT && d < a.dimp) a.n[sout * a.dimp + d] = nreg[i];
        }
        if (tid == 0) a.m[sout] = m_in * (1.0f / MM_LOG2E);
    }
}

// y = o / rms(o) . norm . sigmoid(g) per (row, head); lph lanes (a power of two) per head, eight columns per lane and round
struct OutArgs {
    const bf16_t* o;
    int64_t ldo;
    const bf16_t* g;
    int64_t ldg;
    const float* norm;
    bf16_t* y;
    int64_t ldy, T;
    int H, vdim, vdimp, lph;
    float eps;
};
__global__ __launch_bounds__(256) void memory_output_kernel(const OutArgs a) {
    const int64_t item = ((int64_t)blockIdx.x * 256 + threadIdx.x) / a.lph;
    const int l = threadIdx.x & (a.lph - 1);
    const bool on = item < a.T * a.H;
    const int64_t r = on ? item / a.H : 0;
    const int h = on ? (int)(item - r * a.H) : 0;
    const bf16_t* o = a.o + r * a.ldo + (int64_t)h * a.vdimp;
    float sq = 0.f;
    for (int c = l * 8; c < a.vdimp; c += a.lph * 8) {
        const u32x4_t u = *reinterpret_cast<const u32x4_t*>(o + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) sq += bflo(u[e]) * bflo(u[e]) + bfhi(u[e]) * bfhi(u[e]);
    }
    for (int x = 1; x < a.lph; x <<= 1) sq += __shfl_xor(sq, x, 64);
    if (!on) return;
    const float inv = 1.0f / sqrtf(sq / (float)a.vdim + a.eps);
    const bf16_t* g = a.g + r * a.ldg + (int64_t)h * a.vdimp;
    const float* nm = a.norm + (int64_t)h * a.vdimp;
    bf16_t* y = a.y + r * a.ldy + (int64_t)h * a.vdimp;
    for (int c = l * 8; c < a.vdimp; c += a.lph * 8) {
        const u32x4_t u = *reinterpret_cast<const u32x4_t*>(o + c), gv = *reinterpret_cast<const u32x4_t*>(g + c);
        u32x4_t out;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const float g0 = bflo(gv[e]), g1 = bfhi(gv[e]);
            out[e] = pack2bf(bflo(u[e]) * inv * nm[c + 2 * e] * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-MM_LOG2E * g0)),
                             bfhi(u[e]) * inv * nm[c + 2 * e + 1] * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-MM_LOG2E * g1)));
        }
        *reinterpret_cast<u32x4_t*>(y + c) = out;
    }
}

// y = o / rms(o) . norm . gate over whole rows, one row per workgroup, eight columns per thread and round (two rounds stay in registers); n: true
// number of columns (padding columns of o are zeros)
template <typename O, typename Y>
__global__ __launch_bounds__(1024) void row_norm_gate_kernel(const O* __restrict__ o, int64_t ldo, const Y* __restrict__ gate, int64_t ldg, const float* __restrict__ norm,
                                                             Y* __restrict__ y, int64_t ldy, int n, int np, float eps) {
    __shared__ float s_red[16];
    const int tid = threadIdx.x, nt = blockDim.x;
    const int64_t r = blockIdx.x;
    f32x4_t u[2][2], g[2][2], w[2][2];
    float sq = 0.f;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int c = (tid + i * nt) * 8;
#pragma unroll
        for (int hf = 0; hf < 2; ++hf) {
            u[i][hf] = g[i][hf] = w[i][hf] = f32x4_t{0.f, 0.f, 0.f, 0.f};
            if (c < np) {
                u[i][hf] = mm_ld4<O>(o, r * ldo + c + 4 * hf);
                g[i][hf] = mm_ld4<Y>(gate, r * ldg + c + 4 * hf);
                w[i][hf] = *reinterpret_cast<const f32x4_t*>(norm + c + 4 * hf);
            }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) sq += u[i][0][e] * u[i][0][e] + u[i][1][e] * u[i][1][e];
    }
    for (int c = (tid + 2 * nt) * 8; c < np; c += nt * 8) {
        const f32x4_t a = mm_ld4<O>(o, r * ldo + c), b = mm_ld4<O>(o, r * ldo + c + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) sq += a[e] * a[e] + b[e] * b[e];
    }
    sq = wave_sum(sq);
    if ((tid & 63) == 0) s_red[tid >> 6] = sq;
    __syncthreads();
    sq = 0.f;
    for (int i = 0; i < nt / 64; ++i) sq += s_red[i];
    const float inv = 1.0f / sqrtf(sq / (float)n + eps);
    auto put = [&](int c, f32x4_t v, const f32x4_t& gv, const f32x4_t& wv) {
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = v[e] * inv * wv[e] * gv[e];
        if constexpr (sizeof(Y) == 4) *reinterpret_cast<f32x4_t*>(y + r * ldy + c) = v;
        else *reinterpret_cast<u32x2_t*>(y + r * ldy + c) = u32x2_t{pack2bf(v[0], v[1]), pack2bf(v[2], v[3])};
    };
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int c = (tid + i * nt) * 8;
        if (c < np) {
            put(c, u[i][0], g[i][0], w[i][0]);
            put(c + 4, u[i][1], g[i][1], w[i][1]);
        }
    }
    for (int c = (tid + 2 * nt) * 8; c < np; c += nt * 8)
#pragma unroll
        for (int hf = 0; hf < 2; ++hf)
            put(c + 4 * hf, mm_ld4<O>(o, r * ldo + c + 4 * hf), mm_ld4<Y>(gate, r * ldg + c + 4 * hf), *reinterpret_cast<const f32x4_t*>(norm + c + 4 * hf));
}

template <typename T, int KD, int NW>
int launch_rec(const RecArgs& a, hipStream_t st) {
    if constexpr (NW == 1) {
        if (a.decay) {
            hipLaunchKernelGGL((memory_recurrent_kernel<T, KD, 1, false>), dim3((unsigned)(a.seqs * a.H), (unsigned)((a.vdimp + 63) / 64)), dim3(256), 0, st, a);
            GLM_CHECK_LAUNCH("glm_linear_recurrent");
            return GLM_OK;
        }
    }
    hipLaunchKernelGGL((memory_recurrent_kernel<T, KD, NW, true>), dim3((unsigned)(a.seqs * a.H)), dim3(256 * NW), 0, st, a);
    GLM_CHECK_LAUNCH("glm_memory_recurrent");
    return GLM_OK;
}
template <typename T, int KD>
int launch_rec_v(const RecArgs& a, hipStream_t st) {
    if (a.vdimp <= 64 || a.decay) return launch_rec<T, KD, 1>(a, st);
    if (a.vdimp <= 128) return launch_rec<T, KD, 2>(a, st);
    return launch_rec<T, KD, 4>(a, st);
}
template <typename T>
int run_rec(const RecArgs& a, hipStream_t st) {
    if (a.dimp <= 256 && (a.vdimp <= 256 || (a.decay && a.vdimp <= 65535 * 64))) {
        if (a.dimp <= 64) return launch_rec_v<T, 4>(a, st);
        if (a.dimp <= 128) return launch_rec_v<T, 8>(a, st);
        return launch_rec_v<T, 16>(a, st);
    }
    const size_t lds = (size_t)(2 * a.dimp + a.vdimp) * 4;
    GLM_CHECK_ARG(lds <= 48 * 1024, GLM_ERR_UNSUPPORTED, "glm_memory_recurrent: head sizes %d + %d", a.dimp, a.vdimp);
    if (a.decay) hipLaunchKernelGGL((memory_recurrent_any_kernel<T, false>), dim3((unsigned)(a.seqs * a.H)), dim3(256), lds, st, a);
    else hipLaunchKernelGGL((memory_recurrent_any_kernel<T, true>), dim3((unsigned)(a.seqs * a.H)), dim3(256), lds, st, a);
    GLM_CHECK_LAUNCH("glm_memory_recurrent");
    return GLM_OK;
}

template <int D, bool GATED>
int launch_chunk(const ChunkArgs& a, int seqs, int nseg, hipStream_t st) {
    constexpr int QT = 64 * D * 2, STAGE = 2 * QT + 8192 + 1024;
    constexpr int LDS = (D <= 128 ? 3 : 2) * STAGE + (QT >= 16384 ? 0 : 16384) + (QT >= 32768 ? 0 : 16384) + 7 * 256 + D * 4;
    static_assert(LDS <= 160 * 1024, "LDS of a CU");
    auto kern = memory_chunkwise_kernel<D, GATED>;
    GLM_SET_MAX_LDS(kern, LDS, "glm_memory_chunkwise");
    hipLaunchKernelGGL(kern, dim3((unsigned)(seqs * a.H * a.vtiles), (unsigned)nseg), dim3(512), LDS, st, a);
    GLM_CHECK_LAUNCH("glm_memory_chunkwise");
    return GLM_OK;
}

}  // namespace

extern "C" int glm_memory_recurrent(const void* x, int64_t ldx, int64_t k_off, int64_t v_off, int64_t g_off, const void* hrow, int64_t ldh, const void* wif, int64_t ldw, int wk,
                                    const float* bif, const float* norm, void* y, int64_t ldy, float* S, float* n, float* m, int64_t n_state, const int32_t* pos,
                                    const int32_t* q_start, const int32_t* state_in, const int32_t* state_out, int seqs, int H, int dim, int dimp, int vdim, int vdimp, float cap, float eps,
                                    int f32, glm_stream_t stream) {
    GLM_CHECK_ARG(x && hrow && wif && bif && norm && y && S && n && m && pos && q_start && state_in && state_out, GLM_ERR_INVALID, "glm_memory_recurrent: null pointer");
    GLM_CHECK_ARG(seqs >= 0 && H > 0 && dim > 0 && dimp >= dim && dimp % 8 == 0 && vdim > 0 && vdimp >= vdim && vdimp % 8 == 0 && wk > 0 && wk % 8 == 0 && ldh >= wk && ldw >= wk && n_state > 0 &&
                      k_off >= (int64_t)H * dimp && ldx >= k_off + (int64_t)H * dimp && ldx >= v_off + (int64_t)H * vdimp && ldx >= g_off + (int64_t)H * vdimp && ldy >= (int64_t)H * vdimp &&
                      ldx % 8 == 0 && k_off % 8 == 0 && v_off % 8 == 0 && g_off % 8 == 0 && ldh % 8 == 0 && ldw % 8 == 0 && cap > 0.f && (int64_t)seqs * H < (1ll << 31) &&
                      glm_aligned16(x) && glm_aligned16(hrow) && glm_aligned16(wif) && glm_aligned16(S), GLM_ERR_INVALID,
                  "glm_memory_recurrent: bad shape H=%d dim=%d vdim=%d ldx=%ld", H, dim, vdim, (long)ldx);
    if (seqs == 0) return GLM_OK;
    RecArgs a = {x, ldx, k_off, v_off, g_off, hrow, ldh, wif, ldw, wk, bif, norm, y, ldy, S, n, m, n_state, pos, q_start, state_in, state_out, seqs, H, dim, dimp, vdim, vdimp, cap, eps, nullptr};
    return f32 ? run_rec<float>(a, glm_s(stream)) : run_rec<bf16_t>(a, glm_s(stream));
}

extern "C" int glm_memory_gates(const void* hrow, int64_t ldh, const void* wif, int64_t ldw, int wk, const float* bif, float* gates, int64_t rows, const int32_t* q_start,
                                const int32_t* tile_seq, const int32_t* tile_off, int n_tiles, int H, float cap, glm_stream_t stream) {
    GLM_CHECK_ARG(hrow && wif && bif && gates && q_start && tile_seq && tile_off, GLM_ERR_INVALID, "glm_memory_gates: null pointer");
    GLM_CHECK_ARG(rows >= 0 && H > 0 && H <= 65535 * 16 && n_tiles >= 0 && n_tiles < (1 << 30) && wk > 0 && wk % 8 == 0 && ldh >= wk && ldw >= wk && ldh % 8 == 0 && ldw % 8 == 0 && cap > 0.f &&
                      glm_aligned16(hrow) && glm_aligned16(wif), GLM_ERR_INVALID, "glm_memory_gates: bad shape rows=%ld H=%d wk=%d", (long)rows, H, wk);
    if (n_tiles == 0) return GLM_OK;
    GateArgs a = {(const bf16_t*)hrow, ldh, (const bf16_t*)wif, ldw, wk, bif, gates, rows, q_start, tile_seq, tile_off, H, cap};
    hipLaunchKernelGGL(memory_gates_kernel, dim3((unsigned)(2 * n_tiles), (unsigned)((H + 15) / 16)), dim3(256), 0, glm_s(stream), a);
    GLM_CHECK_LAUNCH("glm_memory_gates");
    return GLM_OK;
}

extern "C" int glm_memory_chunkwise(const void* x, int64_t ldx, int64_t k_off, int64_t v_off, const float* gates, int64_t rows, void* o, int64_t ldo, float* S, float* n, float* m,
                                    int64_t n_state, const int32_t* pos, const int32_t* q_start, const int32_t* state_in, const int32_t* state_out, int seqs, int H, int dim, int dimp,
                                    int vdimp, glm_stream_t stream) {
    GLM_CHECK_ARG(x && gates && o && S && n && m && pos && q_start && state_in && state_out, GLM_ERR_INVALID, "glm_memory_chunkwise: null pointer");
    GLM_CHECK_ARG(seqs >= 0 && rows >= 0 && H > 0 && dim > 0 && dimp >= dim && dimp % 8 == 0 && vdimp > 0 && vdimp % 8 == 0 && n_state > 0 && k_off >= (int64_t)H * dimp &&
                      ldx >= k_off + (int64_t)H * dimp && ldx >= v_off + (int64_t)H * vdimp && ldo >= (int64_t)H * vdimp && ldx % 8 == 0 && k_off % 8 == 0 && v_off % 8 == 0 && ldo % 4 == 0 && ldx < (1 << 24) &&
                      glm_aligned16(x) && (((uintptr_t)o) & 7) == 0, GLM_ERR_INVALID, "glm_memory_chunkwise: bad shape H=%d dim=%d vdimp=%d ldx=%ld", H, dim, vdimp, (long)ldx);
    GLM_CHECK_ARG(dimp <= 256, GLM_ERR_UNSUPPORTED, "glm_memory_chunkwise: key size %d", dimp);
    if (seqs == 0) return GLM_OK;
    ChunkArgs a = {(const bf16_t*)x, ldx, k_off, v_off, gates, rows, (bf16_t*)o, ldo, S, n, m, n_state, pos, q_start, state_in, state_out, H, dim, dimp, vdimp, (vdimp + 63) / 64, nullptr, {}};
    GLM_CHECK_ARG((int64_t)seqs * H * a.vtiles < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_memory_chunkwise: grid too large");
    hipStream_t st = glm_s(stream);
    if (dimp <= 64) return launch_chunk<64, true>(a, seqs, 1, st);
    if (dimp <= 128) return launch_chunk<128, true>(a, seqs, 1, st);
    return launch_chunk<256, true>(a, seqs, 1, st);
}

extern "C" int glm_memory_output(const void* o, int64_t ldo, const void* g, int64_t ldg, const float* norm, void* y, int64_t ldy, int64_t T, int H, int vdim, int vdimp, float eps,
                                 glm_stream_t stream) {
    GLM_CHECK_ARG(o && g && norm && y && T >= 0 && H > 0 && vdim > 0 && vdimp >= vdim && vdimp % 8 == 0 && ldo >= (int64_t)H * vdimp && ldg >= (int64_t)H * vdimp && ldy >= (int64_t)H * vdimp &&
                      ldo % 8 == 0 && ldg % 8 == 0 && ldy % 8 == 0 && glm_aligned16(o) && glm_aligned16(g) && glm_aligned16(y), GLM_ERR_INVALID,
                  "glm_memory_output: bad shape T=%ld H=%d vdim=%d", (long)T, H, vdim);
    if (T == 0) return GLM_OK;
    int lph = 1;
    while (lph < 64 && lph * 8 < vdimp) lph *= 2;
    OutArgs a = {(const bf16_t*)o, ldo, (const bf16_t*)g, ldg, norm, (bf16_t*)y, ldy, T, H, vdim, vdimp, lph, eps};
    const int64_t blocks = (T * H * lph + 255) / 256;
    GLM_CHECK_ARG(blocks < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_memory_output: too many rows");
    hipLaunchKernelGGL(memory_output_kernel, dim3((unsigned)blocks), dim3(256), 0, glm_s(stream), a);
    GLM_CHECK_LAUNCH("glm_memory_output");
    return GLM_OK;
}

extern "C" int glm_linear_recurrent(const void* x, int64_t ldx, int64_t k_off, int64_t v_off, const float* decay, float* o, int64_t ldo, float* S, int64_t n_state, const int32_t* pos,
                                    const int32_t* q_start, const int32_t* state_in, const int32_t* state_out, int seqs, int H, int dimp, int vdimp, int f32, glm_stream_t stream) {
    GLM_CHECK_ARG(x && decay && o && S && pos && q_start && state_in && state_out, GLM_ERR_INVALID, "glm_linear_recurrent: null pointer");
    GLM_CHECK_ARG(seqs >= 0 && H > 0 && dimp > 0 && dimp % 8 == 0 && vdimp > 0 && vdimp % 8 == 0 && n_state > 0 && k_off >= (int64_t)H * dimp && ldx >= k_off + (int64_t)H * dimp &&
                      ldx >= v_off + (int64_t)H * vdimp && ldo >= (int64_t)H * vdimp && ldx % 8 == 0 && k_off % 8 == 0 && v_off % 8 == 0 && (int64_t)seqs * H < (1ll << 31) &&
                      glm_aligned16(x) && glm_aligned16(S), GLM_ERR_INVALID, "glm_linear_recurrent: bad shape H=%d dimp=%d vdimp=%d ldx=%ld", H, dimp, vdimp, (long)ldx);
    if (seqs == 0) return GLM_OK;
    RecArgs a = {};
    a.x = x; a.ldx = ldx; a.k_off = k_off; a.v_off = v_off; a.y = o; a.ldy = ldo; a.S = S; a.n_state = n_state; a.pos = pos; a.q_start = q_start; a.state_in = state_in;
    a.state_out = state_out; a.seqs = seqs; a.H = H; a.dim = a.dimp = dimp; a.vdim = a.vdimp = vdimp; a.decay = decay;
    return f32 ? run_rec<float>(a, glm_s(stream)) : run_rec<bf16_t>(a, glm_s(stream));
}

extern "C" int glm_linear_chunkwise(const void* x, int64_t ldx, int64_t k_off, int64_t v_off, const float* powers, int64_t rows, void* o, int64_t ldo, float* S, int64_t n_state, const int32_t* pos,
                                    const int32_t* q_start, const int32_t* state_in, const int32_t* state_out, int seqs, int H, int dimp, int vdimp, glm_stream_t stream) {
    GLM_CHECK_ARG(x && powers && o && S && pos && q_start && state_in && state_out, GLM_ERR_INVALID, "glm_linear_chunkwise: null pointer");
    GLM_CHECK_ARG(seqs >= 0 && rows >= 0 && H > 0 && dimp > 0 && dimp % 8 == 0 && vdimp > 0 && vdimp % 8 == 0 && n_state > 0 && k_off >= (int64_t)H * dimp && ldx >= k_off + (int64_t)H * dimp &&
                      ldx >= v_off + (int64_t)H * vdimp && ldo >= (int64_t)H * vdimp && ldx % 8 == 0 && k_off % 8 == 0 && v_off % 8 == 0 && ldo % 4 == 0 && ldx < (1 << 24) &&
                      glm_aligned16(x) && (((uintptr_t)o) & 7) == 0, GLM_ERR_INVALID, "glm_linear_chunkwise: bad shape H=%d dimp=%d vdimp=%d ldx=%ld", H, dimp, vdimp, (long)ldx);
    GLM_CHECK_ARG(dimp <= 256, GLM_ERR_UNSUPPORTED, "glm_linear_chunkwise: key size %d", dimp);
    if (seqs == 0) return GLM_OK;
    // segments as long as the chip has room: a chunk that only moves the state costs about a third of a whole one, and all segments shall
    // take the same time, c (t_(s+1) - t_s) + c / 3 t_s
    const int64_t wgs = (int64_t)seqs * H * ((vdimp + 63) / 64);
    int nseg = (int)(256 / (wgs > 0 ? wgs : 1)), most = (int)(rows / seqs / 256);
    nseg = nseg > most ? most : nseg;
    nseg = nseg > MM_MAX_SEG ? MM_MAX_SEG : nseg < 1 ? 1 : nseg;
    ChunkArgs a = {(const bf16_t*)x, ldx, k_off, v_off, nullptr, 0, (bf16_t*)o, ldo, S, nullptr, nullptr, n_state, pos, q_start, state_in, state_out, H, dimp, dimp, vdimp, (vdimp + 63) / 64, powers, {}};
    float left = 1.0f, all = 1.0f;
    for (int i = 0; i < nseg; ++i) all *= 2.0f / 3;
    for (int i = 0; i <= nseg; ++i, left *= 2.0f / 3) a.seg[i] = i == nseg ? 1.0f : (1.0f - left) / (1.0f - all);
    GLM_CHECK_ARG((int64_t)seqs * H * a.vtiles < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_linear_chunkwise: grid too large");
    hipStream_t st = glm_s(stream);
    if (dimp <= 64) return launch_chunk<64, false>(a, seqs, nseg, st);
    if (dimp <= 128) return launch_chunk<128, false>(a, seqs, nseg, st);
    return launch_chunk<256, false>(a, seqs, nseg, st);
}

extern "C" int glm_row_norm_gate(const void* o, int64_t ldo, int o_f32, const void* gate, int64_t ldg, const float* norm, void* y, int64_t ldy, int64_t T, int n, int np, float eps,
                                 int act_f32, glm_stream_t stream) {
    GLM_CHECK_ARG(o && gate && norm && y && T >= 0 && n > 0 && np >= n && np % 8 == 0 && ldo >= np && ldg >= np && ldy >= np && ldo % 8 == 0 && ldg % 8 == 0 && ldy % 8 == 0 &&
                      glm_aligned16(o) && glm_aligned16(gate) && glm_aligned16(norm) && glm_aligned16(y) && (o_f32 || !act_f32), GLM_ERR_INVALID,
                  "glm_row_norm_gate: bad shape T=%ld n=%d np=%d", (long)T, n, np);
    GLM_CHECK_ARG(T < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_row_norm_gate: too many rows");
    if (T == 0) return GLM_OK;
    const dim3 grid((unsigned)T);
    int nt = (np / 8 + 63) / 64 * 64;   // (many rows: half as many threads, two rounds each)
    if (T > 1024 && nt > 64) nt = (nt / 2 + 63) / 64 * 64;
    nt = nt > 1024 ? 1024 : nt;
    hipStream_t st = glm_s(stream);
    if (act_f32) hipLaunchKernelGGL((row_norm_gate_kernel<float, float>), grid, dim3(nt), 0, st, (const float*)o, ldo, (const float*)gate, ldg, norm, (float*)y, ldy, n, np, eps);
    else if (o_f32) hipLaunchKernelGGL((row_norm_gate_kernel<float, bf16_t>), grid, dim3(nt), 0, st, (const float*)o, ldo, (const bf16_t*)gate, ldg, norm, (bf16_t*)y, ldy, n, np, eps);
    else hipLaunchKernelGGL((row_norm_gate_kernel<bf16_t, bf16_t>), grid, dim3(nt), 0, st, (const bf16_t*)o, ldo, (const bf16_t*)gate, ldg, norm, (bf16_t*)y, ldy, n, np, eps);
    GLM_CHECK_LAUNCH("glm_row_norm_gate");
    return GLM_OK;
}
