// group_attn.hip — causal attention with grouped heads (H query heads over G key / value heads) read from paged caches, with
// what a design may add to it, each a parameter: a sliding window or chunks (a token sees its own chunk only, chunks counted from
// position 0 of the sequence), a distance bias per head (slope_h * (i - j) is taken off the scaled score), a learned sink per
// head (mass exp(sink) in the denominator, without key or value), a soft cap on the scores, a gate on the output (per head or per column).
// Head sizes of keys and values are independent.  gfx950 only.
//
// Beside the softmax there are two more forms.  Two maps per head (differential attention): a head has two queries and a key / value head
// two keys, side by side in a row, over the same values; what comes out is norm(o_1 - lam o_2), the norm over the head's columns.
// Sigmoid weights: a visible key counts with sigmoid(score + bias_h), nothing is normalised; the keys are the values, a key's score
// multiplied by a number of its own (group_rows.hip: 1 / rms), so one cache and one LDS tile serve both products.
//
//   group_kv_store       rows of a projection -> the pages of both caches, [block][G][tokens of a block][head size]
//   group_attn_prefill   long portions: 128 query rows of one head, or 64 of two heads of a group, per workgroup
//   group_attn_decode    decoded tokens and short portions: 16 (token, head) rows of one key / value head per workgroup, the keys
//                        split over the waves and over workgroups (glm_attn_merge adds the splits up)
//   group_attn_plain     any head size, bf16 or fp32: one (token, head) per workgroup, vector FMAs, every step in fp32
//
// Keys and values of the step's own tokens are in the cache like all others (group_kv_store), so a portion of a prompt, a decoded
// token and a layer that borrows another layer's cache are the same thing.  The decode form may also take them from the
// projection's rows and store them itself, which saves a decode step the launch in front.
//
// Roofline: MFMA for prefill, HBM for decode (the visible keys and values, read once).  S^T = K . Q^T, fp32 online softmax per lane
// column in log2 units (the distance bias, divided by the scale, is what the score products are added to), O^T += V^T . P^T straight from
// registers.  Tiles come in by LDS-DMA, double-buffered; keys behind
// the last visible one are fetched from a page of zeros (unused cache memory may hold NaNs).  The running maximum is raised only when
// a score exceeds it by more than 2^8 (the sums stay exact: the reference point cancels).
#include "common.h"
#include "attn_lds.h"

namespace {

constexpr float GA_LOG2E = 1.4426950408889634f;
__device__ const u32x4_t ga_zero_page[4] = {};

struct GroupArgs {
    const void* q;        // [rows, ldq], head h at h*dk
    int64_t ldq;
    const void *kc, *vc;  // caches
    int64_t n_blocks;
    int bs, log2_bs;      // tokens per block (log2_bs < 0: not a power of two)
    const int32_t* bt;    // [sequences, bt_stride]
    int64_t bt_stride;
    const int32_t *pos, *seq_of;  // of the rows of q
    const int32_t *q_start, *tile_a, *tile_b;
    int seq0, n_tiles, H, G, dk, dv, window, chunk, nsplit, pair;  // pair: prefill tiles of 64 rows of two heads
    float scale;
    const float *slope, *sink;  // [H] or nullptr
    float cap;                  // soft cap on the scaled score; 0: none
    int maps, sigmoid;          // maps 2: dk holds two keys, dk / 2 columns each
    const float* bias;          // sigmoid: [H]
    const float* kscale;        // [n_blocks * bs] factor of a key's scores (then kc == vc), or nullptr
    float lam, post, eps;       // maps 2: o = post (o_1 - lam o_2) / rms, over vn columns
    int vn;
    const void* gate;           // [rows, ldg]: factor of head h at h or, gate_cols, of column d at h*dv + d; or nullptr
    int64_t ldg;
    int gate_cols;
    const void *knew, *vnew;    // decode: keys / values of the step's own rows, row r at r*ldkv, head g at g*dk / g*dv, or nullptr
    int64_t ldkv;
    const int32_t* slots;       // decode with knew: cache rows they are stored to
    void* out;            // [rows, ldo], head h at h*dv
    int64_t ldo;
    float *part_o, *part_ml;    // nsplit > 1 or two maps: [rows*H*maps][nsplit][dv], [rows*H*maps][nsplit][2]
    int64_t rows;
};

// first position that position p sees
__device__ __forceinline__ int ga_first(const GroupArgs& a, int p) {
    int lo = 0;
    if (a.window > 0) lo = max(lo, p - a.window + 1);
    if (a.chunk > 0) lo = max(lo, p - p % a.chunk);
    return lo;
}
__device__ __forceinline__ int ga_block(const GroupArgs& a, int j) { return a.log2_bs >= 0 ? j >> a.log2_bs : j / a.bs; }
// row of a cache (in units of the head size) of key position j with block id blk, head g
__device__ __forceinline__ int64_t ga_row(const GroupArgs& a, int blk, int j, int g) { return ((int64_t)blk * a.G + g) * a.bs + (j - ga_block(a, j) * a.bs); }
__device__ __forceinline__ int ga_uniform(int v) { return __builtin_amdgcn_readfirstlane(v); }
__device__ __forceinline__ bool ga_ok(const GroupArgs& a, int blk) { return blk >= 0 && blk < a.n_blocks; }
// four columns of a head's gate from column d on
__device__ __forceinline__ f32x4_t ga_gate(const GroupArgs& a, int64_t row, int h, int d) {
    const bf16_t* g = reinterpret_cast<const bf16_t*>(a.gate) + row * a.ldg;
    if (!a.gate_cols) {
        const float f = bf2f(g[h]);
        return f32x4_t{f, f, f, f};
    }
    const u32x2_t u = *reinterpret_cast<const u32x2_t*>(g + (int64_t)h * a.dv + d);
    return f32x4_t{bflo(u[0]), bfhi(u[0]), bflo(u[1]), bfhi(u[1])};
}
// forms of the tiled kernels
// (GA_TWO_MAPS: the scores have a soft cap that 2^score fits under as it is; GA_TWO_MAPS_ANY: any cap, or none)
enum : int { GA_SOFTMAX = 0, GA_TWO_MAPS = 1, GA_SIGMOID_KV = 2, GA_TWO_MAPS_ANY = 3 };
constexpr float GA_CAP_FITS = 55.f;  // cap log2(e) <= 80: the sums of 2^score stay far inside fp32 whatever their number
__host__ __device__ constexpr bool ga_two(int form) { return form == GA_TWO_MAPS || form == GA_TWO_MAPS_ANY; }

// ---------------------------------------------------------------------------------------------------------------------------
struct StoreArgs {
    const char* src;      // row r at r*ld bytes; keys at k_off, values at v_off (bytes)
    int64_t ld, k_off, v_off;
    const int32_t* slots; // [T] block * bs + place, < 0: no cache row
    char *kc, *vc;
    int64_t T, n_slots;
    int G, bs, ku, vu;    // 16-byte units of a key / value head
};
__global__ __launch_bounds__(256) void group_kv_store_kernel(const StoreArgs a) {
    const int per = a.G * (a.ku + a.vu);
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int64_t r = i / per;
    if (r >= a.T) return;
    int u = (int)(i - r * per);
    const int64_t slot = a.slots[r];
    if (slot < 0 || slot >= a.n_slots) return;
    const bool val = u >= a.G * a.ku;
    if (val) u -= a.G * a.ku;
    const int w = val ? a.vu : a.ku, g = u / w, c = u - g * w;
    const u32x4_t x = *reinterpret_cast<const u32x4_t*>(a.src + r * a.ld + (val ? a.v_off : a.k_off) + (int64_t)u * 16);
    char* dst = val ? a.vc : a.kc;
    *reinterpret_cast<u32x4_t*>(dst + (((slot / a.bs * a.G + g) * a.bs + slot % a.bs) * w + c) * 16) = x;
}

// ---------------------------------------------------------------------------------------------------------------------------
// the two products of a 32-key slab and the softmax between them, for NT tiles of 16 query rows (lane c holds row c of each)
// (two maps: of two tiles, tile t holds map t's rows of the queries and meets the keys' half t; in one tile a row's queries are
// zeros in the other map's half)
template <int DK, int DV, int NT, int F>
struct Slab {
    static constexpr bool SPLIT = ga_two(F) && NT == 2;
    static constexpr int KS = DK / 32, KQ = SPLIT ? KS / 2 : KS, VT = DV / 16, KB = DK * 2, VB = DV * 2;
    static constexpr bool VEARLY = DK + DV <= 256;                    // V fragments requested in front of the score products
    static constexpr int KG = KS < 4 ? KS : 4, VG = VEARLY ? VT : 4;  // fragments per request group
    u32x4_t qf[NT][KQ];
    f32x4_t acc[NT][VT];
    float m_run[NT], l_run[NT], slope[NT];                // slope: per key, in units of the unscaled score; sigmoid: the bias in log2 units
    float cap_in, cap_out;                                // soft cap: exponent per unit of score, cap in log2 units (0: none)
    float cap_lim, ca0, ca1, ca2, ca3;                    // scores up to cap_lim: odd polynomial
    int rp[NT], rlo[NT];                                  // position of the lane's row and the first one it sees; rp < 0: no row
    int any_lo[NT], any_hi[NT], full_lo[NT], full_hi[NT]; // keys that some row / every row of the tile sees
    unsigned k_rel[2], v_rel[4];

    __device__ __forceinline__ void init(int lane) {
        const int c = lane & 15, g = lane >> 4;
        // K row c, chunk 4 i + g (its low three bits depend on the parity of i only); V row 4 g + qq
#pragma unroll
        for (int e = 0; e < 2; ++e) k_rel[e] = c * KB + (((4 * e + g) ^ attn_swz(c)) << 4);
        const int qq = (lane >> 2) & 3, pp = lane & 3, vr = 4 * g + qq;
#pragma unroll
        for (int e = 0; e < 4; ++e) v_rel[e] = vr * VB + (((2 * e + (pp >> 1)) ^ attn_swz(vr)) << 4) + ((pp & 1) << 3);
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            m_run[t] = -INFINITY;
            l_run[t] = 0.f;
#pragma unroll
            for (int d = 0; d < VT; ++d) acc[t][d] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        }
    }
    // cap tanh(s / cap) in log2 units, by tanh y = 1 - 2 / (1 + e^(2 y))
    __device__ __forceinline__ void cap_exact(f32x4_t (&s)[2]) const {
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
            for (int r = 0; r < 4; ++r) s[kt][r] = fmaf(-2.f * cap_out, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(s[kt][r] * cap_in)), cap_out);
    }
    // all tiles: up to a fifth of the cap tanh is its odd polynomial of degree 7 (the next term is below 2e-8 of the cap)
    __device__ __forceinline__ void cap_scores(f32x4_t (&s)[NT][2]) const {
        float big = 0.f;
#pragma unroll
        for (int t = 0; t < NT; ++t)
#pragma unroll
            for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                for (int r = 0; r < 4; ++r) big = fmaxf(big, fabsf(s[t][kt][r]));
        if (__any(big > cap_lim)) {
#pragma unroll
            for (int t = 0; t < NT; ++t) cap_exact(s[t]);
            return;
        }
#pragma unroll
        for (int t = 0; t < NT; ++t)
#pragma unroll
            for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float u = s[t][kt][r] * s[t][kt][r];
                    s[t][kt][r] *= fmaf(fmaf(fmaf(ca3, u, ca2), u, ca1), u, ca0);
                }
    }
    // kst, vst: LDS addresses of the slab's first key row and value row; j0: position of its first key
    // kst, vst, fst: ... and of the keys' factors (sigmoid form)
    __device__ __forceinline__ void run(unsigned kst, unsigned vst, int j0, int g, float sc, unsigned fst) {
        bool live[NT], some = false;
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            live[t] = j0 <= any_hi[t] && j0 + 31 >= any_lo[t];
            some = some || live[t];
        }
        if (!some) return;
        u32x2_t vf[VG][2];
        auto read_v = [&](auto D0) {
            static_for<VG>([&](auto I) {
                constexpr int i = decltype(I)::value, d = decltype(D0)::value + i;
                lds_read_tr16_b64<(d >> 2) * 128>(vf[i][0], vst + v_rel[d & 3]);
                lds_read_tr16_b64<(d >> 2) * 128 + 16 * VB>(vf[i][1], vst + v_rel[d & 3]);
            });
        };
        f32x4_t s[NT][2];  // starts from the distance bias: the products are added to it
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const float b0 = F == GA_SOFTMAX ? slope[t] * (float)(j0 + 4 * g - rp[t]) : 0.f;
#pragma unroll
            for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                for (int r = 0; r < 4; ++r) s[t][kt][r] = F == GA_SOFTMAX ? fmaf(slope[t], (float)(16 * kt + r), b0) : 0.f;
        }
        u32x4_t ks[2];
        if constexpr (F == GA_SIGMOID_KV) {  // (in front of the K fragments: in when they are)
            lds_read_b128<0>(ks[0], fst + 16 * g);
            lds_read_b128<64>(ks[1], fst + 16 * g);
        }
        static_for<(KS + KG - 1) / KG>([&](auto GI) {
            constexpr int k0 = decltype(GI)::value * KG, kn = KS - k0 < KG ? KS - k0 : KG;
            constexpr bool last = k0 + KG >= KS;
            u32x4_t kf[2][KG];
            static_for<kn>([&](auto I) {
                constexpr int i = k0 + decltype(I)::value;
                lds_read_b128<(i >> 1) * 128>(kf[0][i - k0], kst + k_rel[i & 1]);
                lds_read_b128<(i >> 1) * 128 + 16 * KB>(kf[1][i - k0], kst + k_rel[i & 1]);
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
                    for (int t = 0; t < NT; ++t) {
                        if (SPLIT && (k0 + i) / KQ != t) continue;
                        s[t][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kf[kt][i]), __builtin_bit_cast(bf16x8_t, qf[t][(k0 + i) % KQ]), s[t][kt], 0, 0, 0);
                    }
        });
        if constexpr (F == GA_SIGMOID_KV) asm volatile("" : "+v"(ks[0]), "+v"(ks[1]));
        bf16x8_t pf[NT];
        if constexpr (F == GA_TWO_MAPS || F == GA_SIGMOID_KV) {  // no maximum: all tiles go through every step together
            if constexpr (F == GA_TWO_MAPS) cap_scores(s);
            if constexpr (F == GA_SIGMOID_KV) {
#pragma unroll
                for (int t = 0; t < NT; ++t)
#pragma unroll
                    for (int kt = 0; kt < 2; ++kt) {
                        const f32x4_t f = __builtin_bit_cast(f32x4_t, ks[kt]);
#pragma unroll
                        for (int r = 0; r < 4; ++r) s[t][kt][r] = fmaf(s[t][kt][r] * sc, f[r], slope[t]);
                    }
            }
            bool edge = false;
#pragma unroll
            for (int t = 0; t < NT; ++t) edge = edge || j0 < full_lo[t] || j0 + 31 > full_hi[t];
            if (edge) {
                const int jl = j0 + 4 * g;
#pragma unroll
                for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                    for (int r = 0; r < 4; ++r)
#pragma unroll
                        for (int t = 0; t < NT; ++t) {
                            const int j = jl + 16 * kt + r, row = F == GA_TWO_MAPS ? 0 : t;  // (two maps: the same tokens)
                            if (j > rp[row] || j < rlo[row]) s[t][kt][r] = -INFINITY;
                        }
            }
#pragma unroll
            for (int t = 0; t < NT; ++t)
#pragma unroll
                for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        float p;
                        if constexpr (F == GA_SIGMOID_KV) {
                            p = __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-s[t][kt][r]));
                        } else {
                            p = __builtin_amdgcn_exp2f(s[t][kt][r]);
                            l_run[t] += p;
                        }
                        pf[t][4 * kt + r] = (__bf16)p;
                    }
        } else {
#pragma unroll
            for (int t = 0; t < NT; ++t) {
                if (!live[t]) {
#pragma unroll
                    for (int i = 0; i < 8; ++i) pf[t][i] = (__bf16)0.f;
                    continue;
                }
                if (F == GA_TWO_MAPS_ANY && cap_out > 0.f) cap_exact(s[t]);
                if (j0 < full_lo[t] || j0 + 31 > full_hi[t]) {
                    const int jl = j0 + 4 * g;
#pragma unroll
                    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            const int j = jl + 16 * kt + r;
                            if (j > rp[t] || j < rlo[t]) s[t][kt][r] = -INFINITY;
                        }
                }
                float mx = -INFINITY;
#pragma unroll
                for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                    for (int r = 0; r < 4; ++r) mx = fmaxf(mx, s[t][kt][r]);
                mx *= sc;
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
                        const float p = __builtin_amdgcn_exp2f(fmaf(s[t][kt][r], sc, -m_use));
                        l_run[t] += p;
                        pf[t][4 * kt + r] = (__bf16)p;
                    }
            }
        }
        static_for<VT / VG>([&](auto GI) {
            constexpr int d0 = decltype(GI)::value * VG;
            if constexpr (!VEARLY) read_v(std::integral_constant<int, d0>{});
            wait_lds();
#pragma unroll
            for (int i = 0; i < VG; ++i) asm volatile("" : "+v"(vf[i][0]), "+v"(vf[i][1]));
#pragma unroll
            for (int i = 0; i < VG; ++i) {
                const u32x4_t vv = {vf[i][0][0], vf[i][0][1], vf[i][1][0], vf[i][1][1]};
#pragma unroll
                for (int t = 0; t < NT; ++t)
                    acc[t][d0 + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, vv), pf[t], acc[t][d0 + i], 0, 0, 0);
            }
        });
    }
    __device__ __forceinline__ void set_cap(const GroupArgs& a) {
        if constexpr (!ga_two(F)) return;
        cap_in = a.cap > 0.f ? 2.f * GA_LOG2E * a.scale / a.cap : 0.f;
        cap_out = a.cap * GA_LOG2E;
        const float k = a.cap > 0.f ? a.scale / a.cap : 0.f, kk = k * k;
        cap_lim = k > 0.f ? 0.2f / k : 0.f;
        ca0 = cap_out * k;
        ca1 = ca0 * kk * (-1.f / 3.f);
        ca2 = ca0 * kk * kk * (2.f / 15.f);
        ca3 = ca0 * kk * kk * kk * (-17.f / 315.f);
        if constexpr (F == GA_TWO_MAPS) {
#pragma unroll
            for (int t = 0; t < NT; ++t) m_run[t] = 0.f;
        }
    }
    __device__ __forceinline__ float mass(int t) const {
        float l = l_run[t];
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);
        return l;
    }
};

// ---------------------------------------------------------------------------------------------------------------------------
// DK, DV: multiples of 64
template <int DK, int DV, int F>
__global__ __launch_bounds__(256, (DK + DV) <= 256 ? 2 : 1) void group_attn_prefill_kernel(const GroupArgs a) {
    using SL = Slab<DK, DV, 2, F>;
    constexpr bool TWO = ga_two(F), KV = F == GA_SIGMOID_KV;
    constexpr int KQ = SL::KQ, VT = SL::VT, KB = SL::KB, VB = SL::VB, KTILE = 64 * KB, VTILE = KV ? 256 : 64 * VB, STAGE = KTILE + VTILE;  // (behind the keys: values, or the keys' factors)
    constexpr int KCPR = DK / 8, VCPR = DV / 8, KDMA = DK / 32, VDMA = KV ? 0 : DV / 32;
    constexpr int MAPC = TWO ? KCPR / 2 : KCPR;  // chunks of one map in an LDS row
    extern __shared__ __attribute__((aligned(16))) char smem[];
    const int tid = threadIdx.x, lane = tid & 63;
    const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4;
    // XCD-aware order: workgroups with equal id % 8 share an XCD and take one contiguous run of (head, tile) items
    const int half = TWO ? 0 : a.pair;  // two heads per tile
    const int total = a.n_tiles * (a.H >> half), per = (total + 7) >> 3;
    const int item = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per || item >= total) return;
    const int h0 = (item / a.n_tiles) << half, tile = item % a.n_tiles, kvh = h0 / (a.H / a.G);
    const int seq = ga_uniform(a.tile_a[tile]), qo = ga_uniform(a.tile_b[tile]);
    const int qs = ga_uniform(a.q_start[seq]), nq = ga_uniform(a.q_start[seq + 1]) - qs;
    if (qo >= nq) return;
    const int p0 = ga_uniform(a.pos[qs]) + qo, plast = p0 + min((128 >> a.pair) - 1, nq - 1 - qo);  // positions of the tile's first and last row
    const int jlo = ga_first(a, p0) & ~63;
    const int n = ((plast - jlo) >> 6) + 1;
    const int32_t* bt = a.bt + (int64_t)(a.seq0 + seq) * a.bt_stride;
    const int dm = TWO ? a.dk / 2 : a.dk;
    SL S;
    S.init(lane);
    S.set_cap(a);
    // this wave's rows: tile t holds rows qo + 64 t + 16 w + c of the head (the two half-dead tiles of the causal edge cost all waves the
    // same) or, of a pair, rows qo + 16 w + c of its head t, or of its map t
    const int trow = a.pair ? 0 : 64;
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        const int r0 = qo + trow * t + 16 * w, r = r0 + c, h = h0 + half * t;
        const bool some = r0 < nq;
        S.rp[t] = r < nq ? p0 - qo + r : -1;
        S.rlo[t] = r < nq ? ga_first(a, S.rp[t]) : 0;
        if constexpr (KV) S.slope[t] = a.bias ? a.bias[h] * GA_LOG2E : 0.f;
        else S.slope[t] = a.slope ? a.slope[h] / a.scale : 0.f;
        const int a0 = p0 - qo + r0, a1 = p0 - qo + min(r0 + 15, nq - 1);
        S.any_lo[t] = some ? ga_first(a, a0) : 1 << 30;
        S.any_hi[t] = some ? a1 : -1;
        S.full_lo[t] = some ? ga_first(a, a1) : 1 << 30;
        S.full_hi[t] = some ? a0 : -1;
        const bf16_t* qp = reinterpret_cast<const bf16_t*>(a.q) + (int64_t)(qs + min(r, nq - 1)) * a.ldq + (int64_t)h * a.dk + (TWO ? t * dm : 0);
#pragma unroll
        for (int i = 0; i < KQ; ++i) {
            const int k = 32 * i + 8 * g;
            S.qf[t][i] = u32x4_t{0, 0, 0, 0};
            if (k < dm) S.qf[t][i] = *reinterpret_cast<const u32x4_t*>(qp + k);
        }
    }
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int i = 0; i < KQ; ++i) asm volatile("" : "+v"(S.qf[t][i]));
    const unsigned base = lds_addr(smem);
    // per-lane source offsets of the DMA pieces: constant over the tiles
    unsigned koff[KDMA], voff[VDMA + 1];
    int krow[KDMA], vrow[VDMA + 1];
    bool kpad[KDMA], vpad[VDMA + 1];
#pragma unroll
    for (int i = 0; i < KDMA; ++i) {
        const int q = (w * KDMA + i) * 64 + lane, row = q / KCPR, ch = (q % KCPR) ^ attn_swz(row);
        krow[i] = row;
        kpad[i] = (ch % MAPC) * 8 >= dm;
        koff[i] = (unsigned)(row * a.dk + (ch / MAPC) * dm + (ch % MAPC) * 8);
    }
#pragma unroll
    for (int i = 0; i < VDMA; ++i) {
        const int q = (w * VDMA + i) * 64 + lane, row = q / VCPR, ch = (q % VCPR) ^ attn_swz(row);
        vrow[i] = row;
        vpad[i] = ch * 8 >= a.dv;
        voff[i] = (unsigned)(row * a.dv + ch * 8);
    }
    // tiles from the last keys to the first: under a distance bias the maximum is found early and stays
    auto issue = [&](int it, int blk) {
        const int j0 = jlo + (n - 1 - it) * 64, left = ga_ok(a, blk) ? plast - j0 + 1 : 0;
        const int64_t row = ga_row(a, blk, j0, kvh);
        const bf16_t* kb = reinterpret_cast<const bf16_t*>(a.kc) + row * a.dk;
        const bf16_t* vb = reinterpret_cast<const bf16_t*>(a.vc) + row * a.dv;
        char* st = smem + (it & 1) * STAGE;
#pragma unroll
        for (int i = 0; i < KDMA; ++i) {
            const void* s = (kpad[i] || krow[i] >= left) ? (const void*)ga_zero_page : (const void*)(kb + koff[i]);
            lds_dma16(s, st + (w * KDMA + i) * 1024);
        }
#pragma unroll
        for (int i = 0; i < VDMA; ++i) {
            const void* s = (vpad[i] || vrow[i] >= left) ? (const void*)ga_zero_page : (const void*)(vb + voff[i]);
            lds_dma16(s, st + KTILE + (w * VDMA + i) * 1024);
        }
        if constexpr (KV) {
            if (w == 0) lds_dma4(a.kscale + (int64_t)(ga_ok(a, blk) ? blk : 0) * a.bs + (j0 - ga_block(a, j0) * a.bs) + lane, st + KTILE);
        }
    };
    const float sc = TWO && a.cap > 0.f ? 1.f : a.scale * GA_LOG2E;  // (capped scores are in log2 units)
    auto block_of = [&](int it) { return bt[ga_block(a, jlo + max(n - 1 - it, 0) * 64)]; };  // 64-key tiles lie in one block
    int blk = block_of(1);
    issue(0, ga_uniform(block_of(0)));
    for (int it = 0; it < n; ++it) {
        wait_vm<0>();
        __builtin_amdgcn_s_barrier();
        if (it + 1 < n) {
            issue(it + 1, ga_uniform(blk));
            blk = block_of(it + 2);
        }
        const unsigned kst = base + (it & 1) * STAGE, vst = kst + (KV ? 0 : KTILE);
#pragma unroll
        for (int s = 1; s >= 0; --s) S.run(kst + s * 32 * KB, vst + s * 32 * VB, jlo + (n - 1 - it) * 64 + s * 32, g, sc, kst + KTILE + s * 128);
    }
    if constexpr (TWO) {
        // both maps of a row are in the same lane: their difference and its norm over the head's columns (padding columns are zeros)
        const float i0 = 1.0f / S.mass(0), i1 = a.lam / S.mass(1);
        float ss = 0.f;
#pragma unroll
        for (int d = 0; d < VT; ++d)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float v = S.acc[0][d][e] * i0 - S.acc[1][d][e] * i1;
                S.acc[0][d][e] = v;
                ss += v * v;
            }
        ss += __shfl_xor(ss, 16, 64);
        ss += __shfl_xor(ss, 32, 64);
        const float f = a.post / sqrtf(ss / (float)a.vn + a.eps);
        const int r = qo + 16 * w + c;
        if (r >= nq) return;
        bf16_t* o = reinterpret_cast<bf16_t*>(a.out) + (int64_t)(qs + r) * a.ldo + (int64_t)h0 * a.dv;
#pragma unroll
        for (int d = 0; d < VT; ++d) {
            const int dim = 16 * d + 4 * g;
            if (dim >= a.dv) continue;
            f32x4_t v = S.acc[0][d] * f;
            if (a.gate) v *= ga_gate(a, qs + r, h0, dim);
            *reinterpret_cast<u32x2_t*>(o + dim) = u32x2_t{pack2bf(v[0], v[1]), pack2bf(v[2], v[3])};
        }
        return;
    }
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        const float l = S.mass(t);
        const int r = qo + trow * t + 16 * w + c, h = h0 + half * t;
        if (r >= nq) continue;
        const float sk = a.sink ? a.sink[h] * GA_LOG2E : -INFINITY;
        const float M = fmaxf(S.m_run[t], sk), f = __builtin_amdgcn_exp2f(S.m_run[t] - M);
        const float inv = KV ? 1.0f : f / (l * f + __builtin_amdgcn_exp2f(sk - M));
        bf16_t* o = reinterpret_cast<bf16_t*>(a.out) + (int64_t)(qs + r) * a.ldo + (int64_t)h * a.dv;
#pragma unroll
        for (int d = 0; d < VT; ++d) {
            const int dim = 16 * d + 4 * g;
            if (dim >= a.dv) continue;
            f32x4_t v = S.acc[t][d] * inv;
            if (a.gate) v *= ga_gate(a, qs + r, h, dim);
            *reinterpret_cast<u32x2_t*>(o + dim) = u32x2_t{pack2bf(v[0], v[1]), pack2bf(v[2], v[3])};
        }
    }
}

// ---------------------------------------------------------------------------------------------------------------------------
// Workgroup = (token tile, key / value head, group of 16 rows, KV split).  Row rho of a tile is token rho / R, head rho % R of the
// R = H / G heads that share the key / value head.  Every one of the NW waves takes each NW-th 32-key slab of the split with its own two LDS
// stages and softmax state: no barrier in the loop.
template <int DK, int DV, int NW, int F>
__global__ __launch_bounds__(NW * 64, 1) void group_attn_decode_kernel(const GroupArgs a, int row_groups) {
    constexpr bool TWO = ga_two(F), KV = F == GA_SIGMOID_KV;
    constexpr int RPG = TWO ? 8 : 16;  // (token, head) rows of a group: 16, or 8 of either map
    using SL = Slab<DK, DV, 1, F>;
    constexpr int KS = SL::KS, VT = SL::VT, KB = SL::KB, VB = SL::VB, KSLAB = 32 * KB, STAGE = KSLAB + (KV ? 256 : 32 * VB);
    constexpr int KCPR = DK / 8, VCPR = DV / 8, KDMA = DK / 16, VDMA = KV ? 0 : DV / 16, MAPC = TWO ? KCPR / 2 : KCPR;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    const int tid = threadIdx.x, lane = tid & 63;
    const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4;
    int item = blockIdx.x;
    const int split = item % a.nsplit;
    item /= a.nsplit;
    const int rg = item % row_groups;
    item /= row_groups;
    const int kvh = item % a.G, tile = item / a.G;
    const int tok0 = ga_uniform(a.tile_a[tile]), ntok = ga_uniform(a.tile_b[tile]), R = a.H / a.G;
    const int pA = ga_uniform(a.pos[tok0]), pB = pA + ntok - 1;
    const int map = TWO ? c >> 3 : 0, rho = rg * RPG + (TWO ? c & 7 : c), tok = rho / R, hh = rho - tok * R, h = kvh * R + hh;
    const bool row_ok = tok < ntok;
    if (rg * RPG >= ntok * R) return;
    const int jlo = pA >= 0 ? ga_first(a, pA) & ~31 : 0;
    const int slabs = pA >= 0 ? ((pB - jlo) >> 5) + 1 : 0, per = (slabs + a.nsplit - 1) / a.nsplit;
    const int s_lo = split * per, s_hi = min(s_lo + per, slabs);
    const int n = s_hi > s_lo + w ? (s_hi - s_lo - w + NW - 1) / NW : 0;  // slabs of this wave: s_hi - 1 - w - NW k, last keys first
    const int dm = TWO ? a.dk / 2 : a.dk;
    SL S;
    S.init(lane);
    S.set_cap(a);
    S.rp[0] = row_ok && pA >= 0 ? pA + tok : -1;
    S.rlo[0] = S.rp[0] >= 0 ? ga_first(a, S.rp[0]) : 0;
    if constexpr (KV) S.slope[0] = a.bias && row_ok ? a.bias[h] * GA_LOG2E : 0.f;
    else S.slope[0] = a.slope && row_ok ? a.slope[h] / a.scale : 0.f;
    {
        const int t0 = rg * RPG / R, t1 = min((rg * RPG + RPG - 1) / R, ntok - 1);
        S.any_lo[0] = ga_first(a, max(pA, 0) + t0);
        S.any_hi[0] = pA + t1;
        S.full_lo[0] = ga_first(a, max(pA, 0) + t1);
        S.full_hi[0] = rg * RPG + RPG <= ntok * R ? pA + t0 : -1;  // rows without a token: masked
    }
    const bf16_t* qp = reinterpret_cast<const bf16_t*>(a.q) + (int64_t)(tok0 + (row_ok ? tok : 0)) * a.ldq + (int64_t)(row_ok ? h : kvh * R) * a.dk;
#pragma unroll
    for (int i = 0; i < KS; ++i) {
        const int k = (TWO ? (i % (KS / 2)) * 32 : 32 * i) + 8 * g;
        S.qf[0][i] = u32x4_t{0, 0, 0, 0};
        if (k < dm && row_ok && (!TWO || i / (KS / 2) == map)) S.qf[0][i] = *reinterpret_cast<const u32x4_t*>(qp + map * dm + k);
    }
#pragma unroll
    for (int i = 0; i < KS; ++i) asm volatile("" : "+v"(S.qf[0][i]));
    const int32_t* bt = a.bt + (int64_t)(a.seq0 + a.seq_of[tok0]) * a.bt_stride;
    // keys of this step come straight from the projection's rows: positions from `own` on (the portion's first).  The tile's own tokens
    // are put into the cache here, by the first of the workgroups that share them
    const int own = a.knew ? pA - (tok0 - a.q_start[a.seq_of[tok0]]) : 1 << 30;
    if (a.knew && split == 0 && rg == 0 && pA >= 0) {
        const int ku = a.dk / 8, per_tok = ku + a.dv / 8;
        for (int i = tid; i < ntok * per_tok; i += NW * 64) {
            const int t = i / per_tok, u = i - t * per_tok;
            const int64_t r = tok0 + t, slot = a.slots[r];
            if (slot < 0 || slot >= a.n_blocks * a.bs) continue;
            const int64_t dst = (slot / a.bs * a.G + kvh) * a.bs + slot % a.bs;
            if (u < ku) reinterpret_cast<u32x4_t*>(const_cast<void*>(a.kc))[dst * ku + u] = *reinterpret_cast<const u32x4_t*>(reinterpret_cast<const bf16_t*>(a.knew) + r * a.ldkv + kvh * a.dk + u * 8);
            else reinterpret_cast<u32x4_t*>(const_cast<void*>(a.vc))[dst * (per_tok - ku) + u - ku] = *reinterpret_cast<const u32x4_t*>(reinterpret_cast<const bf16_t*>(a.vnew) + r * a.ldkv + kvh * a.dv + (u - ku) * 8);
        }
    }
    char* mine = smem + w * 2 * STAGE;
    const unsigned base = lds_addr(mine);
    unsigned koff[KDMA], voff[VDMA + 1];
    int krow[KDMA], vrow[VDMA + 1];
    bool kpad[KDMA], vpad[VDMA + 1];
#pragma unroll
    for (int i = 0; i < KDMA; ++i) {
        const int q = i * 64 + lane, row = q / KCPR, ch = (q % KCPR) ^ attn_swz(row);
        krow[i] = row;
        kpad[i] = (ch % MAPC) * 8 >= dm;
        koff[i] = (unsigned)(row * a.dk + (ch / MAPC) * dm + (ch % MAPC) * 8);
    }
#pragma unroll
    for (int i = 0; i < VDMA; ++i) {
        const int q = i * 64 + lane, row = q / VCPR, ch = (q % VCPR) ^ attn_swz(row);
        vrow[i] = row;
        vpad[i] = ch * 8 >= a.dv;
        voff[i] = (unsigned)(row * a.dv + ch * 8);
    }
    auto key0 = [&](int k) { return jlo + (s_hi - 1 - w - NW * k) * 32; };
    // block ids of this wave's next 64 slabs, one per lane
    auto blocks_from = [&](int k) { return k + lane < n ? bt[ga_block(a, key0(k + lane))] : -1; };
    int ids = n > 0 ? blocks_from(0) : -1;
    auto issue = [&](int k) {
        const int j0 = key0(k), blk = __builtin_amdgcn_readlane(ids, k & 63);
        const int left = ga_ok(a, blk) ? pB - j0 + 1 : 0;
        const int64_t row = ga_row(a, blk, j0, kvh);
        const bf16_t* kb = reinterpret_cast<const bf16_t*>(a.kc) + row * a.dk;
        const bf16_t* vb = reinterpret_cast<const bf16_t*>(a.vc) + row * a.dv;
        char* st = mine + (k & 1) * STAGE;
        if (j0 + 31 < own) {
#pragma unroll
            for (int i = 0; i < KDMA; ++i) lds_dma16<2>((kpad[i] || krow[i] >= left) ? (const void*)ga_zero_page : (const void*)(kb + koff[i]), st + i * 1024);
#pragma unroll
            for (int i = 0; i < VDMA; ++i) lds_dma16<2>((vpad[i] || vrow[i] >= left) ? (const void*)ga_zero_page : (const void*)(vb + voff[i]), st + KSLAB + i * 1024);
            if constexpr (KV) lds_dma4(a.kscale + (int64_t)(ga_ok(a, blk) ? blk : 0) * a.bs + (j0 - ga_block(a, j0) * a.bs) + (lane & 31), st + KSLAB);
            return;
        }
        if constexpr (KV) return;  // (keys with factors are in the cache already: no new rows, `own` is out of reach)
        const bf16_t* kn = reinterpret_cast<const bf16_t*>(a.knew) + (int64_t)(tok0 + j0 - pA) * a.ldkv + kvh * a.dk;
        const bf16_t* vn = reinterpret_cast<const bf16_t*>(a.vnew) + (int64_t)(tok0 + j0 - pA) * a.ldkv + kvh * a.dv;
#pragma unroll
        for (int i = 0; i < KDMA; ++i) {
            const bf16_t* s = j0 + krow[i] >= own ? kn + krow[i] * a.ldkv + ((int)koff[i] - krow[i] * a.dk) : kb + koff[i];
            lds_dma16((kpad[i] || krow[i] >= left) ? (const void*)ga_zero_page : (const void*)s, st + i * 1024);
        }
#pragma unroll
        for (int i = 0; i < VDMA; ++i) {
            const bf16_t* s = j0 + vrow[i] >= own ? vn + vrow[i] * a.ldkv + ((int)voff[i] - vrow[i] * a.dv) : vb + voff[i];
            lds_dma16((vpad[i] || vrow[i] >= left) ? (const void*)ga_zero_page : (const void*)s, st + KSLAB + i * 1024);
        }
    };
    const float sc = TWO && a.cap > 0.f ? 1.f : a.scale * GA_LOG2E;
    if (n > 0) issue(0);
    for (int k = 0; k < n; ++k) {
        if (k + 1 < n) {
            if (((k + 1) & 63) == 0) ids = blocks_from(k + 1);
            issue(k + 1);
            wait_vm<KDMA + VDMA + (KV ? 1 : 0)>();  // slab k is in, slab k + 1 may be on its way
        } else {
            wait_vm<0>();
        }
        const unsigned kst = base + (k & 1) * STAGE;
        S.run(kst, kst + (KV ? 0 : KSLAB), key0(k), g, sc, kst + KSLAB);
    }
    // ---- the waves' sums through LDS (over the stages: every wave is past its last read) ----
    const float l = S.mass(0);
    __syncthreads();
    float* ml = reinterpret_cast<float*>(smem);                    // [NW][16][2]
    float* po = reinterpret_cast<float*>(smem + NW * 16 * 2 * 4);  // [NW][16][DV + 4]
    constexpr int PO = DV + 4;
    if (g == 0) {
        ml[(w * 16 + c) * 2] = KV ? 0.f : S.m_run[0];
        ml[(w * 16 + c) * 2 + 1] = KV ? 1.f : l;
    }
#pragma unroll
    for (int d = 0; d < VT; ++d) *reinterpret_cast<f32x4_t*>(po + (w * 16 + c) * PO + 16 * d + 4 * g) = S.acc[0][d];
    __syncthreads();
    constexpr int QPR = DV / 4;
    for (int i = tid; i < 16 * QPR; i += NW * 64) {
        const int rr = i / QPR, col = (i - rr * QPR) * 4;
        const int rh = rg * RPG + (TWO ? rr & 7 : rr), tk = rh / R, head = kvh * R + (rh - tk * R);
        if (tk >= ntok || col >= a.dv) continue;
        float M = -INFINITY;
#pragma unroll
        for (int x = 0; x < NW; ++x) M = fmaxf(M, ml[(x * 16 + rr) * 2]);
        const float sk = (a.nsplit == 1 && a.sink) ? a.sink[head] * GA_LOG2E : -INFINITY;
        const float Ms = fmaxf(M, sk);
        float L = 0.f;
        f32x4_t o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int x = 0; x < NW; ++x) {
            const float mx = ml[(x * 16 + rr) * 2];
            const float f = mx == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(mx - Ms);
            L += f * ml[(x * 16 + rr) * 2 + 1];
            const f32x4_t v = *reinterpret_cast<const f32x4_t*>(po + (x * 16 + rr) * PO + col);
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] += f * v[e];
        }
        const int64_t row = (int64_t)(tok0 + tk);
        if (!TWO && a.nsplit == 1) {
            if (sk > -INFINITY) L += __builtin_amdgcn_exp2f(sk - Ms);
            o *= KV ? 1.0f : L > 0.f ? 1.0f / L : 0.f;
            if (a.gate) o *= ga_gate(a, row, head, col);
            *reinterpret_cast<u32x2_t*>(reinterpret_cast<bf16_t*>(a.out) + row * a.ldo + (int64_t)head * a.dv + col) = u32x2_t{pack2bf(o[0], o[1]), pack2bf(o[2], o[3])};
        } else {
            const int64_t pr = (TWO ? (row * a.H + head) * 2 + (rr >> 3) : row * a.H + head) * a.nsplit + split;
            *reinterpret_cast<f32x4_t*>(a.part_o + pr * a.dv + col) = o;
            if (col == 0) {
                a.part_ml[pr * 2] = M;
                a.part_ml[pr * 2 + 1] = L;
            }
        }
    }
}

// ---------------------------------------------------------------------------------------------------------------------------
// any head size, fp32 arithmetic throughout: one (row, head) per workgroup, 256 keys at a time, one key per thread
template <typename T>
__device__ __forceinline__ float ga_f(T v);
template <>
__device__ __forceinline__ float ga_f<float>(float v) { return v; }
template <>
__device__ __forceinline__ float ga_f<bf16_t>(bf16_t v) { return bf2f(v); }

template <typename T>
__global__ __launch_bounds__(256) void group_attn_plain_kernel(const GroupArgs a) {
    extern __shared__ __attribute__((aligned(16))) char smem[];
    float* sq = reinterpret_cast<float*>(smem);  // [dk] query
    float* so = sq + a.dk;                        // [maps][dv] output
    float* sp = so + a.maps * a.dv;               // [256] weights, then partial sums
    __shared__ float s_red[4];
    __shared__ int64_t s_row[256];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int h = blockIdx.x % a.H, kvh = h / (a.H / a.G);
    const int64_t r = blockIdx.x / a.H;
    const int p = a.pos[r];
    T* out = reinterpret_cast<T*>(a.out) + r * a.ldo + (int64_t)h * a.dv;
    auto put = [&](int d, float v) {
        if (a.gate) v *= ga_f<T>(reinterpret_cast<const T*>(a.gate)[r * a.ldg + (a.gate_cols ? (int64_t)h * a.dv + d : h)]);
        if constexpr (sizeof(T) == 4) out[d] = v;
        else out[d] = f2bf(v);
    };
    if (p < 0) {
        for (int d = tid; d < a.dv; d += 256) {
            if constexpr (sizeof(T) == 4) out[d] = 0.f;
            else out[d] = 0;
        }
        return;
    }
    const T* q = reinterpret_cast<const T*>(a.q) + r * a.ldq + (int64_t)h * a.dk;
    for (int d = tid; d < a.dk; d += 256) sq[d] = ga_f<T>(q[d]);
    for (int d = tid; d < a.maps * a.dv; d += 256) so[d] = 0.f;
    const int32_t* bt = a.bt + (int64_t)(a.seq0 + a.seq_of[r]) * a.bt_stride;
    const int lo = ga_first(a, p), dm = a.dk / a.maps;
    const float slope = a.slope ? a.slope[h] : 0.f, bias = a.bias ? a.bias[h] : 0.f;
    const int ncol = min(a.dv, 256), parts = 256 / ncol;
    auto total = [&](float v) {  // sum over the workgroup
        v = wave_sum(v);
        __syncthreads();
        if (lane == 0) s_red[wid] = v;
        __syncthreads();
        return s_red[0] + s_red[1] + s_red[2] + s_red[3];
    };
    for (int map = 0; map < a.maps; ++map) {
        float* o = so + map * a.dv;
        float m = a.sink ? a.sink[h] : -INFINITY, l = a.sink ? 1.0f : 0.f;  // the sink's mass from the start
        for (int j0 = lo; j0 <= p; j0 += 256) {
            const int j = j0 + tid;
            float s = -INFINITY;
            __syncthreads();
            if (j <= p) {
                const int blk = bt[ga_block(a, j)];
                const int64_t row = ga_ok(a, blk) ? ga_row(a, blk, j, kvh) : 0;
                s_row[tid] = row;
                const T* k = reinterpret_cast<const T*>(a.kc) + row * a.dk + map * dm;
                float acc = 0.f;
                for (int d = 0; d < dm; d += 4) {  // dm is a multiple of 8
#pragma unroll
                    for (int e = 0; e < 4; ++e) acc = fmaf(sq[map * dm + d + e], ga_f<T>(k[d + e]), acc);
                }
                if (a.kscale) acc *= a.kscale[(int64_t)(ga_ok(a, blk) ? blk : 0) * a.bs + (j - ga_block(a, j) * a.bs)];
                s = acc * a.scale - slope * (float)(p - j);
                if (a.cap > 0.f) s = a.cap * tanhf(s / a.cap);
            }
            float e, alpha = 1.0f;
            if (a.sigmoid) {
                e = j <= p ? 1.0f / (1.0f + expf(-(s + bias))) : 0.f;
            } else {
                const float bm = wave_max(s);
                if (lane == 0) s_red[wid] = bm;
                __syncthreads();
                const float m_new = fmaxf(m, fmaxf(fmaxf(s_red[0], s_red[1]), fmaxf(s_red[2], s_red[3])));
                e = j <= p ? expf(s - m_new) : 0.f;
                alpha = m == -INFINITY ? 0.f : expf(m - m_new);
                l = l * alpha + total(e);
                m = m_new;
            }
            sp[tid] = e;
            __syncthreads();
            const int nk = min(256, p - j0 + 1);
            for (int c0 = 0; c0 < a.dv; c0 += ncol) {
                const int col = c0 + tid % ncol, part = tid / ncol;
                float acc = 0.f;
                if (part < parts && col < a.dv)
                    for (int i = part; i < nk; i += parts) acc = fmaf(sp[i], ga_f<T>(reinterpret_cast<const T*>(a.vc)[s_row[i] * a.dv + col]), acc);
                float* sums = sp + 256;
                sums[tid] = acc;
                __syncthreads();
                if (part == 0 && col < a.dv) {
                    for (int i = 1; i < parts; ++i) acc += sums[i * ncol + tid];
                    o[col] = o[col] * alpha + acc;
                }
                __syncthreads();
            }
        }
        __syncthreads();
        const float inv = a.sigmoid ? 1.0f : l;
        for (int d = tid; d < a.dv; d += 256) {
            if (a.maps == 1) put(d, o[d] / inv);
            else o[d] = o[d] / inv;
        }
    }
    if (a.maps == 1) return;
    __syncthreads();
    float ss = 0.f;
    for (int d = tid; d < a.dv; d += 256) {
        const float v = so[d] - a.lam * so[a.dv + d];
        so[d] = v;  // (a thread's own columns)
        ss = fmaf(v, v, ss);
    }
    const float f = a.post / sqrtf(total(ss) / (float)a.vn + a.eps);
    for (int d = tid; d < a.dv; d += 256) put(d, so[d] * f);
}

template <int DK, int DV, int F>
int launch_prefill(const GroupArgs& a, hipStream_t st) {
    constexpr int LDS = 2 * 64 * (DK + (F == GA_SIGMOID_KV ? 2 : DV)) * 2;
    static_assert(LDS <= 160 * 1024, "LDS of a CU");
    auto kern = group_attn_prefill_kernel<DK, DV, F>;
    GLM_SET_MAX_LDS(kern, LDS, "glm_group_attn_prefill");
    const int64_t per = ((int64_t)a.n_tiles * (a.H >> (ga_two(F) ? 0 : a.pair)) + 7) / 8;
    GLM_CHECK_ARG(per * 8 < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_group_attn_prefill: grid too large");
    hipLaunchKernelGGL(kern, dim3((unsigned)(per * 8)), dim3(256), LDS, st, a);
    GLM_CHECK_LAUNCH("glm_group_attn_prefill");
    return GLM_OK;
}

template <int DK, int DV, int F>
int launch_decode(const GroupArgs& a, int row_groups, hipStream_t st) {
    constexpr int ROW = DK + (F == GA_SIGMOID_KV ? 4 : DV);  // (factors: 256 bytes a slab)
    constexpr int NW = ROW <= 320 ? 4 : 2;  // as many waves as have room for two stages each
    constexpr int STG = NW * 2 * 32 * ROW * 2, RED = NW * 16 * (2 + DV + 4) * 4, LDS = STG > RED ? STG : RED;
    static_assert(LDS <= 160 * 1024, "LDS of a CU");
    auto kern = group_attn_decode_kernel<DK, DV, NW, F>;
    const int64_t grid = (int64_t)a.n_tiles * a.G * row_groups * a.nsplit;
    GLM_CHECK_ARG(grid < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_group_attn_decode: grid too large");
    GLM_SET_MAX_LDS(kern, LDS, "glm_group_attn_decode");
    hipLaunchKernelGGL(kern, dim3((unsigned)grid), dim3(NW * 64), LDS, st, a, row_groups);
    GLM_CHECK_LAUNCH("glm_group_attn_decode");
    return GLM_OK;
}

#define GA_SIZES(F, kk, vv, form, ...)                                    \
    do {                                                                  \
        if (kk == 1 && vv == 1) return F<64, 64, form>(__VA_ARGS__);      \
        if (kk == 1 && vv == 2) return F<64, 128, form>(__VA_ARGS__);     \
        if (kk == 1) return F<64, 256, form>(__VA_ARGS__);                \
        if (kk == 2 && vv == 1) return F<128, 64, form>(__VA_ARGS__);     \
        if (kk == 2 && vv == 2) return F<128, 128, form>(__VA_ARGS__);    \
        if (kk == 2) return F<128, 256, form>(__VA_ARGS__);               \
        if (vv == 1) return F<256, 64, form>(__VA_ARGS__);                \
        if (vv == 2) return F<256, 128, form>(__VA_ARGS__);               \
        return F<256, 256, form>(__VA_ARGS__);                            \
    } while (0)
// (a map of dk / 2 columns is padded to 32, 64 or 128 in LDS: key rows of 64, 128, 256)
#define GA_FORMS(F, ...)                                                                             \
    do {                                                                                             \
        const int unit = a.maps == 2 ? 32 : 64, kk = (a.dk / a.maps + unit - 1) / unit, vv = (a.dv + 63) / 64; \
        if (a.sigmoid) {                                                                             \
            if (kk == 1) return F<64, 64, GA_SIGMOID_KV>(__VA_ARGS__);                               \
            if (kk == 2) return F<128, 128, GA_SIGMOID_KV>(__VA_ARGS__);                             \
            return F<256, 256, GA_SIGMOID_KV>(__VA_ARGS__);                                          \
        }                                                                                            \
        if (a.maps == 2 && a.cap > 0.f && a.cap <= GA_CAP_FITS) GA_SIZES(F, kk, vv, GA_TWO_MAPS, __VA_ARGS__); \
        if (a.maps == 2) GA_SIZES(F, kk, vv, GA_TWO_MAPS_ANY, __VA_ARGS__);                          \
        GA_SIZES(F, kk, vv, GA_SOFTMAX, __VA_ARGS__);                                                \
    } while (0)

int run_prefill(const GroupArgs& a, hipStream_t st) { GA_FORMS(launch_prefill, a, st); }
int run_decode(const GroupArgs& a, int row_groups, hipStream_t st) { GA_FORMS(launch_decode, a, row_groups, st); }

int log2_of(int n) {
    for (int i = 0; i < 30; ++i)
        if (n == 1 << i) return i;
    return -1;
}

// what the three attention entry points share
int group_args(GroupArgs& a, const char* name, const void* q, int64_t ldq, const void* kc, const void* vc, int64_t n_blocks, int bs, const int32_t* bt,
               int64_t bt_stride, int seq0, int H, int G, int dk, int dv, const glm_group_form* f, void* out, int64_t ldo) {
    GLM_CHECK_ARG(q && kc && vc && bt && out && f, GLM_ERR_INVALID, "%s: null pointer", name);
    GLM_CHECK_ARG(H > 0 && G > 0 && H % G == 0 && dk > 0 && dv > 0 && dk % 8 == 0 && dv % 8 == 0 && ldq >= (int64_t)H * dk && ldo >= (int64_t)H * dv && ldq % 8 == 0 && ldo % 4 == 0 &&
                      n_blocks > 0 && bs > 0 && bs % 64 == 0 && bt_stride > 0 && seq0 >= 0 && f->window >= 0 && f->chunk >= 0 && glm_aligned16(q) && glm_aligned16(kc) && glm_aligned16(vc) &&
                      (((uintptr_t)out) & 7) == 0, GLM_ERR_INVALID, "%s: bad shape H=%d G=%d dk=%d dv=%d ldq=%ld ldo=%ld block=%d", name, H, G, dk, dv, (long)ldq, (long)ldo, bs);
    GLM_CHECK_ARG((f->maps == 1 || (f->maps == 2 && dk % 16 == 0 && f->vn > 0 && f->vn <= dv)) && f->cap >= 0.f && (!f->kscale || (f->sigmoid && kc == vc && dk == dv)) &&
                      (!f->sigmoid || (f->maps == 1 && !f->sink && f->cap == 0.f && !f->slope)) && (!f->bias || f->sigmoid) && (!f->gate || (f->ldg >= (f->gate_cols ? (int64_t)H * dv : H) &&
                      (!f->gate_cols || (f->ldg % 4 == 0 && (((uintptr_t)f->gate) & 7) == 0)))), GLM_ERR_INVALID, "%s: parts that do not go together", name);
    a = GroupArgs{};
    a.q = q; a.ldq = ldq; a.kc = kc; a.vc = vc; a.n_blocks = n_blocks; a.bs = bs; a.log2_bs = log2_of(bs); a.bt = bt; a.bt_stride = bt_stride; a.seq0 = seq0;
    a.H = H; a.G = G; a.dk = dk; a.dv = dv; a.out = out; a.ldo = ldo; a.nsplit = 1;
    a.window = f->window; a.chunk = f->chunk; a.scale = f->scale; a.slope = f->slope; a.sink = f->sink; a.cap = f->cap; a.maps = f->maps; a.lam = f->lam; a.post = f->post; a.eps = f->eps;
    a.vn = f->vn; a.sigmoid = f->sigmoid; a.bias = f->bias; a.kscale = f->kscale; a.gate = f->gate; a.ldg = f->ldg; a.gate_cols = f->gate_cols;
    return GLM_OK;
}

// what the tiled kernels take of it
int group_tiled(const GroupArgs& a, const char* name) {
    GLM_CHECK_ARG(a.dk <= 256 && a.dv <= 256 && a.scale > 0.f, GLM_ERR_UNSUPPORTED, "%s: head sizes up to 256 (two maps: together), a positive scale (dk=%d dv=%d)", name, a.dk, a.dv);
    GLM_CHECK_ARG(a.sigmoid ? a.kscale != nullptr : a.maps == 2 ? !a.slope && !a.sink : a.cap == 0.f, GLM_ERR_UNSUPPORTED, "%s: this combination is glm_group_attn_plain's", name);
    return GLM_OK;
}

}  // namespace

extern "C" int glm_group_kv_store(const void* src, int64_t ld, int64_t k_off, int64_t v_off, int f32, const int32_t* slots, int64_t T, void* kc, void* vc, int64_t n_slots, int bs,
                                  int G, int dk, int dv, glm_stream_t stream) {
    const int es = f32 ? 4 : 2;
    GLM_CHECK_ARG(src && slots && kc && vc && T >= 0 && bs > 0 && n_slots > 0 && n_slots % bs == 0 && G > 0 && dk > 0 && dv > 0 && dk % 8 == 0 && dv % 8 == 0 && ld % 8 == 0 && k_off % 8 == 0 && v_off % 8 == 0 &&
                      k_off >= 0 && v_off >= 0 && ld >= k_off + (int64_t)G * dk && ld >= v_off + (int64_t)G * dv && glm_aligned16(src) && glm_aligned16(kc) && glm_aligned16(vc), GLM_ERR_INVALID,
                  "glm_group_kv_store: bad shape T=%ld G=%d dk=%d dv=%d ld=%ld", (long)T, G, dk, dv, (long)ld);
    if (T == 0) return GLM_OK;
    StoreArgs a = {(const char*)src, ld * es, k_off * es, v_off * es, slots, (char*)kc, (char*)vc, T, n_slots, G, bs, dk * es / 16, dv * es / 16};
    const int64_t items = T * G * (a.ku + a.vu);
    GLM_CHECK_ARG((items + 255) / 256 < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_group_kv_store: too many rows");
    hipLaunchKernelGGL(group_kv_store_kernel, dim3((unsigned)((items + 255) / 256)), dim3(256), 0, glm_s(stream), a);
    GLM_CHECK_LAUNCH("glm_group_kv_store");
    return GLM_OK;
}

extern "C" int glm_group_attn_prefill(const void* q, int64_t ldq, const void* kc, const void* vc, int64_t n_blocks, int bs, const int32_t* block_tables, int64_t bt_stride, int seq0,
                                      const int32_t* q_start, const int32_t* pos, const int32_t* tile_seq, const int32_t* tile_off, int n_tiles, int tile_rows, int H, int G, int dk, int dv,
                                      const glm_group_form* form, void* out, int64_t ldo, glm_stream_t stream) {
    GroupArgs a;
    const int rc = group_args(a, "glm_group_attn_prefill", q, ldq, kc, vc, n_blocks, bs, block_tables, bt_stride, seq0, H, G, dk, dv, form, out, ldo);
    if (rc != GLM_OK) return rc;
    GLM_CHECK_ARG(q_start && pos && tile_seq && tile_off && n_tiles >= 0, GLM_ERR_INVALID, "glm_group_attn_prefill: no tiles");
    const int ru = group_tiled(a, "glm_group_attn_prefill");
    if (ru != GLM_OK) return ru;
    GLM_CHECK_ARG(a.maps == 2 ? tile_rows == 64 : tile_rows == 128 || (tile_rows == 64 && (H / G) % 2 == 0), GLM_ERR_UNSUPPORTED,
                  "glm_group_attn_prefill: tiles of %d rows (128, or 64 where heads pair up or have two maps)", tile_rows);
    if (n_tiles == 0) return GLM_OK;
    a.pair = tile_rows == 64;
    a.q_start = q_start; a.pos = pos; a.tile_a = tile_seq; a.tile_b = tile_off; a.n_tiles = n_tiles;
    return run_prefill(a, glm_s(stream));
}

extern "C" int glm_group_attn_decode(const void* q, int64_t ldq, const void* kc, const void* vc, int64_t n_blocks, int bs, const int32_t* block_tables, int64_t bt_stride,
                                     const int32_t* pos, const int32_t* seq_of, const int32_t* tile_tok, const int32_t* tile_n, int n_tiles, int tokens_per_tile, int H, int G, int dk, int dv,
                                     const glm_group_form* form, const void* knew, const void* vnew, int64_t ldkv, const int32_t* q_start,
                                     const int32_t* slots, void* out, int64_t ldo, int nsplit, float* part_o, float* part_ml, glm_stream_t stream) {
    GroupArgs a;
    const int rc = group_args(a, "glm_group_attn_decode", q, ldq, kc, vc, n_blocks, bs, block_tables, bt_stride, 0, H, G, dk, dv, form, out, ldo);
    if (rc != GLM_OK) return rc;
    GLM_CHECK_ARG(pos && seq_of && tile_tok && tile_n && n_tiles >= 0 && tokens_per_tile >= 1 && nsplit >= 1 && nsplit <= 64 && ((nsplit == 1 && form->maps == 1) || (part_o && part_ml)), GLM_ERR_INVALID,
                  "glm_group_attn_decode: bad tiles or splits (%d)", nsplit);
    const int ru = group_tiled(a, "glm_group_attn_decode");
    if (ru != GLM_OK) return ru;
    GLM_CHECK_ARG(!knew || (a.maps == 1 && !a.sigmoid), GLM_ERR_UNSUPPORTED, "glm_group_attn_decode: rows of new keys only in the softmax form with one map");
    GLM_CHECK_ARG(!knew || (vnew && q_start && slots && ldkv >= (int64_t)G * (dk > dv ? dk : dv) && ldkv % 8 == 0 && glm_aligned16(knew) && glm_aligned16(vnew)), GLM_ERR_INVALID,
                  "glm_group_attn_decode: bad rows of new keys and values (ldkv=%ld)", (long)ldkv);
    if (n_tiles == 0) return GLM_OK;
    a.knew = knew; a.vnew = vnew; a.ldkv = ldkv; a.q_start = q_start; a.slots = slots;
    a.pos = pos; a.seq_of = seq_of; a.tile_a = tile_tok; a.tile_b = tile_n; a.n_tiles = n_tiles; a.nsplit = nsplit; a.part_o = part_o; a.part_ml = part_ml;
    const int rpg = a.maps == 2 ? 8 : 16;
    return run_decode(a, (tokens_per_tile * (H / G) + rpg - 1) / rpg, glm_s(stream));
}

extern "C" int glm_group_attn_plain(const void* q, int64_t ldq, const void* kc, const void* vc, int64_t n_blocks, int bs, const int32_t* block_tables, int64_t bt_stride, const int32_t* pos,
                                    const int32_t* seq_of, int64_t rows, int H, int G, int dk, int dv, const glm_group_form* form, void* out,
                                    int64_t ldo, int f32, glm_stream_t stream) {
    GroupArgs a;
    const int rc = group_args(a, "glm_group_attn_plain", q, ldq, kc, vc, n_blocks, bs, block_tables, bt_stride, 0, H, G, dk, dv, form, out, ldo);
    if (rc != GLM_OK) return rc;
    GLM_CHECK_ARG(pos && seq_of && rows >= 0 && rows * H < (1ll << 31), GLM_ERR_INVALID, "glm_group_attn_plain: bad rows (%ld)", (long)rows);
    const size_t lds = (size_t)(dk + a.maps * dv + 512) * 4;
    GLM_CHECK_ARG(lds <= 60 * 1024, GLM_ERR_UNSUPPORTED, "glm_group_attn_plain: head sizes %d + %d", dk, dv);
    if (rows == 0) return GLM_OK;
    a.pos = pos; a.seq_of = seq_of; a.rows = rows;
    if (f32) hipLaunchKernelGGL(group_attn_plain_kernel<float>, dim3((unsigned)(rows * H)), dim3(256), lds, glm_s(stream), a);
    else hipLaunchKernelGGL(group_attn_plain_kernel<bf16_t>, dim3((unsigned)(rows * H)), dim3(256), lds, glm_s(stream), a);
    GLM_CHECK_LAUNCH("glm_group_attn_plain");
    return GLM_OK;
}
