// latent_attn.hip — attention over a paged cache of latent rows (one row c of `rank` values per token, shared by all heads),
// with a sliding window and a learned sink per head, in the ABSORBED form: with k = W_uk c and v = W_uv c,
//
//     q . k = (W_uk^T q) . c          sum_j p_j v_j = W_uv (sum_j p_j c_j)
//
// so a query row attends directly over the cached latents, every row of which is read once for all heads.  The form for few
// query rows per sequence (decode, short portions); long portions expand k and v (window_attn.hip).  gfx950 only.
//
//   latent_prepare   one launch: latent norm + cache store of the step's tokens, and q' = W_uk^T q of the absorbed rows
//   latent_attn      split-KV flash loop over the pages; rows are (token, head) pairs; fp32 scores and softmax
//   latent_up        out = W_uv ctx, times an output gate if there is one
//
// With a rotated key part that all heads share (rotp columns behind the latent's rp in a cache row), queries that go through a latent of
// their own and positions, latent_prepare is two launches: latent_rows (both latents' norms, the rotated key, cache store) in front of
// the query projection and latent_absorb (q' and the rotated query part behind it) after it; the scores then run over rp + rotp
// columns, the values over the first rp.
//
// Roofline of latent_attn at decode: HBM — window * rank * 2 bytes per sequence, read once.  Four waves per 16 query rows share
// every 64-key tile, double-buffered by LDS-DMA.  One LDS image serves both products: chunk ^ swz(key) with
// swz(key) = (key & 3) << 1 | (key >> 2) & 1 is conflict-free for the ds_read_b128 row reads and for the transposed
// ds_read_b64_tr_b16 reads.  Keys outside the sequence's range and padding columns are fetched from a page of zeros, never
// from unused cache memory (whatever lies there would turn a zero weight into a NaN).
#include "common.h"
#include "attn_lds.h"

namespace {

constexpr float LOG2E = 1.4426950408889634f;
constexpr int LA_BT = 1024;  // block-table entries a workgroup caches in LDS

__device__ const u32x4_t la_zero_page[4] = {};

// ---------------------------------------------------------------------------------------------------------------------------
struct PrepArgs {
    const void* q;         // [T, ldqq] queries, head h at h*hd: dimp unrotated columns, then rotp rotated ones
    int64_t ldqq;
    int hd;
    const void* qc;        // [T, ldq] projection rows: raw latent at c_off, raw rotated key part at c_off + rp
    int64_t ldq;
    int c_off;
    int64_t T, Ta;         // rows; rows [0, Ta) are absorbed
    int H, dimp, rank, rp; // rp = rank rounded up to 8
    int rotp, rc;          // rotated columns; rc = rp + rotp, the pitch of cache, c_out and qa rows
    const float* cs;       // [T, rotp / 2, 2] cos, sin of the pairs of columns (2i, 2i+1)
    int cq_off, cq_rank, cq_rp;  // latent of the queries in qc, or cq_out = nullptr
    const float* cq_norm;  // [cq_rp]
    void* cq_out;          // [T, ld_cq]
    int64_t ld_cq;
    const float* norm_w;   // [rp]
    float eps;
    const int32_t* slots;  // [T] cache row of the token, < 0: none
    void* cache;           // [n_slots, rc]
    int64_t n_slots;
    const int32_t* crow;   // [T] row of c_out, < 0: none (nullptr: no c_out)
    void* c_out;           // [n_crows, rc]
    int64_t n_crows;
    const bf16_t* wukt;    // [H, rp, dimp]
    bf16_t* qa;            // [Ta, H, rc]
};

// latent norm of one token by one wave, eight columns per lane and step (the padding columns of the projection are zeros)
template <typename E>
__device__ __forceinline__ void la_ld8(const void* p, int64_t i, float (&v)[8]) {
    if constexpr (sizeof(E) == 2) {
        const u32x4_t u = *reinterpret_cast<const u32x4_t*>(reinterpret_cast<const bf16_t*>(p) + i);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            v[2 * j] = bflo(u[j]);
            v[2 * j + 1] = bfhi(u[j]);
        }
    } else {
        const float* f = reinterpret_cast<const float*>(p) + i;
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = f[j];
    }
}
template <typename E>
__device__ __forceinline__ void la_st8(void* p, int64_t i, const float (&v)[8]) {
    if constexpr (sizeof(E) == 2) {
        *reinterpret_cast<u32x4_t*>(reinterpret_cast<bf16_t*>(p) + i) =
            u32x4_t{pack2bf(v[0], v[1]), pack2bf(v[2], v[3]), pack2bf(v[4], v[5]), pack2bf(v[6], v[7])};
    } else {
        float* f = reinterpret_cast<float*>(p) + i;
#pragma unroll
        for (int j = 0; j < 8; ++j) f[j] = v[j];
    }
}
// RMS norm of columns [off, off + rp) of R rows t0 .. by one wave, their loads together; put(row, column, eight values)
template <typename E, int R, class Put>
__device__ __forceinline__ void norm_rows(const void* x, int64_t ld, int off, int64_t T, int64_t t0, int lane, int rank, int rp, const float* gain, float eps, Put put) {
    float v[R][8], s[R];
#pragma unroll
    for (int i = 0; i < R; ++i) s[i] = 0.f;
    for (int k = lane * 8; k < rp; k += 512) {
#pragma unroll
        for (int i = 0; i < R; ++i) la_ld8<E>(x, min(t0 + i, T - 1) * ld + off + k, v[i]);
#pragma unroll
        for (int i = 0; i < R; ++i)
#pragma unroll
            for (int j = 0; j < 8; ++j) s[i] += v[i][j] * v[i][j];
    }
#pragma unroll
    for (int i = 0; i < R; ++i) s[i] = 1.0f / sqrtf(wave_sum(s[i]) / (float)rank + eps);
    for (int k = lane * 8; k < rp; k += 512) {
        float w[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) w[j] = gain[k + j];
#pragma unroll
        for (int i = 0; i < R; ++i) {
            if (t0 + i >= T) continue;
            if (rp > 512) la_ld8<E>(x, (t0 + i) * ld + off + k, v[i]);  // (one step: the values are still in registers)
#pragma unroll
            for (int j = 0; j < 8; ++j) v[i][j] = v[i][j] * s[i] * w[j];
            put(i, k, v[i]);
        }
    }
}
// pairs (u, v) of eight columns -> (u cos - v sin, v cos + u sin)
__device__ __forceinline__ void la_rotate8(float (&x)[8], const float* cs) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const float c = cs[2 * j], s = cs[2 * j + 1], u = x[2 * j], v = x[2 * j + 1];
        x[2 * j] = u * c - v * s;
        x[2 * j + 1] = v * c + u * s;
    }
}
template <typename E, int R>
__device__ void latent_norm_rows(const PrepArgs& a, int64_t t0, int lane) {
    int64_t slot[R], row[R];
#pragma unroll
    for (int i = 0; i < R; ++i) {
        const int64_t t = min(t0 + i, a.T - 1);
        slot[i] = a.slots[t];
        row[i] = a.crow ? a.crow[t] : -1;
    }
    auto put = [&](int i, int k, const float (&v)[8]) {
        if (slot[i] >= 0 && slot[i] < a.n_slots) la_st8<E>(a.cache, slot[i] * a.rc + k, v);
        if (row[i] >= 0 && row[i] < a.n_crows) la_st8<E>(a.c_out, row[i] * a.rc + k, v);
    };
    norm_rows<E, R>(a.qc, a.ldq, a.c_off, a.T, t0, lane, a.rank, a.rp, a.norm_w, a.eps, put);
    for (int k = lane * 8; k < a.rotp; k += 512)
#pragma unroll
        for (int i = 0; i < R; ++i) {
            if (t0 + i >= a.T) continue;
            float v[8];
            la_ld8<E>(a.qc, (t0 + i) * a.ldq + a.c_off + a.rp + k, v);
            la_rotate8(v, a.cs + (t0 + i) * a.rotp + k);
            put(i, a.rp + k, v);
        }
}
template <typename E, int R>
__device__ void latent_query_rows(const PrepArgs& a, int64_t t0, int lane) {
    norm_rows<E, R>(a.qc, a.ldq, a.cq_off, a.T, t0, lane, a.cq_rank, a.cq_rp, a.cq_norm, a.eps,
                    [&](int i, int k, const float (&v)[8]) { la_st8<E>(a.cq_out, (t0 + i) * a.ld_cq + k, v); });
}

constexpr int PREP_TT = 4;  // 16-token tiles per absorb workgroup

// NR: tokens per wave of the norm's workgroups
template <int NR>
__global__ __launch_bounds__(256) void latent_prepare_kernel(const PrepArgs a, int n_absorb) {
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    if ((int)blockIdx.x >= n_absorb) {
        const int64_t t = ((int64_t)((int)blockIdx.x - n_absorb) * 4 + wid) * NR;
        if (t < a.T) latent_norm_rows<bf16_t, NR>(a, t, lane);
        return;
    }
    // q'[t, h, r] = sum_d W_uk[h, d, r] q[t, h, d]: 64 latent rows x 64 tokens per workgroup, 16 x 64 per wave
    const int nb = (a.rp + 63) / 64, nr = nb + (a.rotp > 0);
    int b = blockIdx.x;
    const int rb = b % nr;
    b /= nr;
    const int h = b % a.H;
    const int64_t t0 = (int64_t)(b / a.H) * (16 * PREP_TT);
    if (rb == nb) {  // the rotated part
        for (int i = tid; i < 16 * PREP_TT * (a.rotp / 8); i += 256) {
            const int64_t t = t0 + i / (a.rotp / 8);
            const int k = i % (a.rotp / 8) * 8;
            if (t >= a.Ta) continue;
            float v[8];
            la_ld8<bf16_t>(a.q, t * a.ldqq + (int64_t)h * a.hd + a.dimp + k, v);
            la_rotate8(v, a.cs + t * a.rotp + k);
            la_st8<bf16_t>(a.qa, (t * a.H + h) * a.rc + a.rp + k, v);
        }
        return;
    }
    const int c = lane & 15, g = lane >> 4;
    const int r0 = rb * 64 + wid * 16;
    const int ar = r0 + c;  // A row of this lane
    const bf16_t* q = reinterpret_cast<const bf16_t*>(a.q);
    f32x4_t acc[PREP_TT];
#pragma unroll
    for (int i = 0; i < PREP_TT; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int k = 8 * g; k < ((a.dimp + 31) & ~31); k += 32) {
        u32x4_t av = {0, 0, 0, 0};
        if (k < a.dimp && ar < a.rp) av = *reinterpret_cast<const u32x4_t*>(a.wukt + ((int64_t)h * a.rp + ar) * a.dimp + k);
#pragma unroll
        for (int i = 0; i < PREP_TT; ++i) {
            const int64_t t = t0 + 16 * i + c;
            u32x4_t bv = {0, 0, 0, 0};
            if (k < a.dimp && t < a.Ta) bv = *reinterpret_cast<const u32x4_t*>(q + t * a.ldqq + (int64_t)h * a.hd + k);
            acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, av), __builtin_bit_cast(bf16x8_t, bv), acc[i], 0, 0, 0);
        }
    }
    const int r = r0 + 4 * g;
    if (r < a.rp) {
#pragma unroll
        for (int i = 0; i < PREP_TT; ++i) {
            const int64_t t = t0 + 16 * i + c;
            if (t < a.Ta)
                *reinterpret_cast<u32x2_t*>(a.qa + (t * a.H + h) * a.rc + r) = u32x2_t{pack2bf(acc[i][0], acc[i][1]), pack2bf(acc[i][2], acc[i][3])};
        }
    }
}

// both latents' norms, the rotated key part and the cache store; blockIdx.y: key side, query side
template <typename E, int NR>
__global__ __launch_bounds__(256) void latent_rows_kernel(const PrepArgs a) {
    const int64_t t = ((int64_t)blockIdx.x * 4 + (threadIdx.x >> 6)) * NR;
    if (t >= a.T) return;
    if (blockIdx.y == 0) latent_norm_rows<E, NR>(a, t, threadIdx.x & 63);
    else latent_query_rows<E, NR>(a, t, threadIdx.x & 63);
}

// fp32: the rotated query part alone
__global__ __launch_bounds__(256) void latent_rotate_f32_kernel(const PrepArgs a) {
    const int n = a.rotp / 8;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x, th = i / n, t = th / a.H;
    const int k = (int)(i % n) * 8, h = (int)(th % a.H);
    if (t >= a.Ta) return;
    float v[8];
    la_ld8<float>(a.q, t * a.ldqq + (int64_t)h * a.hd + a.dimp + k, v);
    la_rotate8(v, a.cs + t * a.rotp + k);
    la_st8<float>(a.qa, th * a.rc + a.rp + k, v);
}

__global__ __launch_bounds__(256) void latent_norm_f32_kernel(const PrepArgs a) {
    const int64_t t = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t < a.T) latent_norm_rows<float, 1>(a, t, threadIdx.x & 63);
}

// cache rows -> contiguous rows (the history in front of a long portion): one wave per row, 16-byte chunks
__global__ __launch_bounds__(256) void latent_gather_kernel(const uint8_t* cache, int64_t n_slots, const int32_t* slots, const int32_t* rows, int64_t n,
                                                            uint8_t* out, int64_t n_rows, int row_bytes) {
    const int64_t i = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (i >= n) return;
    const int64_t s = slots[i], r = rows[i];
    if (s < 0 || s >= n_slots || r < 0 || r >= n_rows) return;
    for (int o = (threadIdx.x & 63) * 16; o < row_bytes; o += 1024)
        *reinterpret_cast<u32x4_t*>(out + r * row_bytes + o) = *reinterpret_cast<const u32x4_t*>(cache + s * row_bytes + o);
}

// ---------------------------------------------------------------------------------------------------------------------------
struct AttnArgs {
    const void* qa;           // [Ta, H, rp]
    const void* cache;        // [n_blocks, block_size, rp]
    const int32_t *tile_tok, *tile_n;  // [n_tiles] first row and row count of a tile (one sequence)
    const int32_t *pos, *seq_of;       // [T]
    const int32_t* bt;        // [S, bt_stride]
    int64_t bt_stride;
    int64_t n_blocks;
    int bs_shift;             // log2(block size)
    int64_t Ta;
    int H, rp, vp, window;      // rp: columns of a cache row (scores), the first vp of them are the values
    float scale;
    const float* sink;        // [H]
    int n_tiles, hb, n_hg, tq, nsplit;  // heads per workgroup, head groups, tokens per tile (at most)
    bf16_t* ctx;              // nsplit == 1: [Ta, H, vp] normalised context
    float* part_o;            // nsplit > 1: [Ta * H, nsplit, vp] unnormalised
    float* part_ml;           // [Ta * H, nsplit, 2] running maximum (log2 units), mass
};

// One wave per (16-row query tile, 16-key quarter of a 64-key tile): it computes those scores over the whole latent, their
// weights, and hands them over through LDS; then the waves divide the latent's columns among themselves for O^T += C^T . P^T.
template <int NCT, int MT>
struct LaCfg {
    static constexpr int NW = 4 * MT, NT = 64 * NW;           // waves, threads
    static constexpr int TILEB = 64 * NCT * 128;
    static constexpr int NST = 2 * TILEB <= 144 * 1024 ? 2 : 1;
    static constexpr int DPW = (4 * NCT + NW - 1) / NW;       // 16-column tiles of the latent per wave
    static constexpr int PB = MT * 2048, MB = MT * 256;       // weights (bf16), row maxima
    static constexpr int LDS = NST * TILEB + PB + MB + 16 + LA_BT * 4;
    static_assert(LDS <= 160 * 1024, "LDS of a CU");
};

template <int NCT, int MT>
__global__ __launch_bounds__(64 * 4 * MT) void latent_attn_kernel(const AttnArgs a) {
    using C = LaCfg<NCT, MT>;
    constexpr int RPAD = NCT * 64, ROWB = RPAD * 2, TILEB = C::TILEB, CPR = RPAD / 8, NST = C::NST, NW = C::NW, DPW = C::DPW, NT = C::NT;
    constexpr int KS = 2 * NCT, NDMA = 8 * NCT, DMAW = (NDMA + NW - 1) / NW;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    const int tid = threadIdx.x, lane = tid & 63;
    const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 15, g = lane >> 4;
    const int kt = w & 3, mw = w >> 2;  // key quarter and row tile of this wave's scores
    int id = blockIdx.x;
    const int split = id % a.nsplit;
    id /= a.nsplit;
    const int hg = id % a.n_hg, tile = id / a.n_hg;
    const int h0 = hg * a.hb, hb = min(a.hb, a.H - h0);
    const int tok0 = a.tile_tok[tile];
    const int ntok = min(a.tile_n[tile], a.tq);
    if (tok0 < 0 || tok0 >= a.Ta || ntok <= 0) return;
    const int p0 = a.pos[tok0], p1 = p0 + ntok - 1, seq = a.seq_of[tok0];
    const int nrows = ntok * hb;
    // tiles start at multiples of 64: a tile lies in one cache block (its halves in one each, with blocks of 32); what is in front
    // of the first visible key or behind the last row's comes from the zero page
    const int first = max(0, p0 - a.window + 1), lo = first & ~63;
    const int ntile = p0 < 0 ? 0 : (p1 - lo + 64) >> 6;  // 64-key tiles of the whole range
    const int per = (ntile + a.nsplit - 1) / a.nsplit;
    const int t0 = split * per, t1 = min(t0 + per, ntile), n = t1 - t0;
    if (n <= 0) {  // an empty split (or an unused row): no mass
        for (int r = tid; r < nrows; r += NT) {
            const int64_t gr = (int64_t)(tok0 + r / hb) * a.H + h0 + r % hb;
            if (a.nsplit > 1) {
                a.part_ml[(gr * a.nsplit + split) * 2] = -INFINITY;
                a.part_ml[(gr * a.nsplit + split) * 2 + 1] = 0.f;
            } else {
                for (int d = 0; d < a.vp; ++d) a.ctx[gr * a.vp + d] = 0;
            }
        }
        return;
    }
    const int bmask = (1 << a.bs_shift) - 1;
    const int klo = lo + t0 * 64;                 // first key of this split
    const int khi = min(p1, lo + t1 * 64 - 1);    // last key of this split
    const int blk0 = klo >> a.bs_shift, nblk = (khi >> a.bs_shift) - blk0 + 1;
    char* aux = smem + NST * TILEB;
    int* flags = reinterpret_cast<int*>(aux + C::PB + C::MB);
    int* bt_lds = flags + 4;
    // (entries of blocks in front of the window may have been given back, -1: no key of theirs is fetched)
    for (int i = tid; i < min(nblk, LA_BT); i += NT) {
        const int64_t b = a.bt[(int64_t)seq * a.bt_stride + blk0 + i];
        bt_lds[i] = (int)min(max(b, (int64_t)0), a.n_blocks - 1);
    }
    if (tid < 4) flags[tid] = 0;
    // this wave's query rows: row 16 mw + c
    const int r_own = 16 * mw + c;
    const bool own = r_own < nrows;
    const int rpos = own ? p0 + r_own / hb : -1;
    u32x4_t qf[KS];
    {
        const bf16_t* q = reinterpret_cast<const bf16_t*>(a.qa) + ((int64_t)(tok0 + (own ? r_own / hb : 0)) * a.H + h0 + (own ? r_own % hb : 0)) * a.rp;
#pragma unroll
        for (int i = 0; i < KS; ++i) {
            const int k = 32 * i + 8 * g;
            qf[i] = u32x4_t{0, 0, 0, 0};
            if (own && k < a.rp) qf[i] = *reinterpret_cast<const u32x4_t*>(q + k);
        }
    }
    __syncthreads();
    const unsigned base = lds_addr(smem), p_addr = base + NST * TILEB, m_addr = p_addr + C::PB, f_addr = m_addr + C::MB, bt_addr = f_addr + 16;
    const bf16_t* cache = reinterpret_cast<const bf16_t*>(a.cache);
    // per-lane source offsets (elements) of the DMA pieces inside a tile: constant over the tiles
    unsigned off[DMAW];
    int orow[DMAW];
    const bool padded = RPAD != a.rp;
#pragma unroll
    for (int i = 0; i < DMAW; ++i) {
        const int q = (i * NW + w) * 64 + lane, row = q / CPR, ch = (q % CPR) ^ attn_swz(row);
        orow[i] = (padded && ch * 8 >= a.rp) ? 1 << 30 : row;
        off[i] = (unsigned)((row & 31) * a.rp + ch * 8);
    }
    auto issue = [&](int it) {
        const int k0 = klo + it * 64;
        int b0, b1;
        const int i0 = (k0 >> a.bs_shift) - blk0, i1 = min(((k0 + 32) >> a.bs_shift) - blk0, nblk - 1);
        asm volatile("ds_read_b32 %0, %2\n\tds_read_b32 %1, %3\n\ts_waitcnt lgkmcnt(0)" : "=&v"(b0), "=&v"(b1) : "v"(bt_addr + i0 * 4), "v"(bt_addr + i1 * 4) : "memory");
        const bf16_t* s0 = cache + (((int64_t)__builtin_amdgcn_readfirstlane(b0) << a.bs_shift) + (k0 & bmask)) * a.rp;
        const bf16_t* s1 = cache + (((int64_t)__builtin_amdgcn_readfirstlane(b1) << a.bs_shift) + ((k0 + 32) & bmask)) * a.rp;
        char* st = smem + (NST == 2 ? (it & 1) * TILEB : 0);
        const int left = khi - k0, skip = first - k0;
        const bool plain = left >= 63 && skip <= 0 && !padded;
#pragma unroll
        for (int i = 0; i < DMAW; ++i) {
            const int piece = i * NW + w;
            if (NDMA % NW != 0 && piece >= NDMA) continue;
            const int row = orow[i];
            const bf16_t* src = (((piece * 64 + lane) / CPR) & 32 ? s1 : s0) + off[i];
            lds_dma16<2>(plain || (row <= left && row >= skip) ? (const void*)src : (const void*)la_zero_page, st + piece * 1024);
        }
    };
    f32x4_t acc[MT][DPW];
    float m_run[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        m_run[m] = -INFINITY;
#pragma unroll
        for (int d = 0; d < DPW; ++d) acc[m][d] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
    float m_own = -INFINITY, l_own = 0.f;
    // loop-invariant LDS offsets of this lane's fragment reads
    unsigned k_rel[2];
#pragma unroll
    for (int e = 0; e < 2; ++e) k_rel[e] = (16 * kt + c) * ROWB + (((4 * e + g) ^ attn_swz(c)) << 4);
    const int qq = (lane >> 2) & 3, pp = lane & 3, vrow = 4 * g + qq;
    // latent tile d of this wave: d NW + w = 4 (d MT + (w >> 2)) + (w & 3)
    const unsigned v_rel = vrow * ROWB + (((2 * (w & 3) + (pp >> 1)) ^ attn_swz(vrow)) << 4) + ((pp & 1) << 3) + (w >> 2) * 128;
    const bool last_v = (DPW - 1) * NW * 16 < a.vp;  // this wave's last column tile may hold values
    const float sc = a.scale * LOG2E;
#pragma unroll
    for (int i = 0; i < KS; ++i) asm volatile("" : "+v"(qf[i]));  // landed before the DMAs are counted
    issue(0);
    for (int it = 0; it < n; ++it) {
        wait_vm<0>();
        __builtin_amdgcn_s_barrier();
        if (NST == 2 && it + 1 < n) issue(it + 1);
        if (tid == 0) asm volatile("ds_write_b32 %0, %1" ::"v"(f_addr + ((it + 1) & 1) * 4), "v"(0) : "memory");
        const unsigned st = base + (NST == 2 ? (it & 1) * TILEB : 0);
        // ---- scores of 16 keys x 16 rows over the whole latent, two accumulation chains ----
        f32x4_t s2[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
        constexpr int FG = MT == 4 ? 4 : 8;  // fragments per request group
        static_for<(KS + FG - 1) / FG>([&](auto G) {
            constexpr int i0 = decltype(G)::value * FG, ni = KS - i0 < FG ? KS - i0 : FG;
            u32x4_t kf[FG];
            static_for<ni>([&](auto I) { constexpr int i = i0 + decltype(I)::value; lds_read_b128<(i >> 1) * 128>(kf[i - i0], st + k_rel[i & 1]); });
            wait_lds();
#pragma unroll
            for (int i = 0; i < ni; ++i) asm volatile("" : "+v"(kf[i]));
#pragma unroll
            for (int i = 0; i < ni; ++i)
                s2[i & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kf[i]), __builtin_bit_cast(bf16x8_t, qf[i0 + i]), s2[i & 1], 0, 0, 0);
        });
        // ---- softmax of row c: this lane holds keys 16 kt + 4 g + r ----
        const int key0 = klo + it * 64;
        float x[4], mx = -INFINITY;
        if (key0 > p1 - a.window && key0 + 63 <= p0) {  // every row sees every key
#pragma unroll
            for (int r = 0; r < 4; ++r) x[r] = (s2[0][r] + s2[1][r]) * sc;
        } else {
            const int d0 = rpos - (key0 + 16 * kt + 4 * g);
#pragma unroll
            for (int r = 0; r < 4; ++r) x[r] = (rpos >= 0 && d0 - r >= 0 && d0 - r < a.window) ? (s2[0][r] + s2[1][r]) * sc : -INFINITY;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) mx = fmaxf(mx, x[r]);
        // The reference point of a row is raised only when a score exceeds it by more than 2^8 (it cancels in the end).  The
        // weights are formed against the reference as it is; if any row of the workgroup needs a higher one, all waves see the
        // flag behind the barrier, agree on new references and form the weights again.
        auto weights = [&]() {
            const float m_use = m_own == -INFINITY ? 0.f : m_own;
            float p[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) p[r] = __builtin_amdgcn_exp2f(x[r] - m_use);
            const u32x2_t v = {pack2bf(p[0], p[1]), pack2bf(p[2], p[3])};
            asm volatile("ds_write_b64 %0, %1" ::"v"(p_addr + ((mw * 2 + (kt >> 1)) * 64 + lane) * 16 + (kt & 1) * 8), "v"(v) : "memory");
            return (p[0] + p[1]) + (p[2] + p[3]);
        };
        float lp = weights();
        if (__any(mx > m_own + 8.0f || (m_own == -INFINITY && mx > -INFINITY))) asm volatile("ds_write_b32 %0, %1" ::"v"(f_addr + (it & 1) * 4), "v"(1) : "memory");
        wait_lds();
        __builtin_amdgcn_s_barrier();
        int raise;
        asm volatile("ds_read_b32 %0, %1\n\ts_waitcnt lgkmcnt(0)" : "=v"(raise) : "v"(f_addr + (it & 1) * 4) : "memory");
        if (__builtin_amdgcn_readfirstlane(raise)) {
            mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
            mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
            if (g == 0) asm volatile("ds_write_b32 %0, %1" ::"v"(m_addr + (mw * 16 + c) * 16 + kt * 4), "v"(mx) : "memory");
            wait_lds();
            __builtin_amdgcn_s_barrier();
#pragma unroll
            for (int m = 0; m < MT; ++m) {
                f32x4_t q4;
                asm volatile("ds_read_b128 %0, %1\n\ts_waitcnt lgkmcnt(0)" : "=v"(q4) : "v"(m_addr + (m * 16 + c) * 16) : "memory");
                const float m_new = fmaxf(m_run[m], fmaxf(fmaxf(q4[0], q4[1]), fmaxf(q4[2], q4[3])));
                const float alpha = m_new == -INFINITY ? 1.0f : __builtin_amdgcn_exp2f(m_run[m] - m_new);
#pragma unroll
                for (int d = 0; d < DPW; ++d) acc[m][d] *= alpha;
                m_run[m] = m_new;
                if (m == mw) {
                    l_own *= alpha;
                    m_own = m_new;
                }
            }
            lp = weights();
            wait_lds();
            __builtin_amdgcn_s_barrier();
        }
        l_own += lp;
        // ---- O^T += C^T . P^T on this wave's latent columns, 32 keys at a time ----
#pragma unroll
        for (int k2 = 0; k2 < 2; ++k2) {
            u32x4_t pf[MT];
#pragma unroll
            for (int m = 0; m < MT; ++m) asm volatile("ds_read_b128 %0, %1" : "=v"(pf[m]) : "v"(p_addr + ((m * 2 + k2) * 64 + lane) * 16));
            const unsigned va = st + v_rel + k2 * 32 * ROWB;
            static_for<(DPW + FG - 1) / FG>([&](auto G) {
                constexpr int d0 = decltype(G)::value * FG, nd = DPW - d0 < FG ? DPW - d0 : FG;
                u32x2_t vf[FG][2];
                static_for<nd>([&](auto I) {
                    constexpr int d = d0 + decltype(I)::value;
                    if ((4 * NCT % NW == 0 || d * NW + w < 4 * NCT) && (d + 1 < DPW || last_v)) {
                        lds_read_tr16_b64<d * MT * 128>(vf[d - d0][0], va);
                        lds_read_tr16_b64<d * MT * 128>(vf[d - d0][1], va + 16 * ROWB);
                    }
                });
                wait_lds();
#pragma unroll
                for (int m = 0; m < MT; ++m) asm volatile("" : "+v"(pf[m]));
#pragma unroll
                for (int d = 0; d < nd; ++d) asm volatile("" : "+v"(vf[d][0]), "+v"(vf[d][1]));
#pragma unroll
                for (int d = 0; d < nd; ++d) {
                    const u32x4_t vv = {vf[d][0][0], vf[d][0][1], vf[d][1][0], vf[d][1][1]};
                    if ((4 * NCT % NW == 0 || (d0 + d) * NW + w < 4 * NCT) && (d0 + d + 1 < DPW || last_v)) {
#pragma unroll
                        for (int m = 0; m < MT; ++m)
                            acc[m][d0 + d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, vv), __builtin_bit_cast(bf16x8_t, pf[m]), acc[m][d0 + d], 0, 0, 0);
                    }
                }
            });
        }
        if (NST == 1 && it + 1 < n) {
            __builtin_amdgcn_s_barrier();
            issue(it + 1);
        }
    }
    // ---- masses of the four key quarters meet in LDS ----
    l_own += __shfl_xor(l_own, 16, 64);
    l_own += __shfl_xor(l_own, 32, 64);
    if (g == 0) asm volatile("ds_write_b32 %0, %1" ::"v"(m_addr + (mw * 16 + c) * 16 + kt * 4), "v"(l_own) : "memory");
    wait_lds();
    __builtin_amdgcn_s_barrier();
    // ---- rows out: lane holds latent columns 16 (d NW + w) + 4 g .. of row c of every row tile ----
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        f32x4_t q4;
        asm volatile("ds_read_b128 %0, %1\n\ts_waitcnt lgkmcnt(0)" : "=v"(q4) : "v"(m_addr + (m * 16 + c) * 16) : "memory");
        const float l = (q4[0] + q4[1]) + (q4[2] + q4[3]);
        const int r = 16 * m + c;
        if (r >= nrows) continue;
        const int hd = h0 + r % hb;
        const int64_t gr = (int64_t)(tok0 + r / hb) * a.H + hd;
        if (a.nsplit == 1) {
            const float sk = a.sink[hd] * LOG2E;
            const float M = fmaxf(m_run[m], sk);
            const float f = __builtin_amdgcn_exp2f(m_run[m] - M);
            const float inv = f / (l * f + __builtin_amdgcn_exp2f(sk - M));
#pragma unroll
            for (int d = 0; d < DPW; ++d) {
                const int dim = 16 * (d * NW + w) + 4 * g;
                if (dim < a.vp)
                    *reinterpret_cast<u32x2_t*>(a.ctx + gr * a.vp + dim) = u32x2_t{pack2bf(acc[m][d][0] * inv, acc[m][d][1] * inv), pack2bf(acc[m][d][2] * inv, acc[m][d][3] * inv)};
            }
        } else {
            const int64_t pr = gr * a.nsplit + split;
#pragma unroll
            for (int d = 0; d < DPW; ++d) {
                const int dim = 16 * (d * NW + w) + 4 * g;
                if (dim < a.vp) *reinterpret_cast<f32x4_t*>(a.part_o + pr * a.vp + dim) = acc[m][d];
            }
            if (w == 0 && g == 0) {
                a.part_ml[pr * 2] = m_run[m];
                a.part_ml[pr * 2 + 1] = l;
            }
        }
    }
}

template <int NCT, int MT>
int launch_latent_attn(const AttnArgs& a, hipStream_t st) {
    using C = LaCfg<NCT, MT>;
    auto kern = latent_attn_kernel<NCT, MT>;
    GLM_SET_MAX_LDS(kern, C::LDS, "glm_latent_attn");
    const int64_t grid = (int64_t)a.n_tiles * a.n_hg * a.nsplit;
    GLM_CHECK_ARG(grid < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_latent_attn: grid too large");
    hipLaunchKernelGGL(kern, dim3((unsigned)grid), dim3(C::NT), C::LDS, st, a);
    GLM_CHECK_LAUNCH("glm_latent_attn");
    return GLM_OK;
}

// most query rows per workgroup (16 MT) whose fragments and sums the registers hold
constexpr int la_max_rows(int nct) { return nct > 9 ? 16 : nct > 4 ? 32 : 64; }

template <int NCT>
int launch_latent_attn_mt(const AttnArgs& a, int mt, hipStream_t st) {
    if constexpr (la_max_rows(NCT) >= 64) {
        if (mt > 2) return launch_latent_attn<NCT, 4>(a, st);
    }
    if constexpr (la_max_rows(NCT) >= 32) {
        if (mt > 1) return launch_latent_attn<NCT, 2>(a, st);
    }
    return launch_latent_attn<NCT, 1>(a, st);
}

// ---------------------------------------------------------------------------------------------------------------------------
// fp32: one wave per (token, head), 64 keys per step (one per lane), then the latent dimensions over the lanes
constexpr int LF_MAXR = 2048;

template <int NV>  // latent values per lane
__global__ __launch_bounds__(256) void latent_attn_f32_kernel(const AttnArgs a, float* ctx) {
    extern __shared__ __attribute__((aligned(16))) float sq[];  // [4][rp]
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int64_t grow = (int64_t)blockIdx.x * 4 + wid;
    const bool live = grow < a.Ta * a.H;
    const int64_t t = live ? grow / a.H : 0;
    const int h = live ? (int)(grow % a.H) : 0;
    const int p = a.pos[t];
    float* q = sq + wid * a.rp;
    const float* qa = reinterpret_cast<const float*>(a.qa) + (t * a.H + h) * a.rp;
    for (int i = lane; i < a.rp; i += 64) q[i] = qa[i];
    __syncthreads();
    if (!live) return;
    float acc[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) acc[i] = 0.f;
    float m = a.sink[h], l = 1.0f;  // the sink's mass is in from the start
    const int lo = max(0, p - a.window + 1);
    const int32_t* bt = a.bt + (int64_t)a.seq_of[t] * a.bt_stride;
    const float* cache = reinterpret_cast<const float*>(a.cache);
    const int bs = 1 << a.bs_shift;
    for (int k0 = lo; k0 <= p; k0 += 64) {
        const int key = k0 + lane;
        int64_t row = 0;
        float s = -INFINITY;
        if (key <= p) {
            const int64_t b = min(max((int64_t)bt[key >> a.bs_shift], (int64_t)0), a.n_blocks - 1);
            row = (b << a.bs_shift) + (key & (bs - 1));
            const float* cr = cache + row * a.rp;
            float d = 0.f;
            for (int i = 0; i < a.rp; i += 4) {
                const f32x4_t cv = *reinterpret_cast<const f32x4_t*>(cr + i), qv = *reinterpret_cast<const f32x4_t*>(q + i);
                d = fmaf(cv[0], qv[0], d);
                d = fmaf(cv[1], qv[1], d);
                d = fmaf(cv[2], qv[2], d);
                d = fmaf(cv[3], qv[3], d);
            }
            s = d * a.scale;
        }
        const float m_new = fmaxf(m, wave_max(s));
        const float alpha = expf(m - m_new);
        const float pv = key <= p ? expf(s - m_new) : 0.f;
        l = l * alpha + wave_sum(pv);
#pragma unroll
        for (int i = 0; i < NV; ++i) acc[i] *= alpha;
        m = m_new;
        const int nk = min(64, p - k0 + 1);
        for (int k = 0; k < nk; ++k) {
            const float pk = __shfl(pv, k, 64);
            const int64_t rk = __shfl((long long)row, k, 64);
#pragma unroll
            for (int i = 0; i < NV; ++i)
                if (lane + 64 * i < a.vp) acc[i] = fmaf(pk, cache[rk * a.rp + lane + 64 * i], acc[i]);
        }
    }
    const float inv = 1.0f / l;
#pragma unroll
    for (int i = 0; i < NV; ++i)
        if (lane + 64 * i < a.vp) ctx[grow * a.vp + lane + 64 * i] = p < 0 ? 0.f : acc[i] * inv;
}

struct UpArgs {
    const bf16_t* ctx;   // [Ta, H, rp]
    const bf16_t* wuv;   // [H, vdimp, rp]
    bf16_t* out;         // [T, ldo], head h at h*vdimp
    const bf16_t* gate;  // [T, ldg] laid out like out: factors of the rows, or nullptr
    int64_t ldg;
    int64_t ldo, Ta;
    int H, vdimp, rp;
};

// out[t, h, :] = W_uv[h] . ctx[t, h, :]: per wave 16 tokens and 16 value rows of one head, operands straight from memory, eight
// K steps of both in flight
__global__ __launch_bounds__(256) void latent_up_kernel(const UpArgs a) {
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int c = lane & 15, g = lane >> 4;
    const int nv = (a.vdimp + 15) / 16;
    const int item = blockIdx.x * 4 + wid;
    if (item >= a.H * nv) return;
    const int h = item / nv, v0 = (item % nv) * 16;
    const int64_t t = (int64_t)blockIdx.y * 16 + c;
    const bf16_t* wr = a.wuv + ((int64_t)h * a.vdimp + min(v0 + c, a.vdimp - 1)) * a.rp;
    const bf16_t* xr = a.ctx + (min(t, a.Ta - 1) * a.H + h) * a.rp;
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < a.rp; k0 += 256) {
        u32x4_t av[8], bv[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const int k = k0 + 32 * i + 8 * g;
            const bool ok = k < a.rp;
            av[i] = *reinterpret_cast<const u32x4_t*>(wr + (ok ? k : 0));
            bv[i] = *reinterpret_cast<const u32x4_t*>(xr + (ok ? k : 0));
            if (!ok) av[i] = bv[i] = u32x4_t{0, 0, 0, 0};
        }
#pragma unroll
        for (int i = 0; i < 8; ++i)
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, av[i]), __builtin_bit_cast(bf16x8_t, bv[i]), acc, 0, 0, 0);
    }
    const int v = v0 + 4 * g;
    if (a.gate && t < a.Ta && v < a.vdimp) {
        const u32x2_t gt = *reinterpret_cast<const u32x2_t*>(a.gate + t * a.ldg + (int64_t)h * a.vdimp + v);
        acc *= f32x4_t{bflo(gt[0]), bfhi(gt[0]), bflo(gt[1]), bfhi(gt[1])};
    }
    if (t < a.Ta && v < a.vdimp)
        *reinterpret_cast<u32x2_t*>(a.out + t * a.ldo + (int64_t)h * a.vdimp + v) = u32x2_t{pack2bf(acc[0], acc[1]), pack2bf(acc[2], acc[3])};
}

int pick_nct(int rp) {
    for (int n : {1, 2, 3, 4, 6, 8, 9, 16})
        if (rp <= 64 * n) return n;
    return -1;
}

}  // namespace

extern "C" int glm_latent_prepare(const void* qc, int64_t ldq, int c_off, int64_t T, int64_t Ta, int H, int dimp, int rank, int rp, const float* norm_w,
                                  float eps, const int32_t* slots, void* cache, int64_t n_slots, const int32_t* crow, void* c_out, int64_t n_crows,
                                  const void* wukt, void* qa, int act_f32, glm_stream_t stream) {
    GLM_CHECK_ARG(qc && norm_w && slots && cache && T >= 0 && Ta >= 0 && Ta <= T && H > 0 && rank > 0 && rp >= rank && rp % 8 == 0 && c_off % 8 == 0 &&
                      ldq % 8 == 0 && ldq >= (int64_t)c_off + rank && dimp % 8 == 0 && c_off >= H * dimp && n_slots > 0 && (!crow || (c_out && n_crows > 0)),
                  GLM_ERR_INVALID, "glm_latent_prepare: bad shape T=%ld Ta=%ld H=%d dimp=%d rank=%d", (long)T, (long)Ta, H, dimp, rank);
    GLM_CHECK_ARG(act_f32 || Ta == 0 || (wukt && qa && glm_aligned16(wukt) && glm_aligned16(qc)), GLM_ERR_INVALID, "glm_latent_prepare: absorbed rows need W_uk^T and q'");
    if (T == 0) return GLM_OK;
    PrepArgs a = {};
    a.q = a.qc = qc; a.ldqq = a.ldq = ldq; a.hd = dimp; a.c_off = c_off;
    a.T = T; a.Ta = Ta; a.H = H; a.dimp = dimp; a.rank = rank; a.rp = a.rc = rp;
    a.norm_w = norm_w; a.eps = eps; a.slots = slots; a.cache = cache; a.n_slots = n_slots; a.crow = crow; a.c_out = c_out; a.n_crows = n_crows;
    a.wukt = (const bf16_t*)wukt; a.qa = (bf16_t*)qa;
    const bool many = !act_f32 && T >= 2048;
    const int64_t nnorm = many ? (T + 15) / 16 : (T + 3) / 4;
    if (act_f32) {
        hipLaunchKernelGGL(latent_norm_f32_kernel, dim3((unsigned)nnorm), dim3(256), 0, glm_s(stream), a);
    } else {
        const int64_t nabs = Ta > 0 ? (int64_t)((rp + 63) / 64) * H * ((Ta + 16 * PREP_TT - 1) / (16 * PREP_TT)) : 0;
        GLM_CHECK_ARG(nabs + nnorm < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_latent_prepare: grid too large");
        if (many) hipLaunchKernelGGL(latent_prepare_kernel<4>, dim3((unsigned)(nabs + nnorm)), dim3(256), 0, glm_s(stream), a, (int)nabs);
        else hipLaunchKernelGGL(latent_prepare_kernel<1>, dim3((unsigned)(nabs + nnorm)), dim3(256), 0, glm_s(stream), a, (int)nabs);
    }
    GLM_CHECK_LAUNCH("glm_latent_prepare");
    return GLM_OK;
}

extern "C" int glm_latent_rows(const void* qc, int64_t ldq, int c_off, int rank, int rp, int rotp, const float* norm_w, const float* cs, float eps, const int32_t* slots, void* cache,
                               int64_t n_slots, const int32_t* crow, void* c_out, int64_t n_crows, int cq_off, int cq_rank, int cq_rp, const float* cq_norm, void* cq_out,
                               int64_t ld_cq, int64_t T, int act_f32, glm_stream_t stream) {
    GLM_CHECK_ARG(qc && norm_w && slots && cache && T >= 0 && rank > 0 && rp >= rank && rp % 8 == 0 && rotp >= 0 && rotp % 8 == 0 && (rotp == 0 || cs) && c_off >= 0 && c_off % 8 == 0 &&
                      ldq % 8 == 0 && ldq >= (int64_t)c_off + rp + rotp && n_slots > 0 && (!crow || (c_out && n_crows > 0)) && glm_aligned16(qc) && glm_aligned16(cache), GLM_ERR_INVALID,
                  "glm_latent_rows: bad shape T=%ld rank=%d rot=%d", (long)T, rank, rotp);
    GLM_CHECK_ARG(!cq_out || (cq_norm && cq_off >= 0 && cq_off % 8 == 0 && cq_rank > 0 && cq_rp >= cq_rank && cq_rp % 8 == 0 && ldq >= (int64_t)cq_off + cq_rp && ld_cq >= cq_rp &&
                              ld_cq % 8 == 0 && glm_aligned16(cq_out)), GLM_ERR_INVALID, "glm_latent_rows: bad query latent of %d columns", cq_rank);
    if (T == 0) return GLM_OK;
    PrepArgs a = {};
    a.qc = qc; a.ldq = ldq; a.c_off = c_off; a.T = T; a.rank = rank; a.rp = rp; a.rotp = rotp; a.rc = rp + rotp; a.cs = cs;
    a.norm_w = norm_w; a.eps = eps; a.slots = slots; a.cache = cache; a.n_slots = n_slots; a.crow = crow; a.c_out = c_out; a.n_crows = n_crows;
    a.cq_off = cq_off; a.cq_rank = cq_rank; a.cq_rp = cq_rp; a.cq_norm = cq_norm; a.cq_out = cq_out; a.ld_cq = ld_cq;
    const int nr = !act_f32 && T >= 2048 ? 4 : 1;
    const dim3 grid((unsigned)((T + 4 * nr - 1) / (4 * nr)), cq_out ? 2 : 1);
    if (act_f32) hipLaunchKernelGGL((latent_rows_kernel<float, 1>), grid, dim3(256), 0, glm_s(stream), a);
    else if (nr == 4) hipLaunchKernelGGL((latent_rows_kernel<bf16_t, 4>), grid, dim3(256), 0, glm_s(stream), a);
    else hipLaunchKernelGGL((latent_rows_kernel<bf16_t, 1>), grid, dim3(256), 0, glm_s(stream), a);
    GLM_CHECK_LAUNCH("glm_latent_rows");
    return GLM_OK;
}

extern "C" int glm_latent_absorb(const void* q, int64_t ldq, int64_t Ta, int H, int dimp, int rp, int rotp, const float* cs, const void* wukt, void* qa, int act_f32,
                                 glm_stream_t stream) {
    GLM_CHECK_ARG(q && qa && Ta >= 0 && H > 0 && dimp > 0 && dimp % 8 == 0 && rp > 0 && rp % 8 == 0 && rotp >= 0 && rotp % 8 == 0 && (rotp == 0 || cs) && ldq % 8 == 0 &&
                      ldq >= (int64_t)H * (dimp + rotp) && (act_f32 || (wukt && glm_aligned16(wukt))) && glm_aligned16(q) && glm_aligned16(qa), GLM_ERR_INVALID,
                  "glm_latent_absorb: bad shape Ta=%ld H=%d dimp=%d", (long)Ta, H, dimp);
    if (Ta == 0 || (act_f32 && rotp == 0)) return GLM_OK;
    PrepArgs a = {};
    a.q = q; a.ldqq = ldq; a.hd = dimp + rotp; a.T = Ta; a.Ta = Ta; a.H = H; a.dimp = dimp; a.rank = a.rp = rp; a.rotp = rotp; a.rc = rp + rotp; a.cs = cs;
    a.wukt = (const bf16_t*)wukt; a.qa = (bf16_t*)qa;
    const int64_t nb = act_f32 ? (Ta * H * (rotp / 8) + 255) / 256 : (int64_t)((rp + 63) / 64 + (rotp > 0)) * H * ((Ta + 16 * PREP_TT - 1) / (16 * PREP_TT));
    GLM_CHECK_ARG(nb < (1ll << 31), GLM_ERR_UNSUPPORTED, "glm_latent_absorb: grid too large");
    if (act_f32) hipLaunchKernelGGL(latent_rotate_f32_kernel, dim3((unsigned)nb), dim3(256), 0, glm_s(stream), a);
    else hipLaunchKernelGGL(latent_prepare_kernel<1>, dim3((unsigned)nb), dim3(256), 0, glm_s(stream), a, (int)nb);
    GLM_CHECK_LAUNCH("glm_latent_absorb");
    return GLM_OK;
}

extern "C" int glm_latent_gather(const void* cache, int64_t n_slots, const int32_t* slots, const int32_t* rows, int64_t n, void* out, int64_t n_rows,
                                 int row_bytes, glm_stream_t stream) {
    GLM_CHECK_ARG(cache && slots && rows && out && n >= 0 && row_bytes > 0 && row_bytes % 16 == 0 && glm_aligned16(cache) && glm_aligned16(out), GLM_ERR_INVALID,
                  "glm_latent_gather: bad arguments (n=%ld row_bytes=%d)", (long)n, row_bytes);
    if (n == 0) return GLM_OK;
    hipLaunchKernelGGL(latent_gather_kernel, dim3((unsigned)((n + 3) / 4)), dim3(256), 0, glm_s(stream), (const uint8_t*)cache, n_slots, slots, rows, n,
                       (uint8_t*)out, n_rows, row_bytes);
    GLM_CHECK_LAUNCH("glm_latent_gather");
    return GLM_OK;
}

// query rows (tokens x heads) per tile the absorbed kernel takes for a latent of rp columns: 16, 32 or 64
extern "C" int glm_latent_attn_max_rows(int rp) {
    const int n = pick_nct(rp);
    return n < 0 ? 0 : la_max_rows(n);
}

extern "C" int glm_latent_attn(const void* qa, const void* cache, int64_t n_blocks, int block_size, const int32_t* tile_tok, const int32_t* tile_n,
                               int n_tiles, int tokens_per_tile, const int32_t* pos, const int32_t* seq_of, const int32_t* block_tables, int64_t bt_stride,
                               int64_t Ta, int H, int rp, int vp, int window, float scale, const float* sink, int nsplit, void* ctx, float* part_o,
                               float* part_ml, int act_f32, glm_stream_t stream) {
    GLM_CHECK_ARG(qa && cache && pos && seq_of && block_tables && sink && n_blocks > 0 && Ta >= 0 && H > 0 && vp > 0 && rp >= vp && rp % 8 == 0 && vp % 8 == 0 && window > 0 &&
                      bt_stride > 0, GLM_ERR_INVALID, "glm_latent_attn: bad shape Ta=%ld H=%d rp=%d window=%d", (long)Ta, H, rp, window);
    int sh = 0;
    while ((1 << sh) < block_size) ++sh;
    GLM_CHECK_ARG((1 << sh) == block_size && block_size >= 32, GLM_ERR_UNSUPPORTED, "glm_latent_attn: block size %d is not a power of two >= 32", block_size);
    if (Ta == 0) return GLM_OK;
    AttnArgs a = {qa, cache, tile_tok, tile_n, pos, seq_of, block_tables, bt_stride, n_blocks, sh, Ta, H, rp, vp, window, scale, sink,
                  n_tiles, 0, 0, tokens_per_tile, nsplit, (bf16_t*)ctx, part_o, part_ml};
    hipStream_t st = glm_s(stream);
    if (act_f32) {
        GLM_CHECK_ARG(ctx && rp <= LF_MAXR, GLM_ERR_UNSUPPORTED, "glm_latent_attn(fp32): latent of %d columns", rp);
        const int64_t nb = (Ta * H + 3) / 4;
        const size_t lds = (size_t)4 * rp * 4;
        if (rp <= 128) hipLaunchKernelGGL(latent_attn_f32_kernel<2>, dim3((unsigned)nb), dim3(256), lds, st, a, (float*)ctx);
        else if (rp <= 512) hipLaunchKernelGGL(latent_attn_f32_kernel<8>, dim3((unsigned)nb), dim3(256), lds, st, a, (float*)ctx);
        else hipLaunchKernelGGL(latent_attn_f32_kernel<32>, dim3((unsigned)nb), dim3(256), lds, st, a, (float*)ctx);
        GLM_CHECK_LAUNCH("glm_latent_attn(fp32)");
        return GLM_OK;
    }
    GLM_CHECK_ARG(tile_tok && tile_n && n_tiles > 0 && tokens_per_tile > 0 && nsplit >= 1 && nsplit <= 64, GLM_ERR_INVALID, "glm_latent_attn: bad tiles");
    GLM_CHECK_ARG(nsplit > 1 ? (part_o && part_ml) : ctx != nullptr, GLM_ERR_INVALID, "glm_latent_attn: no output for %d splits", nsplit);
    const int nct = pick_nct(rp), maxrows = glm_latent_attn_max_rows(rp);
    GLM_CHECK_ARG(nct > 0, GLM_ERR_UNSUPPORTED, "glm_latent_attn: latent of %d columns", rp);
    a.n_hg = (H + maxrows - 1) / maxrows;
    a.hb = (H + a.n_hg - 1) / a.n_hg;
    GLM_CHECK_ARG(tokens_per_tile * a.hb <= maxrows, GLM_ERR_INVALID, "glm_latent_attn: %d tokens x %d heads exceed %d rows", tokens_per_tile, a.hb, maxrows);
    const int64_t range = ((int64_t)bt_stride * block_size < (int64_t)window + tokens_per_tile ? (int64_t)bt_stride * block_size : (int64_t)window + tokens_per_tile);
    GLM_CHECK_ARG((range / nsplit + 128) / block_size + 2 <= LA_BT, GLM_ERR_UNSUPPORTED, "glm_latent_attn: %ld keys per split exceed the block-table slice", (long)(range / nsplit));
    const int rows = tokens_per_tile * a.hb, mt = rows <= 16 ? 1 : rows <= 32 ? 2 : 4;
    switch (nct) {
        case 1: return launch_latent_attn_mt<1>(a, mt, st);
        case 2: return launch_latent_attn_mt<2>(a, mt, st);
        case 3: return launch_latent_attn_mt<3>(a, mt, st);
        case 4: return launch_latent_attn_mt<4>(a, mt, st);
        case 6: return launch_latent_attn_mt<6>(a, mt, st);
        case 8: return launch_latent_attn_mt<8>(a, mt, st);
        case 9: return launch_latent_attn_mt<9>(a, mt, st);
        default: return launch_latent_attn_mt<16>(a, mt, st);
    }
}

extern "C" int glm_latent_up(const void* ctx, const void* wuv, void* out, const void* gate, int64_t ldg, int64_t ldo, int64_t Ta, int H, int vdimp, int rp, glm_stream_t stream) {
    GLM_CHECK_ARG((!gate || (ldg >= (int64_t)H * vdimp && ldg % 4 == 0)), GLM_ERR_INVALID, "glm_latent_up: bad gate (ldg=%ld)", (long)ldg);
    GLM_CHECK_ARG(ctx && wuv && out && Ta >= 0 && H > 0 && vdimp > 0 && vdimp % 8 == 0 && rp > 0 && rp % 8 == 0 && ldo >= (int64_t)H * vdimp && ldo % 4 == 0 &&
                      glm_aligned16(ctx) && glm_aligned16(wuv), GLM_ERR_INVALID, "glm_latent_up: bad shape Ta=%ld H=%d vdimp=%d", (long)Ta, H, vdimp);
    GLM_CHECK_ARG((Ta + 15) / 16 <= 65535, GLM_ERR_UNSUPPORTED, "glm_latent_up: too many rows");
    if (Ta == 0) return GLM_OK;
    UpArgs a = {(const bf16_t*)ctx, (const bf16_t*)wuv, (bf16_t*)out, (const bf16_t*)gate, ldg, ldo, Ta, H, vdimp, rp};
    const int items = H * ((vdimp + 15) / 16);
    hipLaunchKernelGGL(latent_up_kernel, dim3((unsigned)((items + 3) / 4), (unsigned)((Ta + 15) / 16)), dim3(256), 0, glm_s(stream), a);
    GLM_CHECK_LAUNCH("glm_latent_up");
    return GLM_OK;
}
