// Causal attention over a latent cache that serves as key and value at once, for gfx950.
//
// Queries arrive in latent space (q . W_uk, one vector of `rank` per head), so all heads of a
// token share every cache row: a query row is a (token, head) pair, R = tokens * heads rows per
// entry, all against the same keys.  A workgroup takes 16 WR rows and a stretch of the sequence,
// and walks it 32 WP positions at a time (WR * WP = 4 groups of two wavefronts), the cache rows
// staged once in LDS:
//   scores  S[p][row] = sum_d c[p][d] q[row][d]   first operand: c rows as they lie; each wavefront
//                                                  of a pair takes half of the group's positions
//   output  O[d][row] = sum_p c[p][d] w[row][p]   first operand: c columns (transposing LDS read);
//                                                  each takes half of the columns
// so that a lane's results belong to one row.  In between the scores pass through LDS, where both
// wavefronts read them as second operand of the output product and keep the running maximum and sum of their rows.  Softmax in 32-bit; for bf16 the
// weights enter the product as two bf16 pieces.  With WP > 1 the groups of a row block split the
// positions and merge through LDS; with several stretches per row block a second kernel merges those.
#include "seq_common.h"
#include "llaminar_amd/seq_api.h"

namespace llamql
{
    constexpr int LAT_THREADS = 512;
    constexpr int LAT_TARGET = 256; // workgroups aimed at before rows are no longer split
    // positions of a turn that a group takes: 64 where it has the row block to itself and the registers allow
    constexpr int lat_group(int nout, bool qreg, int wr) { return wr == 4 && nout < 32 && qreg ? 64 : 32; }
    constexpr int LAT_MIN_STRETCH = 64; // positions: shorter stretches cost more in partial results than they gain

    // Staged rows lie without padding (a row is a multiple of all 32 banks), their 16-byte pieces permuted by the row:
    // piece q of row r is at q ^ lat_swizzle(r).  Eight rows' equal pieces then lie in different banks (the
    // scores' reads), and so do two neighbouring pieces of four rows (the transposing reads).
    __device__ __forceinline__ int lat_swizzle(int r) { return ((r & 3) << 1) | ((r >> 2) & 1); }

    __device__ __forceinline__ float fast_exp(float x) { return __builtin_amdgcn_exp2f(x * 1.4426950408889634f); }

    // Columns 16 (tile0 + t) .. + 15 of 32 staged rows as a second operand (see load_columns); tile0 a multiple of 4
    __device__ __forceinline__ bf16x8 lat_columns(const bf16 *rows, int ld, int tile0, int t, int lane)
    {
        typedef __attribute__((address_space(3))) bf16x4 *lds4;
        const int i = lane & 15, r = 8 * (lane >> 4) + (i >> 2);
        const int piece = (2 * t + ((i & 3) >> 1)) & 7;
        const bf16 *p = rows + r * ld + 16 * tile0 + ((2 * t) >> 3) * 64 + (i & 1) * 4;
        const bf16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds4)(p + (piece ^ ((i >> 2) << 1)) * 8));
        const bf16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds4)(p + 4 * ld + (piece ^ (((i >> 2) << 1) | 1)) * 8));
        return __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
    }
    __device__ __forceinline__ f32x8 lat_columns(const float *rows, int ld, int tile0, int t, int lane)
    {
        const int c = lane & 15, piece = 4 * (tile0 + t) + (c >> 2);
        f32x8 v;
#pragma unroll
        for (int j = 0; j < 8; ++j)
            v[j] = rows[(8 * (lane >> 4) + j) * ld + (piece ^ lat_swizzle(j)) * 4 + (c & 3)];
        return v;
    }

    struct LatentArgs
    {
        const void *q;
        const void *cache;
        const int32_t *row0, *ntok, *slot, *pos;
        int first, heads, rank, cap, chunk, nsplit, slices, rcap;
        float scale;
        void *o;
        float *part_o, *part_ml;
    };

    // NOUT: 16-column output tiles of a row block, half of them per wavefront.  QREG: the query rows stay in
    // registers (rank <= 16 NOUT); otherwise they are read again for every turn and blockIdx.z also counts
    // slices of the output.  FULL: the rank is 16 NOUT exactly, so that no product hangs on a condition.
    template <typename T, int NOUT, bool QREG, bool FULL, int WR>
    __global__ void __launch_bounds__(LAT_THREADS)
        latent_attention_kernel(LatentArgs p)
    {
        using O = Operand<T>;
        using V = typename O::V;
        typedef T t4 __attribute__((ext_vector_type(4)));
        constexpr int WP = 4 / WR;
        constexpr int PG = lat_group(NOUT, QREG, WR), PT = PG * WP; // positions of a group, of a turn
        constexpr int PS = PG / 32;                               // steps of 32 positions
        constexpr int PW = sizeof(T) == 2 ? 2 : 1; // pieces of a softmax weight
        constexpr int SLD = PG + 4;
        constexpr int NT = NOUT / 2;               // output tiles of a wavefront
        extern __shared__ __attribute__((aligned(16))) char smem[];
        __shared__ __attribute__((aligned(16))) float s_s[4][16 * SLD];
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
        const int c = lane & 15, g = lane >> 4;
        const int half = wave & 1, group = wave >> 1, wr = group % WR, wp = group / WR;
        const int ei = QREG ? blockIdx.z : blockIdx.z / p.slices;
        const int slice = QREG ? 0 : blockIdx.z % p.slices;
        const int e = p.first + ei, split = blockIdx.y;
        const int R = p.ntok[e] * p.heads, pos0 = p.pos[e];
        const int rb = blockIdx.x * 16 * WR;
        if (rb >= R)
            return;
        const int last_row = rb + 16 * WR - 1 < R ? rb + 16 * WR - 1 : R - 1;
        const int kmax = pos0 + last_row / p.heads; // newest position any row of the block sees
        const int k0 = split * p.chunk;
        if (k0 > kmax || kmax >= p.cap)
            return;
        const int k1 = k0 + p.chunk < kmax + 1 ? k0 + p.chunk : kmax + 1;

        const int rank = FULL ? 16 * NOUT : p.rank;
        const int ksteps = rank >> 5;
        const int ld = rank;
        const T *cache = static_cast<const T *>(p.cache) + (size_t)p.slot[e] * p.cap * rank;

        // The cache rows of a turn: TPR threads a row.  With two buffers the next turn's rows are requested
        // before this turn's products and put down in the middle of them.
        constexpr int TPR = LAT_THREADS / PT;
        constexpr int LOADS = NOUT * (int)sizeof(T) >= TPR ? NOUT * (int)sizeof(T) / TPR : 1; // 16-byte pieces a thread, when QREG
        constexpr bool AHEAD = QREG && WP == 1;
        constexpr int BATCH = LOADS < 8 || AHEAD ? LOADS : WP == 4 && NOUT >= 32 ? 4 : 8; // held at once
        const int pieces = rank * (int)sizeof(T) / 16;
        const int srow = threadIdx.x / TPR, sseg = threadIdx.x % TPR;
        u32x4 held[QREG ? BATCH : 1];
        auto request = [&](int p0, int i0) __attribute__((always_inline)) {
            // rows past the end are masked; they only must be numbers
            const u32x4 *src = reinterpret_cast<const u32x4 *>(cache + (size_t)(p0 + srow <= kmax ? p0 + srow : kmax) * rank) + sseg;
#pragma unroll
            for (int i = 0; i < BATCH; ++i)
                held[i] = src[sseg + (i0 + i) * TPR < pieces ? (i0 + i) * TPR : 0];
        };
        auto put = [&](int buf, int i0) __attribute__((always_inline)) {
            u32x4 *dst = reinterpret_cast<u32x4 *>(reinterpret_cast<T *>(smem) + (buf * PT + srow) * ld);
#pragma unroll
            for (int i = 0; i < BATCH; ++i)
                if (sseg + (i0 + i) * TPR < pieces)
                    dst[(sseg + (i0 + i) * TPR) ^ lat_swizzle(srow)] = held[i];
        };
        if constexpr (AHEAD)
            request(k0, 0);

        const int qrow = rb + wr * 16 + c < R ? rb + wr * 16 + c : R - 1;
        const T *q = static_cast<const T *>(p.q) + ((size_t)p.row0[e] * p.heads + qrow) * rank + 8 * g;
        V qreg[QREG ? NOUT / 2 : 1];
        if (QREG)
        {
#pragma unroll
            for (int ks = 0; ks < NOUT / 2; ++ks)
                if (ks < ksteps)
                    qreg[ks] = O::load(q + ks * 32);
        }
        const int limit = rb + wr * 16 + c < R ? pos0 + qrow / p.heads : -1; // newest position this lane's row c sees
        const int tile0 = slice * NOUT + half * NT;                         // the wavefront's first output tile
        const int out_tiles = FULL || (rank >> 4) - tile0 > NT ? NT : (rank >> 4) - tile0;

        float m = -INFINITY, l = 0.0f; // of row c; l: this lane's positions only
        f32x4 acc[NT];
#pragma unroll
        for (int t = 0; t < NT; ++t)
            acc[t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        int buf = 0;
        if constexpr (AHEAD)
        {
            put(0, 0);
            if (k0 + PT < k1)
                request(k0 + PT, 0);
        }
        for (int kt = k0; kt < k1; kt += PT)
        {
            if constexpr (!AHEAD)
            {
                __syncthreads();
                if constexpr (QREG)
                {
#pragma unroll
                    for (int i = 0; i < LOADS; i += BATCH)
                    {
                        request(kt, i);
                        put(0, i);
                    }
                }
                else
                {
                    const int pos = kt + srow <= kmax ? kt + srow : kmax;
                    const u32x4 *src = reinterpret_cast<const u32x4 *>(cache + (size_t)pos * rank);
                    u32x4 *dst = reinterpret_cast<u32x4 *>(reinterpret_cast<T *>(smem) + srow * ld);
                    for (int i = sseg; i < pieces; i += TPR)
                        dst[i ^ lat_swizzle(srow)] = src[i];
                }
            }
            __syncthreads();

            // (the swizzle of a row of a 16-row block is that of the row in the block)
            const T *mine = reinterpret_cast<const T *>(smem) + (buf * PT + wp * PG) * ld;
            const u32x4 *keys = reinterpret_cast<const u32x4 *>(mine + (half * (PG / 2) + c) * ld);
            const int key_swizzle = lat_swizzle(c);
            auto key = [&](int block, int ks) __attribute__((always_inline)) {
                const u32x4 *row = keys + block * (16 * pieces);
                if constexpr (sizeof(T) == 2)
                    return __builtin_bit_cast(bf16x8, row[(4 * ks + g) ^ key_swizzle]);
                else
                    return __builtin_shufflevector(__builtin_bit_cast(f32x4, row[(8 * ks + 2 * g) ^ key_swizzle]),
                                                   __builtin_bit_cast(f32x4, row[(8 * ks + 2 * g + 1) ^ key_swizzle]), 0, 1, 2, 3, 4, 5, 6, 7);
            };
            f32x4 s[PS][2];
#pragma unroll
            for (int b = 0; b < PS; ++b)
                s[b][0] = s[b][1] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
            if (QREG)
            {
#pragma unroll
                for (int ks = 0; ks < NOUT / 2; ++ks)
                    if (ks < ksteps)
                    {
#pragma unroll
                        for (int b = 0; b < PS; ++b)
                            s[b][ks & 1] = O::mma(key(b, ks), qreg[ks], s[b][ks & 1]);
                    }
            }
            else
                for (int ks = 0; ks < ksteps; ks += 2) // (the rank is a multiple of 64)
                {
                    const V a0 = O::load(q + ks * 32), a1 = O::load(q + ks * 32 + 32);
#pragma unroll
                    for (int b = 0; b < PS; ++b)
                    {
                        s[b][0] = O::mma(key(b, ks), a0, s[b][0]);
                        s[b][1] = O::mma(key(b, ks + 1), a1, s[b][1]);
                    }
                }
#pragma unroll
            for (int b = 0; b < PS; ++b) // lane: row c, positions 4 g .. 4 g + 3
                *reinterpret_cast<f32x4 *>(&s_s[group][c * SLD + half * (PG / 2) + 16 * b + 4 * g]) = s[b][0] + s[b][1];
            if constexpr (AHEAD)
            {
                if (kt + PT < k1)
                {
                    put(buf ^ 1, 0);
                    if (kt + 2 * PT < k1)
                        request(kt + 2 * PT, 0);
                }
            }
            __syncthreads();

            // row c, positions 32 b + 8 g .. + 7 of the group's
            f32x8 w[PS];
            float mx = m;
#pragma unroll
            for (int b = 0; b < PS; ++b)
            {
                w[b] = Operand<float>::load(&s_s[group][c * SLD + 32 * b + 8 * g]);
#pragma unroll
                for (int j = 0; j < 8; ++j)
                {
                    w[b][j] = kt + wp * PG + 32 * b + 8 * g + j <= limit ? w[b][j] * p.scale : -INFINITY;
                    mx = fmaxf(mx, w[b][j]);
                }
            }
            mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
            mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
            const float base = mx == -INFINITY ? 0.0f : mx;
            const float alpha = fast_exp(m - base);
            m = mx;
            l *= alpha;
            V wv[PS][PW];
#pragma unroll
            for (int b = 0; b < PS; ++b)
            {
#pragma unroll
                for (int j = 0; j < 8; ++j)
                {
                    w[b][j] = fast_exp(w[b][j] - base);
                    l += w[b][j];
                }
                split_pieces<T, PW>(w[b], wv[b]);
            }
#pragma unroll
            for (int t = 0; t < NT; ++t)
                acc[t] = acc[t] * alpha;
            constexpr int VG = sizeof(T) == 2 ? 4 : 2; // independent products in a row (NT is a multiple)
#pragma unroll
            for (int b = 0; b < PS; ++b)
#pragma unroll
                for (int t = 0; t < NT; t += VG)
                    if (t < out_tiles)
                    {
                        V v[VG];
#pragma unroll
                        for (int k = 0; k < VG; ++k) // (tiles past the rank come in fours: none is begun)
                            v[k] = lat_columns(mine + 32 * b * ld, ld, tile0, t + k, lane);
#pragma unroll
                        for (int i = 0; i < PW; ++i)
#pragma unroll
                            for (int k = 0; k < VG; ++k)
                                acc[t + k] = O::mma(v[k], wv[b][i], acc[t + k]);
                    }
            if constexpr (AHEAD)
                buf ^= 1;
        }
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);

        if (WP > 1)
        {
            // merge the groups of each row block: [group][16 rows][16 NOUT columns], then (m, l) of their rows
            __syncthreads();
            float *s_o = reinterpret_cast<float *>(smem);
            float *s_ml = &s_s[0][0];
            constexpr int OLD = NOUT * 16 + 4;
#pragma unroll
            for (int t = 0; t < NT; ++t)
                if (t < out_tiles)
                    *reinterpret_cast<f32x4 *>(s_o + (group * 16 + c) * OLD + (half * NT + t) * 16 + 4 * g) = acc[t];
            if (half == 0 && g == 0)
            {
                s_ml[(group * 16 + c) * 2] = m;
                s_ml[(group * 16 + c) * 2 + 1] = l;
            }
            __syncthreads();
            // per row: the groups' factors e^(m_w - M) (over the sum, when the result is final)
            float *s_f = s_ml + 128;
            if (threadIdx.x < WR * 16)
            {
                const int row = threadIdx.x;
                float M = -INFINITY;
#pragma unroll
                for (int w = 0; w < WP; ++w)
                    M = fmaxf(M, s_ml[(w * WR * 16 + row) * 2]);
                const float base = M == -INFINITY ? 0.0f : M;
                float L = 0.0f, f[WP];
#pragma unroll
                for (int w = 0; w < WP; ++w)
                {
                    f[w] = fast_exp(s_ml[(w * WR * 16 + row) * 2] - base);
                    L += f[w] * s_ml[(w * WR * 16 + row) * 2 + 1];
                }
                const float inv = p.nsplit == 1 ? 1.0f / L : 1.0f;
#pragma unroll
                for (int w = 0; w < WP; ++w)
                    s_f[w * WR * 16 + row] = f[w] * inv;
                if (p.nsplit > 1 && slice == 0 && rb + row < R)
                {
                    const size_t at = ((size_t)ei * p.nsplit + split) * p.rcap + rb + row;
                    p.part_ml[at * 2] = M;
                    p.part_ml[at * 2 + 1] = L;
                }
            }
            __syncthreads();
            // a wavefront takes every eighth row
            const int columns = rank - slice * NOUT * 16 < NOUT * 16 ? rank - slice * NOUT * 16 : NOUT * 16;
            for (int row = wave; row < WR * 16 && rb + row < R; row += LAT_THREADS / 64)
                for (int d = lane * 4; d < columns; d += 256)
                {
                    f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
                    for (int w = 0; w < WP; ++w)
                        y = y + *reinterpret_cast<const f32x4 *>(s_o + (w * WR * 16 + row) * OLD + d) * s_f[w * WR * 16 + row];
                    const int col = slice * NOUT * 16 + d;
                    if (p.nsplit == 1)
                        *reinterpret_cast<t4 *>(static_cast<T *>(p.o) + ((size_t)p.row0[e] * p.heads + rb + row) * rank + col) =
                            __builtin_convertvector(y, t4);
                    else
                        *reinterpret_cast<f32x4 *>(p.part_o + (((size_t)ei * p.nsplit + split) * p.rcap + rb + row) * rank + col) = y;
                }
            return;
        }
        const int row = rb + wr * 16 + c;
        if (row >= R)
            return;
        const size_t at = ((size_t)ei * p.nsplit + split) * p.rcap + row;
        const float inv = 1.0f / l;
#pragma unroll
        for (int t = 0; t < NT; ++t)
            if (t < out_tiles)
            {
                const int col = (tile0 + t) * 16 + 4 * g;
                if (p.nsplit == 1)
                    *reinterpret_cast<t4 *>(static_cast<T *>(p.o) + ((size_t)p.row0[e] * p.heads + row) * rank + col) =
                        __builtin_convertvector(acc[t] * inv, t4);
                else
                    *reinterpret_cast<f32x4 *>(p.part_o + at * rank + col) = acc[t];
            }
        if (p.nsplit > 1 && half == 0 && g == 0 && slice == 0)
        {
            p.part_ml[at * 2] = m;
            p.part_ml[at * 2 + 1] = l;
        }
    }

    // o = sum_s o_s e^(m_s - M) / sum_s l_s e^(m_s - M): one workgroup per query row and 128 columns, eight groups
    // of 32 threads dealing the stretches among themselves
    constexpr int LAT_MERGE_COLS = 128;
    template <typename T>
    __global__ void __launch_bounds__(256)
        latent_merge_kernel(LatentArgs p)
    {
        typedef T t4 __attribute__((ext_vector_type(4)));
        __shared__ __attribute__((aligned(16))) float s_y[8][LAT_MERGE_COLS];
        __shared__ float s_w[LAT_TARGET + 256];
        __shared__ float s_red[4];
        const int ei = blockIdx.y, e = p.first + ei, row = blockIdx.x;
        if (row >= p.ntok[e] * p.heads)
            return;
        const int limit = p.pos[e] + row / p.heads;
        if (limit >= p.cap)
            return;
        const int used = limit / p.chunk + 1;
        const size_t at = (size_t)ei * p.nsplit * p.rcap + row;
        const int group = threadIdx.x >> 5, d = blockIdx.z * LAT_MERGE_COLS + (threadIdx.x & 31) * 4;
        float M = -INFINITY;
        for (int s = threadIdx.x; s < used; s += 256)
            M = fmaxf(M, p.part_ml[(at + (size_t)s * p.rcap) * 2]);
#pragma unroll
        for (int off = 32; off > 0; off >>= 1)
            M = fmaxf(M, __shfl_xor(M, off, 64));
        if ((threadIdx.x & 63) == 0)
            s_red[threadIdx.x >> 6] = M;
        __syncthreads();
        M = fmaxf(fmaxf(s_red[0], s_red[1]), fmaxf(s_red[2], s_red[3]));
        float L = 0.0f;
        for (int s = threadIdx.x; s < used; s += 256)
        {
            const size_t k = (at + (size_t)s * p.rcap) * 2;
            const float f = expf(p.part_ml[k] - M);
            s_w[s] = f;
            L += f * p.part_ml[k + 1];
        }
        L = block_sum<256>(L, s_red);
        f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f};
        if (d < p.rank)
        {
#pragma unroll 8
            for (int s = group; s < used; s += 8)
                y = y + *reinterpret_cast<const f32x4 *>(p.part_o + (at + (size_t)s * p.rcap) * p.rank + d) * s_w[s];
        }
        *reinterpret_cast<f32x4 *>(&s_y[group][(threadIdx.x & 31) * 4]) = y;
        __syncthreads();
        if (threadIdx.x < 32 && d < p.rank)
        {
#pragma unroll
            for (int k = 1; k < 8; ++k)
                y = y + *reinterpret_cast<const f32x4 *>(&s_y[k][threadIdx.x * 4]);
            *reinterpret_cast<t4 *>(static_cast<T *>(p.o) + ((size_t)p.row0[e] * p.heads + row) * p.rank + d) =
                __builtin_convertvector(y * (1.0f / L), t4);
        }
    }

    template <typename T>
    __global__ void __launch_bounds__(256)
        latent_append_kernel(const float *__restrict__ x, int ldx, const float *__restrict__ norm, float eps, int k_real,
                             const int32_t *__restrict__ row_slot, const int32_t *__restrict__ row_pos,
                             T *__restrict__ cache, int rank, int cap)
    {
        typedef T t4 __attribute__((ext_vector_type(4)));
        __shared__ float s_sum[4];
        const int m = blockIdx.x, pos = row_pos[m];
        const f32x4 *row = reinterpret_cast<const f32x4 *>(x + (size_t)m * ldx);
        float sum = 0.0f;
        for (int i = threadIdx.x; i < rank / 4; i += 256)
        {
            const f32x4 v = row[i];
            sum += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
        }
        sum = block_sum<256>(sum, s_sum);
        if (pos < 0 || pos >= cap)
            return;
        const float inv = 1.0f / sqrtf(sum / (float)k_real + eps);
        T *dst = cache + ((size_t)row_slot[m] * cap + pos) * rank;
        for (int i = threadIdx.x; i < rank / 4; i += 256)
            *reinterpret_cast<t4 *>(dst + 4 * i) =
                __builtin_convertvector(row[i] * inv * reinterpret_cast<const f32x4 *>(norm)[i], t4);
    }

    namespace
    {
        template <typename T, int NOUT, bool QREG, bool FULL, int WR>
        bool latent_launch(const char *fn, const LatentArgs &p, int row_blocks, int n, hipStream_t st)
        {
            static LdsGrant grant;
            constexpr int WP = 4 / WR;
            size_t lds = (size_t)lat_group(NOUT, QREG, WR) * WP * (QREG && WP == 1 ? 2 : 1) * p.rank * sizeof(T);
            const size_t merge = WP > 1 ? (size_t)64 * (NOUT * 16 + 4) * 4 : 0;
            lds = lds > merge ? lds : merge;
            constexpr size_t most = 142 * 1024; // beside the scores
            if (lds > most)
                return fail(fn, "rank=%d does not fit the LDS", p.rank);
            if (lds > 48 * 1024 && allow_lds(grant, reinterpret_cast<const void *>(&latent_attention_kernel<T, NOUT, QREG, FULL, WR>), most) != hipSuccess)
                return fail(fn, "cannot reserve %zu bytes of LDS", lds);
            hipLaunchKernelGGL((latent_attention_kernel<T, NOUT, QREG, FULL, WR>), dim3(row_blocks, p.nsplit, n * p.slices),
                               dim3(LAT_THREADS), lds, st, p);
            return launched(fn);
        }
        template <typename T, int NOUT, bool QREG, bool FULL>
        bool latent_stretches(const char *fn, const LatentArgs &p, int wr, int row_blocks, int n, hipStream_t st)
        {
            if (wr == 1)
                return latent_launch<T, NOUT, QREG, FULL, 1>(fn, p, row_blocks, n, st);
            if (wr == 2)
                return latent_launch<T, NOUT, QREG, FULL, 2>(fn, p, row_blocks, n, st);
            return latent_launch<T, NOUT, QREG, FULL, 4>(fn, p, row_blocks, n, st);
        }

        template <typename T, int NOUT, bool QREG>
        bool latent_rows(const char *fn, const LatentArgs &p, int wr, int row_blocks, int n, hipStream_t st)
        {
            if constexpr (QREG && sizeof(T) == 2)
            {
                if (p.rank == 16 * NOUT)
                    return latent_stretches<T, NOUT, QREG, true>(fn, p, wr, row_blocks, n, st);
            }
            return latent_stretches<T, NOUT, QREG, false>(fn, p, wr, row_blocks, n, st);
        }

        // how a call is cut up: wavefronts per row group and stretches of the sequence
        struct LatentPlan
        {
            int wr, row_blocks, chunk, nsplit;
        };
        LatentPlan latent_plan(int n, int max_ntok, int max_len, int heads, int rank, int elem)
        {
            LatentPlan pl{};
            const int R = max_ntok * heads;
            pl.wr = R <= 16 ? 1 : R <= 32 ? 2 : 4;
            while (pl.wr < 4)
            {
                const int wp = 4 / pl.wr;
                if ((size_t)32 * wp * rank * elem <= 140 * 1024)
                    break;
                pl.wr *= 2;
            }
            const int pt = pl.wr == 4 ? (rank > 256 ? 32 : 64) : 32 * (4 / pl.wr);
            pl.row_blocks = ceil_div(R, 16 * pl.wr);
            int nsplit = ceil_div(LAT_TARGET, pl.row_blocks * n);
            const int most = ceil_div(max_len, pt > LAT_MIN_STRETCH ? pt : LAT_MIN_STRETCH);
            nsplit = nsplit < most ? nsplit : most;
            pl.chunk = round_up(ceil_div(max_len, nsplit), pt);
            pl.nsplit = ceil_div(max_len, pl.chunk);
            return pl;
        }
    } // namespace
} // namespace llamql

using namespace llamql;

extern "C" bool llam_seq_latent_append(const float *d_x, int ldx, const float *d_norm, float eps, int k_real,
                                       const int32_t *d_row_slot, const int32_t *d_row_pos, void *d_cache, int M,
                                       int rank, int cap, int dtype, int device_id, void *stream)
{
    static const char *fn = "llam_seq_latent_append";
    if (M < 0 || rank < 1 || cap < 1 || k_real < 1 || k_real > rank || ldx < rank)
        return fail(fn, "bad size (M=%d rank=%d cap=%d)", M, rank, cap);
    if (M == 0)
        return true;
    if (!d_x || !d_norm || !d_row_slot || !d_row_pos || !d_cache)
        return fail(fn, "null pointer");
    if ((rank % PAD) != 0 || (ldx % 4) != 0 || !aligned16(d_x) || !aligned16(d_norm) || !aligned16(d_cache))
        return fail(fn, "misaligned rows");
    if (!set_device(fn, device_id))
        return false;
    if (dtype == LLAM_SEQ_F32)
        hipLaunchKernelGGL(latent_append_kernel<float>, dim3(M), dim3(256), 0, as_stream(stream), d_x, ldx, d_norm, eps,
                           k_real, d_row_slot, d_row_pos, static_cast<float *>(d_cache), rank, cap);
    else
        hipLaunchKernelGGL(latent_append_kernel<bf16>, dim3(M), dim3(256), 0, as_stream(stream), d_x, ldx, d_norm, eps,
                           k_real, d_row_slot, d_row_pos, static_cast<bf16 *>(d_cache), rank, cap);
    return launched(fn);
}

extern "C" size_t llam_seq_latent_scratch_floats(int max_rows, int slots, int heads, int rank, int cap)
{
    if (max_rows < 1 || slots < 1 || heads < 1 || rank < 1 || cap < 1)
        return 0;
    // rows that are split: fewer than LAT_TARGET workgroups of at most 64 rows, at most about
    // 2 LAT_TARGET of them after the split; every entry of a call takes at least one row group
    return ((size_t)2 * LAT_TARGET + slots) * 64 * ((size_t)rank + 2);
}

extern "C" bool llam_seq_latent_attention(const void *d_q, const void *d_cache, const llam_seq_entries *e, int first,
                                          int n, int max_ntok, int max_len, int heads, int rank, int cap, float scale,
                                          void *d_o, float *d_scratch, size_t scratch_floats, int dtype, int device_id,
                                          void *stream)
{
    static const char *fn = "llam_seq_latent_attention";
    if (n < 0 || first < 0 || heads < 1 || rank < 1 || cap < 1 || max_ntok < 1 || max_len < 1 || max_len > cap)
        return fail(fn, "bad size (n=%d heads=%d rank=%d cap=%d max_ntok=%d max_len=%d)", n, heads, rank, cap, max_ntok, max_len);
    if (n == 0)
        return true;
    if (!d_q || !d_cache || !e || !e->d_row0 || !e->d_ntok || !e->d_slot || !e->d_pos || !d_o || !d_scratch)
        return fail(fn, "null pointer");
    if ((rank % PAD) != 0 || !aligned16(d_q) || !aligned16(d_cache) || !aligned16(d_o) || !aligned16(d_scratch))
        return fail(fn, "rank=%d must be a multiple of %d, rows 16-byte aligned", rank, PAD);
    if (dtype != LLAM_SEQ_BF16 && dtype != LLAM_SEQ_F32)
        return fail(fn, "dtype %d", dtype);
    const LatentPlan pl = latent_plan(n, max_ntok, max_len, heads, rank, dtype == LLAM_SEQ_F32 ? 4 : 2);
    LatentArgs p{};
    p.q = d_q, p.cache = d_cache, p.row0 = e->d_row0, p.ntok = e->d_ntok, p.slot = e->d_slot, p.pos = e->d_pos;
    p.first = first, p.heads = heads, p.rank = rank, p.cap = cap, p.chunk = pl.chunk, p.nsplit = pl.nsplit;
    p.scale = scale, p.o = d_o, p.slices = 1;
    p.rcap = max_ntok * heads;
    const size_t parts = (size_t)n * pl.nsplit * p.rcap;
    if (pl.nsplit > 1 && parts * ((size_t)rank + 2) > scratch_floats)
        return fail(fn, "scratch too small");
    p.part_o = d_scratch, p.part_ml = d_scratch + parts * rank;
    if (n > 65535 || pl.nsplit > 65535)
        return fail(fn, "too many entries");
    if (!set_device(fn, device_id))
        return false;
    hipStream_t st = as_stream(stream);
    bool ok;
    if (dtype == LLAM_SEQ_F32)
    {
        if (rank <= 128)
            ok = latent_rows<float, 8, true>(fn, p, pl.wr, pl.row_blocks, n, st);
        else
        {
            p.slices = ceil_div(rank, 256);
            ok = latent_rows<float, 16, false>(fn, p, pl.wr, pl.row_blocks, n, st);
        }
    }
    else if (rank <= 128)
        ok = latent_rows<bf16, 8, true>(fn, p, pl.wr, pl.row_blocks, n, st);
    else if (rank <= 256)
        ok = latent_rows<bf16, 16, true>(fn, p, pl.wr, pl.row_blocks, n, st);
    else if (rank <= 512)
        ok = latent_rows<bf16, 32, true>(fn, p, pl.wr, pl.row_blocks, n, st);
    else
    {
        p.slices = ceil_div(rank, 256);
        ok = latent_rows<bf16, 16, false>(fn, p, pl.wr, pl.row_blocks, n, st);
    }
    if (!ok || pl.nsplit == 1)
        return ok;
    if (dtype == LLAM_SEQ_F32)
        hipLaunchKernelGGL(latent_merge_kernel<float>, dim3(p.rcap, n, ceil_div(rank, LAT_MERGE_COLS)), dim3(256), 0, st, p);
    else
        hipLaunchKernelGGL(latent_merge_kernel<bf16>, dim3(p.rcap, n, ceil_div(rank, LAT_MERGE_COLS)), dim3(256), 0, st, p);
    return launched(fn);
}
