// Causal grouped-query attention over a key/value cache, with rotary positions and an optional chunk mask, for gfx950.
//
// The query heads of a key/value head share its cache rows: a query row is a (token, head of the group) pair,
// R = tokens * heads / kv_heads rows per entry and key/value head.  A workgroup takes 16 WR RG rows and walks the
// positions its rows see, in tiles staged in LDS; WR = 4: every wavefront has rows of its own and all positions
// of a tile, WR = 1: the wavefronts share 16 rows, deal the positions and merge at the end.
//   scores  S[p][row] = sum_d k[p][d] q[row][d]   first operand: key rows as they lie
//   output  O[d][row] = sum_p v[p][d] w[row][p]   first operand: value columns (transposing LDS read)
// so that a lane's results belong to one row.  Of two score tiles a lane (c, g) holds positions 4 g .. 4 g + 3 and
// 16 + 4 g .. 16 + 4 g + 3 of row c, and the value columns are read in that order: the weights are the second
// operand of the output product as they lie.  Softmax in 32-bit; for bf16 the weights enter the product as two
// bf16 pieces.  With several stretches of positions per row block a second kernel merges them.
//
// The cache is a ring of rows, position p in row p mod ring: with a chunk mask nothing older than a chunk is seen,
// so a ring of a chunk and a step's tokens is enough for a sequence of any length.
#include "seq_common.h"
#include "llaminar_amd/seq_api.h"

namespace llamql
{
    constexpr int ATT_THREADS = 256;
    constexpr int ATT_TARGET = 512; // workgroups aimed at before positions are no longer split
    constexpr int ATT_ROWS = 128;   // most rows of a block

    // 16-byte piece q of staged row r lies at q ^ att_swizzle(r): equal pieces of eight rows and two neighbouring
    // pieces of four rows 4 g .. 4 g + 3 lie in different banks
    __device__ __forceinline__ int att_swizzle(int r) { return ((r & 3) << 1) | ((r >> 2) & 1); }
    __device__ __forceinline__ float att_exp(float x) { return __builtin_amdgcn_exp2f(x * 1.4426950408889634f); }

    // Columns 16 t .. 16 t + 15 of 32 staged rows as an operand: lane (c, g) gets rows 4 g .. and 16 + 4 g .. of column c
    __device__ __forceinline__ bf16x8 att_columns(const bf16 *rows, int ld, int t, int lane)
    {
        typedef __attribute__((address_space(3))) bf16x4 *lds4;
        const int i = lane & 15, g = lane >> 4;
        const int piece = (2 * t + ((i & 3) >> 1)) ^ (((i >> 2) << 1) | (g & 1));
        const bf16 *p = rows + (4 * g + (i >> 2)) * ld + piece * 8 + (i & 1) * 4;
        const bf16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds4)p);
        const bf16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds4)(p + 16 * ld));
        return __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
    }
    __device__ __forceinline__ f32x8 att_columns(const float *rows, int ld, int t, int lane)
    {
        const int c = lane & 15, g = lane >> 4, piece = 4 * t + (c >> 2);
        f32x8 v;
#pragma unroll
        for (int j = 0; j < 8; ++j)
        {
            const int r = (j < 4 ? 0 : 12) + 4 * g + j;
            v[j] = rows[r * ld + (piece ^ att_swizzle(r)) * 4 + (c & 3)];
        }
        return v;
    }

    struct AttentionArgs
    {
        const void *q, *k, *v;
        const int32_t *row0, *ntok, *slot, *pos;
        int first, heads, groups, ring, chunk; // chunk: INT_MAX without a mask
        int stretch, nsplit, rcap, block_rows;
        float scale;
        void *o;
        int ldo;
        float *part_o, *part_ml;
    };

    // first position that position i sees
    __device__ __forceinline__ int att_low(int i, int chunk) { return i / chunk * chunk; }

    template <typename T, int DK, int DV, int WR, int RG>
    __global__ void __launch_bounds__(ATT_THREADS, sizeof(T) == 2 && WR == 4 && DK + DV <= 256 ? 2 : 1)
        attention_kernel(AttentionArgs p)
    {
        using O = Operand<T>;
        using V = typename O::V;
        typedef T t4 __attribute__((ext_vector_type(4)));
        constexpr bool SHORT = sizeof(T) == 2;
        constexpr int WP = 4 / WR;
        constexpr int PG = SHORT && WR == 4 ? 64 : 32; // positions of a wavefront, of a tile
        constexpr int PT = PG * WP;
        constexpr int PS = PG / 32, NB = PG / 16;
        constexpr int KS = DK / 32, NT = DV / 16;
        constexpr int PW = SHORT ? 2 : 1;       // pieces of a softmax weight
        constexpr bool AHEAD = SHORT && WR == 4; // two buffers, the next tile on its way
        constexpr int KP = DK * (int)sizeof(T) / 16, VP = DV * (int)sizeof(T) / 16; // 16-byte pieces of a row
        constexpr int KL = PT * KP / ATT_THREADS, VL = PT * VP / ATT_THREADS;       // of a thread
        constexpr int TILE = PT * (DK + DV);
        extern __shared__ __attribute__((aligned(16))) char smem[];
        __shared__ float s_ml[4][16][2], s_f[4][16];
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
        const int c = lane & 15, g = lane >> 4;
        const int wr = WR == 1 ? 0 : wave, wp = WR == 1 ? wave : 0;
        const int ei = blockIdx.z / p.groups, kv = blockIdx.z - ei * p.groups;
        const int e = p.first + ei, split = blockIdx.y;
        const int per = p.heads / p.groups;
        const int R = p.ntok[e] * per, pos0 = p.pos[e], row0 = p.row0[e];
        const int rb = (gridDim.x - 1 - blockIdx.x) * 16 * RG * WR; // the longest walks first
        if (rb >= R)
            return;
        const int last_row = rb + 16 * RG * WR - 1 < R ? rb + 16 * RG * WR - 1 : R - 1;
        const int pfirst = pos0 + rb / per, kmax = pos0 + last_row / per; // positions of the block's tokens
        const int low0 = att_low(pfirst, p.chunk);
        const int k0 = low0 + split * p.stretch;
        if (k0 > kmax)
            return;
        const int k1 = k0 + p.stretch < kmax + 1 ? k0 + p.stretch : kmax + 1;

        const size_t head = (size_t)p.slot[e] * p.groups + kv;
        const u32x4 *kcache = static_cast<const u32x4 *>(p.k) + head * p.ring * KP;
        const u32x4 *vcache = static_cast<const u32x4 *>(p.v) + head * p.ring * VP;
        u32x4 hk[AHEAD ? KL : 1], hv[AHEAD ? VL : 1];
        // rows past the end are masked; they only must be numbers
        auto source = [&](int p0, int row) __attribute__((always_inline)) {
            int at = p0 % p.ring + (p0 + row <= kmax ? row : kmax - p0);
            return at >= p.ring ? at - p.ring : at;
        };
        auto request = [&](int p0) __attribute__((always_inline)) {
#pragma unroll
            for (int i = 0; i < (AHEAD ? KL : 0); ++i)
            {
                const int n = threadIdx.x + i * ATT_THREADS;
                hk[i] = kcache[(size_t)source(p0, n / KP) * KP + n % KP];
            }
#pragma unroll
            for (int i = 0; i < (AHEAD ? VL : 0); ++i)
            {
                const int n = threadIdx.x + i * ATT_THREADS;
                hv[i] = vcache[(size_t)source(p0, n / VP) * VP + n % VP];
            }
        };
        auto put = [&](int buf) __attribute__((always_inline)) {
            u32x4 *dk = reinterpret_cast<u32x4 *>(reinterpret_cast<T *>(smem) + buf * TILE), *dv = dk + PT * KP;
#pragma unroll
            for (int i = 0; i < (AHEAD ? KL : 0); ++i)
            {
                const int n = threadIdx.x + i * ATT_THREADS, r = n / KP;
                dk[r * KP + ((n % KP) ^ att_swizzle(r))] = hk[i];
            }
#pragma unroll
            for (int i = 0; i < (AHEAD ? VL : 0); ++i)
            {
                const int n = threadIdx.x + i * ATT_THREADS, r = n / VP;
                dv[r * VP + ((n % VP) ^ att_swizzle(r))] = hv[i];
            }
        };
        if constexpr (AHEAD)
            request(k0);

        V q[RG][KS];
        int limit[RG], low[RG]; // positions this lane's row c sees
#pragma unroll
        for (int r = 0; r < RG; ++r)
        {
            const int row = rb + (wr * RG + r) * 16 + c, in = row < R ? row : R - 1;
            const int tok = in / per;
            limit[r] = pos0 + tok; // (rows past the end repeat the last one)
            low[r] = att_low(pos0 + tok, p.chunk);
            const T *src = static_cast<const T *>(p.q) + ((size_t)(row0 + tok) * p.heads + kv * per + in - tok * per) * DK + 8 * g;
#pragma unroll
            for (int ks = 0; ks < KS; ++ks)
                q[r][ks] = O::load(src + ks * 32);
        }

        float m[RG], l[RG]; // of row c; l: this lane's positions only
        f32x4 acc[RG][NT];
#pragma unroll
        for (int r = 0; r < RG; ++r)
        {
            m[r] = -INFINITY, l[r] = 0.0f;
#pragma unroll
            for (int t = 0; t < NT; ++t)
                acc[r][t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        }
        int buf = 0;
        if constexpr (AHEAD)
        {
            put(0);
            if (k0 + PT < k1)
                request(k0 + PT);
        }
        for (int kt = k0; kt < k1; kt += PT)
        {
            if constexpr (!AHEAD)
            {
                __syncthreads();
                u32x4 *dk = reinterpret_cast<u32x4 *>(smem), *dv = dk + PT * KP;
                constexpr int KB = KL < 8 ? KL : 8, VB = VL < 8 ? VL : 8; // held at once
#pragma unroll 1
                for (int i0 = 0; i0 < KL; i0 += KB)
                {
                    u32x4 held[KB];
#pragma unroll
                    for (int i = 0; i < KB; ++i)
                    {
                        const int n = threadIdx.x + (i0 + i) * ATT_THREADS;
                        held[i] = kcache[(size_t)source(kt, n / KP) * KP + n % KP];
                    }
#pragma unroll
                    for (int i = 0; i < KB; ++i)
                    {
                        const int n = threadIdx.x + (i0 + i) * ATT_THREADS, r = n / KP;
                        dk[r * KP + ((n % KP) ^ att_swizzle(r))] = held[i];
                    }
                }
#pragma unroll 1
                for (int i0 = 0; i0 < VL; i0 += VB)
                {
                    u32x4 held[VB];
#pragma unroll
                    for (int i = 0; i < VB; ++i)
                    {
                        const int n = threadIdx.x + (i0 + i) * ATT_THREADS;
                        held[i] = vcache[(size_t)source(kt, n / VP) * VP + n % VP];
                    }
#pragma unroll
                    for (int i = 0; i < VB; ++i)
                    {
                        const int n = threadIdx.x + (i0 + i) * ATT_THREADS, r = n / VP;
                        dv[r * VP + ((n % VP) ^ att_swizzle(r))] = held[i];
                    }
                }
            }
            __syncthreads();

            const T *keys = reinterpret_cast<const T *>(smem) + buf * TILE, *values = keys + PT * DK + wp * PG * DV;
            const u32x4 *krow = reinterpret_cast<const u32x4 *>(keys) + (wp * PG + c) * KP; // (the swizzle of row 16 b + c is that of c)
            const int sw = att_swizzle(c);
            f32x4 s[RG][NB];
#pragma unroll
            for (int b = 0; b < NB; ++b)
            {
#pragma unroll
                for (int r = 0; r < RG; ++r)
                    s[r][b] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
                for (int ks = 0; ks < KS; ++ks)
                {
                    V a;
                    if constexpr (SHORT)
                        a = __builtin_bit_cast(bf16x8, krow[b * 16 * KP + ((4 * ks + g) ^ sw)]);
                    else
                        a = __builtin_shufflevector(__builtin_bit_cast(f32x4, krow[b * 16 * KP + ((8 * ks + 2 * g) ^ sw)]),
                                                    __builtin_bit_cast(f32x4, krow[b * 16 * KP + ((8 * ks + 2 * g + 1) ^ sw)]), 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
                    for (int r = 0; r < RG; ++r)
                        s[r][b] = O::mma(a, q[r][ks], s[r][b]);
                }
            }
            if constexpr (AHEAD)
            {
                if (kt + PT < k1)
                {
                    put(buf ^ 1);
                    if (kt + 2 * PT < k1)
                        request(kt + 2 * PT);
                }
            }

            V w[RG][PS][PW];
#pragma unroll
            for (int r = 0; r < RG; ++r)
            {
                f32x8 x[PS];
                float mx = m[r];
                // (selected without a branch: around one the compiler has mixed up the elements of the result)
                const unsigned from = kt + wp * PG + 4 * g - low[r];
                const unsigned span = limit[r] - low[r]; // (a stretch is whole tiles: what is past it is past the limit)
#pragma unroll
                for (int b = 0; b < PS; ++b)
#pragma unroll
                    for (int j = 0; j < 8; ++j)
                    {
                        const float y = s[r][2 * b + (j >> 2)][j & 3] * p.scale;
                        x[b][j] = from + (32 * b + (j < 4 ? 0 : 12) + j) <= span ? y : -INFINITY;
                        mx = fmaxf(mx, x[b][j]);
                    }
                mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
                mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
                const float base = mx == -INFINITY ? 0.0f : mx;
                const float alpha = att_exp(m[r] - base);
                m[r] = mx;
                float sum = 0.0f;
#pragma unroll
                for (int b = 0; b < PS; ++b)
                {
#pragma unroll
                    for (int j = 0; j < 8; ++j)
                    {
                        x[b][j] = att_exp(x[b][j] - base);
                        sum += x[b][j];
                    }
                    split_pieces<T, PW>(x[b], w[r][b]);
                }
                l[r] = l[r] * alpha + sum;
#pragma unroll
                for (int t = 0; t < NT; ++t)
                    acc[r][t] = acc[r][t] * alpha;
            }
#pragma unroll
            for (int b = 0; b < PS; ++b)
#pragma unroll
                for (int t = 0; t < NT; ++t)
                {
                    const V v = att_columns(values + 32 * b * DV, DV, t, lane);
#pragma unroll
                    for (int i = 0; i < PW; ++i)
#pragma unroll
                        for (int r = 0; r < RG; ++r)
                            acc[r][t] = O::mma(v, w[r][b][i], acc[r][t]);
                }
            if constexpr (AHEAD)
                buf ^= 1;
        }
#pragma unroll
        for (int r = 0; r < RG; ++r)
        {
            l[r] += __shfl_xor(l[r], 16, 64);
            l[r] += __shfl_xor(l[r], 32, 64);
        }
        auto result = [&](int row) __attribute__((always_inline)) {
            const int tok = row / per;
            return static_cast<T *>(p.o) + (size_t)(row0 + tok) * p.ldo + (size_t)(kv * per + row - tok * per) * DV;
        };
        const size_t part = ((size_t)blockIdx.z * p.nsplit + split) * p.rcap;

        if constexpr (WR == 1)
        {
            // merge the wavefronts: [wavefront][16 rows][DV columns]
            __syncthreads();
            float *s_o = reinterpret_cast<float *>(smem);
            constexpr int OLD = DV + 4;
#pragma unroll
            for (int t = 0; t < NT; ++t)
                *reinterpret_cast<f32x4 *>(s_o + (wave * 16 + c) * OLD + 16 * t + 4 * g) = acc[0][t];
            if (g == 0)
            {
                s_ml[wave][c][0] = m[0];
                s_ml[wave][c][1] = l[0];
            }
            __syncthreads();
            if (threadIdx.x < 16)
            {
                const int row = threadIdx.x;
                float M = -INFINITY;
#pragma unroll
                for (int w = 0; w < 4; ++w)
                    M = fmaxf(M, s_ml[w][row][0]);
                const float base = M == -INFINITY ? 0.0f : M;
                float L = 0.0f, f[4];
#pragma unroll
                for (int w = 0; w < 4; ++w)
                {
                    f[w] = att_exp(s_ml[w][row][0] - base);
                    L += f[w] * s_ml[w][row][1];
                }
                const float inv = p.nsplit == 1 ? 1.0f / L : 1.0f;
#pragma unroll
                for (int w = 0; w < 4; ++w)
                    s_f[w][row] = f[w] * inv;
                if (p.nsplit > 1 && rb + row < R)
                {
                    p.part_ml[(part + rb + row) * 2] = M;
                    p.part_ml[(part + rb + row) * 2 + 1] = L;
                }
            }
            __syncthreads();
            for (int n = threadIdx.x; n < 16 * DV / 4; n += ATT_THREADS)
            {
                const int row = n / (DV / 4), d = n % (DV / 4) * 4;
                if (rb + row >= R)
                    break;
                f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
                for (int w = 0; w < 4; ++w)
                    y = y + *reinterpret_cast<const f32x4 *>(s_o + (w * 16 + row) * OLD + d) * s_f[w][row];
                if (p.nsplit == 1)
                    *reinterpret_cast<t4 *>(result(rb + row) + d) = __builtin_convertvector(y, t4);
                else
                    *reinterpret_cast<f32x4 *>(p.part_o + (part + rb + row) * DV + d) = y;
            }
            return;
        }
#pragma unroll
        for (int r = 0; r < RG; ++r)
        {
            const int row = rb + (wr * RG + r) * 16 + c;
            if (row >= R)
                continue;
            const float inv = 1.0f / l[r];
            T *out = result(row);
#pragma unroll
            for (int t = 0; t < NT; ++t)
            {
                if (p.nsplit == 1)
                    *reinterpret_cast<t4 *>(out + 16 * t + 4 * g) = __builtin_convertvector(acc[r][t] * inv, t4);
                else
                    *reinterpret_cast<f32x4 *>(p.part_o + (part + row) * DV + 16 * t + 4 * g) = acc[r][t];
            }
            if (p.nsplit > 1 && g == 0)
            {
                p.part_ml[(part + row) * 2] = m[r];
                p.part_ml[(part + row) * 2 + 1] = l[r];
            }
        }
    }

    // o = sum_s o_s e^(m_s - M) / sum_s l_s e^(m_s - M): a workgroup per query row, its wavefronts dealing the stretches
    template <typename T, int DV>
    __global__ void __launch_bounds__(ATT_THREADS)
        attention_merge_kernel(AttentionArgs p)
    {
        typedef T t4 __attribute__((ext_vector_type(4)));
        constexpr int LANES = DV / 4, TEAMS = ATT_THREADS / LANES;
        __shared__ __attribute__((aligned(16))) float s_y[TEAMS][DV];
        const int ei = blockIdx.y / p.groups, kv = blockIdx.y - ei * p.groups, e = p.first + ei, row = blockIdx.x;
        const int per = p.heads / p.groups;
        if (row >= p.ntok[e] * per)
            return;
        const int tok = row / per, pos0 = p.pos[e];
        const int low = att_low(pos0 + row / p.block_rows * p.block_rows / per, p.chunk); // of the row's block
        int used = (pos0 + tok - low) / p.stretch + 1;
        used = used < p.nsplit ? used : p.nsplit;
        const size_t at = (size_t)blockIdx.y * p.nsplit * p.rcap + row;
        const int team = threadIdx.x / LANES, d = threadIdx.x % LANES * 4, lane = threadIdx.x & 63;
        // every wavefront works out the factors, a stretch a lane
        float M = -INFINITY, L = 0.0f;
        f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int s0 = 0; s0 < used; s0 += 64)
        {
            const size_t k = (at + (size_t)(s0 + lane < used ? s0 + lane : s0) * p.rcap) * 2;
            const float m = s0 + lane < used ? p.part_ml[k] : -INFINITY, l = p.part_ml[k + 1];
            float top = fmaxf(m, M);
#pragma unroll
            for (int off = 32; off > 0; off >>= 1)
                top = fmaxf(top, __shfl_xor(top, off, 64));
            const float base = top == -INFINITY ? 0.0f : top;
            const float f = expf(m - base), before = expf(M - base);
            L = L * before + wave_sum64(f * l);
            y = y * before;
            M = top;
            const int n = used - s0 < 64 ? used - s0 : 64;
            for (int s = team; s < n + team; s += 4 * TEAMS)
#pragma unroll
                for (int j = 0; j < 4; ++j)
                {
                    const bool in = s + j * TEAMS < n;
                    const int mine = in ? s + j * TEAMS : 0;
                    const float w = __shfl(f, mine, 64);
                    const f32x4 o = *reinterpret_cast<const f32x4 *>(p.part_o + (at + (size_t)(s0 + mine) * p.rcap) * DV + d);
                    y = y + o * (in ? w : 0.0f);
                }
        }
        *reinterpret_cast<f32x4 *>(&s_y[team][d]) = y;
        __syncthreads();
        if (team == 0)
        {
#pragma unroll
            for (int k = 1; k < TEAMS; ++k)
                y = y + *reinterpret_cast<const f32x4 *>(&s_y[k][d]);
            T *out = static_cast<T *>(p.o) + (size_t)(p.row0[e] + tok) * p.ldo + (size_t)(kv * per + row - tok * per) * DV;
            *reinterpret_cast<t4 *>(out + d) = __builtin_convertvector(y * (1.0f / L), t4);
        }
    }

    // ---- rotary positions, cache rows ---------------------------------------------------------------
    struct RotaryArgs
    {
        const float *proj;
        int ldp;
        const double *turns;
        int half; // pairs
        const int32_t *row_slot, *row_pos;
        void *q, *k, *v;
        int heads, groups, dim, vdim, ring, append;
    };

    // Workgroup = up to 1024 neighbouring values of one row.  Angles: the turns as a fraction in double, so that far
    // positions keep 32-bit accuracy.
    template <typename T>
    __global__ void __launch_bounds__(256)
        rotary_kernel(RotaryArgs p)
    {
        typedef T t4 __attribute__((ext_vector_type(4)));
        __shared__ float s_cos[128], s_sin[128];
        const int m = blockIdx.x, pos = p.row_pos[m];
        if ((int)threadIdx.x < p.half)
        {
            const double a = p.turns[threadIdx.x] * (double)pos;
            const float f = (float)(2.0 * (a - rint(a)));
            s_cos[threadIdx.x] = cospif(f);
            s_sin[threadIdx.x] = sinpif(f);
        }
        __syncthreads();
        const int col = (blockIdx.y * 256 + threadIdx.x) * 4;
        const int nq = p.heads * p.dim, nk = p.append ? p.groups * p.dim : 0, nv = p.append ? p.groups * p.vdim : 0;
        if (col >= nq + nk + nv || pos < 0)
            return;
        const float *row = p.proj + (size_t)m * p.ldp;
        f32x4 x = *reinterpret_cast<const f32x4 *>(row + col);
        if (col < nq + nk)
        {
            const int d = col & (p.dim - 1);
            const float *head = row + col - d;
#pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                const int n = d + i;
                if (n < p.half)
                    x[i] = x[i] * s_cos[n] - head[n + p.half] * s_sin[n];
                else if (n < 2 * p.half)
                    x[i] = x[i] * s_cos[n - p.half] + head[n - p.half] * s_sin[n - p.half];
            }
        }
        T *dst;
        if (col < nq)
            dst = static_cast<T *>(p.q) + (size_t)m * nq + col;
        else
        {
            const size_t slot = p.row_slot[m];
            const int at = pos % p.ring;
            if (col < nq + nk)
            {
                const int h = (col - nq) / p.dim, d = (col - nq) & (p.dim - 1);
                dst = static_cast<T *>(p.k) + ((slot * p.groups + h) * p.ring + at) * p.dim + d;
            }
            else
            {
                const int h = (col - nq - nk) / p.vdim, d = (col - nq - nk) & (p.vdim - 1);
                dst = static_cast<T *>(p.v) + ((slot * p.groups + h) * p.ring + at) * p.vdim + d;
            }
        }
        *reinterpret_cast<t4 *>(dst) = __builtin_convertvector(x, t4);
    }

    namespace
    {
        bool head_size(int n) { return n == 64 || n == 128 || n == 256; }

        bool attention_sizes(const char *fn, const llam_seq_attention_args *a, int dtype)
        {
            if (!a)
                return fail(fn, "null pointer");
            if (dtype != LLAM_SEQ_BF16 && dtype != LLAM_SEQ_F32)
                return fail(fn, "dtype %d", dtype);
            if (a->heads < 1 || a->kv_heads < 1 || (a->heads % a->kv_heads) != 0)
                return fail(fn, "heads=%d must be a multiple of kv_heads=%d", a->heads, a->kv_heads);
            if (!head_size(a->dim) || !head_size(a->vdim))
                return fail(fn, "dim=%d vdim=%d: heads are padded to 64, 128 or 256", a->dim, a->vdim);
            if (a->ring < 128 || (a->ring % 128) != 0 || a->chunk < 0)
                return fail(fn, "ring=%d must be a multiple of 128 (chunk=%d)", a->ring, a->chunk);
            return true;
        }

        template <typename T, int DK, int DV, int WR, int RG>
        bool attention_launch(const char *fn, const AttentionArgs &p, int row_blocks, int z, hipStream_t st)
        {
            static LdsGrant grant;
            constexpr bool SHORT = sizeof(T) == 2;
            constexpr size_t tile = (size_t)(SHORT && WR == 4 ? 64 : 32) * (4 / WR) * (DK + DV) * sizeof(T) * (SHORT && WR == 4 ? 2 : 1);
            constexpr size_t merge = WR == 1 ? (size_t)64 * (DV + 4) * 4 : 0, lds = tile > merge ? tile : merge;
            static_assert(lds <= 136 * 1024, "tiles must fit the LDS");
            if (lds > 48 * 1024 && allow_lds(grant, reinterpret_cast<const void *>(&attention_kernel<T, DK, DV, WR, RG>), lds) != hipSuccess)
                return fail(fn, "cannot reserve %zu bytes of LDS", lds);
            hipLaunchKernelGGL((attention_kernel<T, DK, DV, WR, RG>), dim3(row_blocks, p.nsplit, z), dim3(ATT_THREADS), lds, st, p);
            return launched(fn);
        }
        template <typename T, int DK, int DV>
        bool attention_rows(const char *fn, AttentionArgs &p, int n, int max_ntok, int max_len, size_t scratch_floats, hipStream_t st)
        {
            constexpr bool NARROW = sizeof(T) == 2 || DK + DV <= 256; // positions dealt to the wavefronts fit the LDS
            constexpr int RG = sizeof(T) == 2 && DK + DV <= 384 ? 2 : 1; // (registers)
            const int per = p.heads / p.groups, R = max_ntok * per;
            const bool narrow = NARROW && R <= 16;
            p.block_rows = narrow ? 16 : 64 * RG;
            p.rcap = R;
            const int row_blocks = ceil_div(R, p.block_rows), z = n * p.groups;
            const int pt = narrow ? 128 : 64;
            // positions from the first that a block's first row sees to its last row's own
            const long reach = (long)p.chunk + p.block_rows / per + 1;
            const int sight = reach < max_len ? (int)reach : max_len;
            int nsplit = ceil_div(ATT_TARGET, row_blocks * z);
            const int most = ceil_div(sight, pt);
            nsplit = nsplit < most ? nsplit : most;
            p.stretch = round_up(ceil_div(sight, nsplit), pt);
            p.nsplit = ceil_div(sight, p.stretch);
            const size_t parts = (size_t)z * p.nsplit * p.rcap;
            if (p.nsplit > 1 && parts * (DV + 2) > scratch_floats)
                return fail(fn, "scratch too small");
            if (row_blocks > 65535 || z > 65535 || p.nsplit > 65535)
                return fail(fn, "too many entries or rows");
            p.part_ml = p.part_o + parts * DV;
            bool ok;
            if constexpr (NARROW)
                ok = narrow ? attention_launch<T, DK, DV, 1, 1>(fn, p, row_blocks, z, st) : attention_launch<T, DK, DV, 4, RG>(fn, p, row_blocks, z, st);
            else
                ok = attention_launch<T, DK, DV, 4, RG>(fn, p, row_blocks, z, st);
            if (!ok || p.nsplit == 1)
                return ok;
            hipLaunchKernelGGL((attention_merge_kernel<T, DV>), dim3(R, z), dim3(ATT_THREADS), 0, st, p);
            return launched(fn);
        }
        template <typename T, int DK, typename... Rest>
        bool attention_values(int vdim, Rest &&...rest)
        {
            return vdim == 64 ? attention_rows<T, DK, 64>(rest...) : vdim == 128 ? attention_rows<T, DK, 128>(rest...) : attention_rows<T, DK, 256>(rest...);
        }
        template <typename T, typename... Rest>
        bool attention_keys(int dim, int vdim, Rest &&...rest)
        {
            return dim == 64 ? attention_values<T, 64>(vdim, rest...) : dim == 128 ? attention_values<T, 128>(vdim, rest...) : attention_values<T, 256>(vdim, rest...);
        }
    } // namespace
} // namespace llamql

using namespace llamql;

extern "C" size_t llam_seq_attention_scratch_floats(int vdim)
{
    // positions are split only below ATT_TARGET workgroups of at most ATT_ROWS rows, into fewer than twice as many
    return vdim < 1 ? 0 : (size_t)2 * ATT_TARGET * ATT_ROWS * ((size_t)vdim + 2);
}

extern "C" bool llam_seq_rotary(const llam_seq_attention_args *a, const float *d_proj, int ldp, bool append, const double *d_turns,
                                int rot_dims, const int32_t *d_row_slot, const int32_t *d_row_pos, void *d_q, int M, int dtype,
                                int device_id, void *stream)
{
    static const char *fn = "llam_seq_rotary";
    if (!attention_sizes(fn, a, dtype))
        return false;
    const int columns = a->heads * a->dim + (append ? a->kv_heads * (a->dim + a->vdim) : 0);
    if (M < 0 || ldp < columns || (ldp % 4) != 0 || rot_dims < 0 || (rot_dims % 2) != 0 || rot_dims > a->dim)
        return fail(fn, "bad size (M=%d ldp=%d rot_dims=%d)", M, ldp, rot_dims);
    if (M == 0)
        return true;
    if (!d_proj || (rot_dims && !d_turns) || !d_row_slot || !d_row_pos || !d_q || (append && (!a->d_k || !a->d_v)))
        return fail(fn, "null pointer");
    if (!aligned16(d_proj) || !aligned16(d_q) || !aligned16(a->d_k) || !aligned16(a->d_v))
        return fail(fn, "misaligned rows");
    if (!set_device(fn, device_id))
        return false;
    RotaryArgs p{d_proj, ldp, d_turns, rot_dims / 2, d_row_slot, d_row_pos, d_q, a->d_k, a->d_v, a->heads, a->kv_heads, a->dim, a->vdim, a->ring, append};
    const dim3 grid(M, ceil_div(columns, 1024));
    if (dtype == LLAM_SEQ_F32)
        hipLaunchKernelGGL(rotary_kernel<float>, grid, dim3(256), 0, as_stream(stream), p);
    else
        hipLaunchKernelGGL(rotary_kernel<bf16>, grid, dim3(256), 0, as_stream(stream), p);
    return launched(fn);
}

extern "C" bool llam_seq_attention(const llam_seq_attention_args *a, const void *d_q, const llam_seq_entries *e, int first, int n,
                                   int max_ntok, int max_len, void *d_o, int ldo, float *d_scratch, size_t scratch_floats,
                                   int dtype, int device_id, void *stream)
{
    static const char *fn = "llam_seq_attention";
    if (!attention_sizes(fn, a, dtype))
        return false;
    if (n < 0 || first < 0 || max_ntok < 1 || max_len < 1 || ldo < a->heads * a->vdim || (ldo % 8) != 0)
        return fail(fn, "bad size (n=%d max_ntok=%d max_len=%d ldo=%d)", n, max_ntok, max_len, ldo);
    const long sight = a->chunk > 0 && a->chunk - 1 + (long)max_ntok < max_len ? a->chunk - 1 + (long)max_ntok : max_len;
    if (sight > a->ring)
        return fail(fn, "%ld positions in sight of an entry, the cache keeps %d", sight, a->ring);
    if (n == 0)
        return true;
    if (!d_q || !a->d_k || !a->d_v || !e || !e->d_row0 || !e->d_ntok || !e->d_slot || !e->d_pos || !d_o || !d_scratch)
        return fail(fn, "null pointer");
    if (!aligned16(d_q) || !aligned16(a->d_k) || !aligned16(a->d_v) || !aligned16(d_o) || !aligned16(d_scratch))
        return fail(fn, "misaligned rows");
    if (!set_device(fn, device_id))
        return false;
    AttentionArgs p{};
    p.q = d_q, p.k = a->d_k, p.v = a->d_v, p.row0 = e->d_row0, p.ntok = e->d_ntok, p.slot = e->d_slot, p.pos = e->d_pos;
    p.first = first, p.heads = a->heads, p.groups = a->kv_heads, p.ring = a->ring, p.chunk = a->chunk > 0 ? a->chunk : 0x3fffffff;
    p.scale = a->scale, p.o = d_o, p.ldo = ldo, p.part_o = d_scratch;
    hipStream_t st = as_stream(stream);
    if (dtype == LLAM_SEQ_F32)
        return attention_keys<float>(a->dim, a->vdim, fn, p, n, max_ntok, max_len, scratch_floats, st);
    return attention_keys<bf16>(a->dim, a->vdim, fn, p, n, max_ntok, max_len, scratch_floats, st);
}
