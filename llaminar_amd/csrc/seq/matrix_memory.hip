// Matrix-memory recurrence (per head: memory S [dim x vdim], normaliser n [dim], running maximum m),
// for gfx950.
//
// The normaliser is carried as one more column of S: a column whose value is 1 for every token.
// S and the outputs have vdim + 16 columns, column vdim being n (the other 15 stay zero).
//
// Decoding streams S once through the chip (read, update, write: HBM-bound).  Prompts run in chunks of
// LC tokens.  With F_t the sum of the log forget gates from the chunk's start to t, m0 the running
// maximum before it and a_j = i_j - F_j, the recurrence unrolls to
//   m_t = F_t + max(m0, max_{j<=t} a_j)
//   S_t' q = e^(F_t + m0 - m_t) S_0' q + sum_{j<=t} e^(F_t + a_j - m_t) (k_j . q) v_j
//   S_end = e^(F_end + m0 - m_end) S_0 + sum_j e^(F_end + a_j - m_end) k_j v_j'
// in three launches: the gates (one wavefront per head walks the portion; F, a and F - m in double, so
// that differences of long sums keep 32-bit accuracy), the token-by-token products of every chunk
// (independent of each other), and the walk over the chunks, where a wavefront owns 16 columns of
// S in its accumulators from the first chunk to the last.  An accumulator tile is also a second
// operand of the next product as it lies: lane (c, g) holds rows 4 g .. 4 g + 3, and the first operand
// is read in the same order.  In bf16, S and the gated values enter the products in three pieces,
// i.e. as 32-bit values; q, k and v are bf16 (the output format of a projection).
#include "seq_common.h"
#include "llaminar_amd/seq_api.h"

namespace llamql
{
    struct MemoryArgs
    {
        const float *proj;
        int ldp;
        const float *gate_bias, *norm;
        float *state, *m;
        void *y;
        int ldy;
        int heads, dim, vdim, vdim_real;
        float q_scale, gate_cap, eps;
        const int32_t *row0, *ntok, *slot, *pos;
        int entry;      // first entry of the call
        double *ga, *a; // [rows][heads]: F_t - m_t, a_t
        float *mt;      // [rows][heads]: m_t
        float *m0;      // [heads]: m before the portion
        float *prod;    // [chunks][heads][LC][LC]
        float *num;     // [rows][heads][vdim + 16]; decoding: [entries][heads][splits][vdim + 16]
        int splits;     // decoding: workgroups along dim
        void *qk;       // T [2][heads][rows of the portion][dim]: scaled q, then k
        int qk_rows;
    };

    __device__ __forceinline__ void memory_gates(const MemoryArgs &p, const float *row, int h, float &i, float &f)
    {
        const float *raw = row + (size_t)p.heads * 2 * (p.dim + p.vdim);
        const float zi = raw[h] + p.gate_bias[h], zf = raw[p.heads + h] + p.gate_bias[p.heads + h];
        i = p.gate_cap * tanhf(zi / p.gate_cap);
        const float c = p.gate_cap * tanhf(zf / p.gate_cap);
        f = fminf(c, 0.0f) - log1pf(expf(-fabsf(c)));
    }

    // ---- decoding -------------------------------------------------------------------------------
    // Workgroup = 64 columns of one head's memory of one sequence, and a stretch of its rows.
    constexpr int STEP_ROWS = 64; // rows of a stretch when there are several
    template <typename T>
    __global__ void __launch_bounds__(256)
        memory_step_kernel(MemoryArgs p)
    {
        __shared__ float s_q[512], s_k[512];
        __shared__ __attribute__((aligned(16))) float s_o[16][64];
        const int h = blockIdx.y, ei = blockIdx.z, e = p.entry + ei;
        const int ldv = p.vdim + 16, blocks = (ldv + 63) >> 6;
        const int split = blockIdx.x / blocks, block = blockIdx.x - split * blocks;
        const int rows = p.splits > 1 ? STEP_ROWS : p.dim, first = split * rows;
        const int r = p.row0[e], slot = p.slot[e];
        const float *row = p.proj + (size_t)r * p.ldp;
        const int col = block * 64 + (threadIdx.x & 15) * 4, d0 = threadIdx.x >> 4;
        const bool fresh = p.pos[e] == 0;
        float *S = p.state + (((size_t)slot * p.heads + h) * p.dim + first) * ldv + col;
        const bool live = col < ldv;

        f32x4 v = {0.0f, 0.0f, 0.0f, 0.0f};
        if (col < p.vdim)
        {
            v = *reinterpret_cast<const f32x4 *>(row + (size_t)p.heads * 2 * p.dim + h * p.vdim + col);
#pragma unroll
            for (int j = 0; j < 4; ++j)
                v[j] = rounded<T>(v[j]);
        }
        else if (col == p.vdim)
            v[0] = 1.0f;
        for (int d = threadIdx.x; d < rows; d += 256)
        {
            s_q[d] = rounded<T>(row[h * p.dim + first + d] * p.q_scale);
            s_k[d] = rounded<T>(row[(p.heads + h) * p.dim + first + d]);
        }
        constexpr int U = STEP_ROWS / 16; // the first rows are requested before the gates are worked out
        f32x4 s[U];
#pragma unroll
        for (int u = 0; u < U; ++u)
        {
            s[u] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
            if (live && !fresh)
                s[u] = *reinterpret_cast<const f32x4 *>(S + (size_t)(d0 + 16 * u) * ldv);
        }
        float gi, gf;
        memory_gates(p, row, h, gi, gf);
        const float m_old = fresh ? 0.0f : p.m[slot * p.heads + h];
        const float m_new = fmaxf(gf + m_old, gi);
        const float keep = expf(gf + m_old - m_new), take = expf(gi - m_new);
        v = v * take;
        __syncthreads();
        f32x4 o = {0.0f, 0.0f, 0.0f, 0.0f};
        if (live)
            for (int d = d0; d < rows; d += STEP_ROWS)
            {
                if (d != d0)
                {
#pragma unroll
                    for (int u = 0; u < U; ++u)
                        s[u] = fresh ? f32x4{0.0f, 0.0f, 0.0f, 0.0f} : *reinterpret_cast<const f32x4 *>(S + (size_t)(d + 16 * u) * ldv);
                }
#pragma unroll
                for (int u = 0; u < U; ++u)
                {
                    s[u] = s[u] * keep + v * s_k[d + 16 * u];
                    *reinterpret_cast<f32x4 *>(S + (size_t)(d + 16 * u) * ldv) = s[u];
                    o = o + s[u] * s_q[d + 16 * u];
                }
            }
        *reinterpret_cast<f32x4 *>(&s_o[d0][(threadIdx.x & 15) * 4]) = o;
        __syncthreads();
        if (threadIdx.x < 64 && block * 64 + threadIdx.x < ldv)
        {
            float sum = 0.0f;
#pragma unroll
            for (int k = 0; k < 16; ++k)
                sum += s_o[k][threadIdx.x];
            p.num[(((size_t)ei * p.heads + h) * p.splits + split) * ldv + block * 64 + threadIdx.x] = sum;
        }
    }

    // ---- prompts: gates -------------------------------------------------------------------------
    // A wavefront scans a chunk by itself; the running maximum passes from chunk to chunk by the chunks' totals.
    constexpr int GATE_WAVES = 16;
    template <int LC>
    __global__ void __launch_bounds__(GATE_WAVES * 64)
        memory_gates_kernel(MemoryArgs p)
    {
        __shared__ double s_total[GATE_WAVES], s_top[GATE_WAVES];
        const int h = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, e = p.entry;
        const int r0 = p.row0[e], n = p.ntok[e], slot = p.slot[e];
        float m = p.pos[e] == 0 ? 0.0f : p.m[slot * p.heads + h];
        if (threadIdx.x == 0)
            p.m0[h] = m;
        for (int t0 = 0; t0 < n; t0 += GATE_WAVES * LC)
        {
            const int t = t0 + wave * LC + lane;
            const bool in = lane < LC && t < n;
            float gi = -INFINITY, gf = 0.0f;
            if (in)
                memory_gates(p, p.proj + (size_t)(r0 + t) * p.ldp, h, gi, gf);
            double F = gf;
#pragma unroll
            for (int off = 1; off < 64; off <<= 1)
            {
                const double o = __shfl_up(F, off, 64);
                if (lane >= off)
                    F += o;
            }
            const double a = (double)gi - F;
            double top = in ? a : -INFINITY;
#pragma unroll
            for (int off = 1; off < 64; off <<= 1)
            {
                const double o = __shfl_up(top, off, 64);
                if (lane >= off)
                    top = fmax(top, o);
            }
            __syncthreads();
            if (lane == 63)
            {
                s_total[wave] = F;
                s_top[wave] = top;
            }
            __syncthreads();
            // the running maximum is a 32-bit number of the recurrence
            float mine = m;
            for (int w = 0; w < GATE_WAVES; ++w)
            {
                if (w == wave)
                    mine = m;
                if (t0 + w * LC < n)
                    m = (float)(s_total[w] + fmax((double)m, s_top[w]));
            }
            if (in)
            {
                const float mt = (float)(F + fmax((double)mine, top));
                const size_t at = (size_t)(r0 + t) * p.heads + h;
                p.ga[at] = F - (double)mt;
                p.a[at] = a;
                p.mt[at] = mt;
            }
        }
        if (threadIdx.x == 0)
            p.m[slot * p.heads + h] = m;
    }

    // ---- prompts: products within a chunk ----------------------------------------------------------
    // prod[t][j] = e^(F_t + a_j - m_t) (q_t . k_j) for j <= t, else 0.  Wavefront w: rows 16 w ...  It also leaves
    // its rows of q (scaled) and k as T for the walk over the chunks.
    template <typename T, int LC>
    __global__ void __launch_bounds__(LC * 4)
        memory_product_kernel(MemoryArgs p)
    {
        using O = Operand<T>;
        using V = typename O::V;
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c = lane & 15, g = lane >> 4;
        const int h = blockIdx.y, chunk = blockIdx.x, e = p.entry;
        const int n = p.ntok[e] - chunk * LC < LC ? p.ntok[e] - chunk * LC : LC;
        if (n <= 0)
            return;
        const int r0 = p.row0[e] + chunk * LC;
        auto row = [&](int t) { return p.proj + (size_t)(r0 + (t < n ? t : n - 1)) * p.ldp; };
        const float *q = row(wave * 16 + c) + h * p.dim + 8 * g;
        T *qk = static_cast<T *>(p.qk) + ((size_t)h * p.qk_rows + chunk * LC + wave * 16 + c) * p.dim + 8 * g;
        const size_t k_after = (size_t)p.heads * p.qk_rows * p.dim;
        const float *k[LC / 16];
#pragma unroll
        for (int j = 0; j < LC / 16; ++j)
            k[j] = row(j * 16 + c) + (p.heads + h) * p.dim + 8 * g;
        f32x4 acc[LC / 16];
#pragma unroll
        for (int j = 0; j < LC / 16; ++j)
            acc[j] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        for (int s = 0; s < p.dim; s += 32)
        {
            V a[1], b[1];
            split_pieces<T, 1>(Operand<float>::load(q + s) * p.q_scale, a);
            *reinterpret_cast<V *>(qk + s) = a[0];
#pragma unroll
            for (int j = 0; j < LC / 16; ++j)
                if (j <= wave)
                {
                    split_pieces<T, 1>(Operand<float>::load(k[j] + s), b);
                    acc[j] = O::mma(a[0], b[0], acc[j]);
                    if (j == wave)
                        *reinterpret_cast<V *>(qk + k_after + s) = b[0];
                }
        }
        float *out = p.prod + ((size_t)chunk * p.heads + h) * LC * LC;
#pragma unroll
        for (int j = 0; j < LC / 16; ++j)
        {
            const int tj = j * 16 + c;
            const double aj = p.a[(size_t)(r0 + (tj < n ? tj : n - 1)) * p.heads + h];
#pragma unroll
            for (int r = 0; r < 4; ++r)
            {
                const int t = wave * 16 + 4 * g + r;
                float y = 0.0f;
                if (tj <= t && t < n)
                    y = acc[j][r] * expf((float)(p.ga[(size_t)(r0 + t) * p.heads + h] + aj));
                out[t * LC + tj] = y;
            }
        }
    }

    // ---- prompts: the walk over the chunks ----------------------------------------------------------
    // Workgroup = up to four wavefronts of 16 columns each, of one head.  DT: 16-row tiles of S (dim <= 16 DT); FULL:
    // dim is 16 DT exactly, so that no product hangs on a condition.
    // What the next chunk needs from memory (q and k for the LDS, this column's values, the products) is
    // requested before the matrix work of the current one.
    template <typename T, int LC, int DT, bool FULL>
    __global__ void __launch_bounds__(256)
        memory_chunk_kernel(MemoryArgs p)
    {
        using O = Operand<T>;
        using V = typename O::V;
        typedef T t4 __attribute__((ext_vector_type(4)));
        constexpr int NP = O::PIECES;
        constexpr int LPAD = 16 / sizeof(T);
        constexpr int TPR = 256 / LC;                            // threads of a row when q and k are staged
        constexpr int LOADS = DT * 16 * (int)sizeof(T) / 16 / TPR; // 16-byte pieces of a row per thread
        constexpr bool AHEAD = LOADS <= 8;                       // staged rows of the next chunk fit the registers
        extern __shared__ __attribute__((aligned(16))) char smem[];
        __shared__ float s_carry[LC], s_gate[LC]; // e^(F_t + m0 - m_t), e^(F_end + a_j - m_end)
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c = lane & 15, g = lane >> 4;
        const int h = blockIdx.y, e = p.entry;
        const int ntok = p.ntok[e], slot = p.slot[e], row0 = p.row0[e];
        const int dim = FULL ? 16 * DT : p.dim;
        const int ldv = p.vdim + 16, ld = dim + LPAD;
        const int col = (blockIdx.x * 4 + wave) * 16 + c;
        const bool live = (blockIdx.x * 4 + wave) * 16 < ldv; // of the wavefront
        const bool ones = (blockIdx.x * 4 + wave) * 16 == p.vdim;
        T *sq = reinterpret_cast<T *>(smem), *sk = sq + LC * ld;
        const int dtiles = FULL ? DT : dim >> 4;

        f32x4 S[DT];
        float *state = p.state + ((size_t)slot * p.heads + h) * dim * ldv + (live ? col : 0);
        const bool fresh = p.pos[e] == 0;
#pragma unroll
        for (int t = 0; t < DT; ++t)
        {
            S[t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
            if (t < dtiles && !fresh && live)
            {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    S[t][r] = state[(size_t)(16 * t + 4 * g + r) * ldv];
            }
        }

        const int srow = threadIdx.x / TPR, sseg = threadIdx.x % TPR, pieces = dim * (int)sizeof(T) / 16;
        const T *qrows = static_cast<const T *>(p.qk) + (size_t)h * p.qk_rows * dim;
        const T *krows = qrows + (size_t)p.heads * p.qk_rows * dim;
        u32x4 hq[AHEAD ? LOADS : 1], hk[AHEAD ? LOADS : 1];
        f32x8 hv[LC / 32];
        double h_ga = 0.0, h_a = 0.0, h_end = 0.0;
        float h_mt = 0.0f;
        auto request = [&](int t0) __attribute__((always_inline)) {
            const int n = ntok - t0 < LC ? ntok - t0 : LC;
            const int r0 = row0 + t0;
            if constexpr (AHEAD)
            {
                // (the product kernel wrote whole chunks: rows past the portion repeat its last one)
                const u32x4 *q = reinterpret_cast<const u32x4 *>(qrows + (size_t)(t0 + srow) * dim) + sseg;
                const u32x4 *k = reinterpret_cast<const u32x4 *>(krows + (size_t)(t0 + srow) * dim) + sseg;
#pragma unroll
                for (int i = 0; i < LOADS; ++i)
                {
                    const int at = sseg + i * TPR < pieces ? i * TPR : 0;
                    hq[i] = q[at];
                    hk[i] = k[at];
                }
            }
            const size_t end = (size_t)(r0 + n - 1) * p.heads + h;
            const int t = threadIdx.x & (LC - 1);
            const size_t at = (size_t)(r0 + (t < n ? t : n - 1)) * p.heads + h;
            h_ga = p.ga[at];
            h_a = p.a[at];
            h_end = p.ga[end];
            h_mt = p.mt[end];
#pragma unroll
            for (int s = 0; s < LC / 32; ++s)
#pragma unroll
                for (int j = 0; j < 8; ++j)
                {
                    const int tt = 32 * s + 8 * g + j;
                    hv[s][j] = ones || !live ? 0.0f
                                             : p.proj[(size_t)(r0 + (tt < n ? tt : n - 1)) * p.ldp + (size_t)p.heads * 2 * dim + h * p.vdim + col];
                }
        };
        request(0);
        float m0 = p.m0[h];
        for (int t0 = 0; t0 < ntok; t0 += LC)
        {
            const int n = ntok - t0 < LC ? ntok - t0 : LC;
            const int r0 = row0 + t0;
            const float decay = expf((float)(h_end + (double)m0));
            const float m_end = h_mt;
            __syncthreads();
            if (threadIdx.x < LC)
            {
                const int t = threadIdx.x;
                s_carry[t] = t < n ? expf((float)(h_ga + (double)m0)) : 0.0f;
                s_gate[t] = t < n ? expf((float)(h_end + h_a)) : 0.0f;
            }
            {
                u32x4 *dq = reinterpret_cast<u32x4 *>(sq + srow * ld) + sseg, *dk = reinterpret_cast<u32x4 *>(sk + srow * ld) + sseg;
                if constexpr (AHEAD)
                {
#pragma unroll
                    for (int i = 0; i < LOADS; ++i)
                        if (sseg + i * TPR < pieces)
                        {
                            dq[i * TPR] = hq[i];
                            dk[i * TPR] = hk[i];
                        }
                }
                else
                {
                    const u32x4 *q = reinterpret_cast<const u32x4 *>(qrows + (size_t)(t0 + srow) * dim) + sseg;
                    const u32x4 *k = reinterpret_cast<const u32x4 *>(krows + (size_t)(t0 + srow) * dim) + sseg;
#pragma unroll 4
                    for (int i = 0; sseg + i < pieces; i += TPR)
                    {
                        dq[i] = q[i];
                        dk[i] = k[i];
                    }
                }
            }
            f32x8 x[LC / 32];
#pragma unroll
            for (int s = 0; s < LC / 32; ++s)
                x[s] = hv[s];
            __syncthreads();
            // the chunk's products, 16 rows at a time (a row block needs columns up to its own)
            const float *prod = p.prod + ((size_t)(t0 / LC) * p.heads + h) * LC * LC;
            f32x8 w[LC / 16][LC / 32];
#pragma unroll
            for (int i = 0; i < LC / 16; ++i)
#pragma unroll
                for (int s = 0; s < LC / 32; ++s)
                    if (32 * s <= 16 * i + 15)
                        w[i][s] = Operand<float>::load(prod + (16 * i + c) * LC + 32 * s + 8 * g);
            if (t0 + LC < ntok)
                request(t0 + LC);
            if (live)
            {
                // values of this column, as they are and gated
                V v[LC / 32], gv[LC / 32][NP];
#pragma unroll
                for (int s = 0; s < LC / 32; ++s)
                {
                    if (ones)
                    {
#pragma unroll
                        for (int j = 0; j < 8; ++j)
                            x[s][j] = c == 0 && 32 * s + 8 * g + j < n ? 1.0f : 0.0f;
                    }
                    V one[1];
                    split_pieces<T, 1>(x[s], one);
                    v[s] = one[0];
                    f32x8 y;
#pragma unroll
                    for (int j = 0; j < 8; ++j)
                        y[j] = (float)one[0][j] * s_gate[32 * s + 8 * g + j];
                    split_pieces<T, NP>(y, gv[s]);
                }
                // carried part: q . S
                f32x4 out[LC / 16];
#pragma unroll
                for (int i = 0; i < LC / 16; ++i)
                    out[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
                for (int t = 0; t < DT; t += 2)
                    if (t < dtiles)
                    {
                        V b[NP], a[LC / 16];
                        split_pieces<T, NP>(__builtin_shufflevector(S[t], S[t + 1], 0, 1, 2, 3, 4, 5, 6, 7), b);
#pragma unroll
                        for (int i = 0; i < LC / 16; ++i)
                        {
                            const T *qr = sq + (16 * i + c) * ld + 16 * t + 4 * g;
                            const t4 lo = *reinterpret_cast<const t4 *>(qr), hi = *reinterpret_cast<const t4 *>(qr + 16);
                            a[i] = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
                        }
#pragma unroll
                        for (int k = 0; k < NP; ++k)
#pragma unroll
                            for (int i = 0; i < LC / 16; ++i)
                                out[i] = O::mma(a[i], b[k], out[i]);
                    }
                // plus the chunk's own tokens
#pragma unroll
                for (int i = 0; i < LC / 16; ++i)
                {
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        out[i][r] *= s_carry[16 * i + 4 * g + r];
                }
#pragma unroll
                for (int s = 0; s < LC / 32; ++s)
#pragma unroll
                    for (int i = 0; i < LC / 16; ++i)
                        if (32 * s <= 16 * i + 15)
                        {
                            V q[NP];
                            split_pieces<T, NP>(w[i][s], q);
#pragma unroll
                            for (int k = 0; k < NP; ++k)
                                out[i] = O::mma(q[k], v[s], out[i]);
                        }
#pragma unroll
                for (int i = 0; i < LC / 16; ++i)
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                    {
                        const int t = 16 * i + 4 * g + r;
                        if (t < n)
                            p.num[((size_t)(r0 + t) * p.heads + h) * ldv + col] = out[i][r];
                    }
                // S of the next chunk
#pragma unroll
                for (int t = 0; t < DT; ++t)
                    if (t < dtiles)
                    {
#pragma unroll
                        for (int r = 0; r < 4; ++r)
                            S[t][r] *= decay;
                    }
#pragma unroll
                for (int t = 0; t < DT; t += 4)
                    if (t < dtiles)
                    {
#pragma unroll
                        for (int s = 0; s < LC / 32; ++s)
                        {
                            V k[4];
#pragma unroll
                            for (int u = 0; u < 4; ++u)
                                k[u] = load_columns(sk + 32 * s * ld + 16 * (t + u), ld, lane);
#pragma unroll
                            for (int i = 0; i < NP; ++i)
#pragma unroll
                                for (int u = 0; u < 4; ++u)
                                    S[t + u] = O::mma(k[u], gv[s][i], S[t + u]);
                        }
                    }
            }
            m0 = m_end;
        }
        if (live)
        {
#pragma unroll
            for (int t = 0; t < DT; ++t)
                if (t < dtiles)
                {
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        state[(size_t)(16 * t + 4 * g + r) * ldv] = S[t][r];
                }
        }
    }

    // ---- output: normaliser, head norm, gate ------------------------------------------------------------
    // Workgroup = one head of one row.  DECODE: also the new running maximum of the sequence.
    template <typename T, bool DECODE>
    __global__ void __launch_bounds__(128)
        memory_output_kernel(MemoryArgs p)
    {
        __shared__ float s_sum[2];
        const int h = blockIdx.x;
        const int e = p.entry + (DECODE ? blockIdx.y : 0);
        const int r = DECODE ? p.row0[e] : p.row0[e] + blockIdx.y;
        const float *row = p.proj + (size_t)r * p.ldp;
        const int ldv = p.vdim + 16;
        const int splits = DECODE ? p.splits : 1;
        const float *num = p.num + ((size_t)(DECODE ? blockIdx.y : r) * p.heads + h) * splits * ldv;
        float m;
        if (DECODE)
        {
            float gi, gf;
            memory_gates(p, row, h, gi, gf);
            float *keep = p.m + p.slot[e] * p.heads + h;
            m = fmaxf(gf + (p.pos[e] == 0 ? 0.0f : *keep), gi);
            __syncthreads();
            if (threadIdx.x == 0)
                *keep = m;
        }
        else
            m = p.mt[(size_t)r * p.heads + h];
        // columns 4 threadIdx.x .. + 3, and 512 further on (the first are kept for the second pass)
        auto total = [&](int d) {
            f32x4 o = *reinterpret_cast<const f32x4 *>(num + d);
            for (int k = 1; k < splits; ++k)
                o = o + *reinterpret_cast<const f32x4 *>(num + (size_t)k * ldv + d);
            return o;
        };
        const float inv = 1.0f / (fmaxf(fabsf(total(p.vdim)[0]), expf(-m)) + 1e-6f);
        const int d0 = threadIdx.x * 4;
        f32x4 kept = {0.0f, 0.0f, 0.0f, 0.0f};
        float sum = 0.0f;
        for (int d = d0; d < p.vdim; d += 512)
        {
            const f32x4 o = total(d) * inv;
            if (d == d0)
                kept = o;
            sum += o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3];
        }
        sum = block_sum<128>(sum, s_sum);
        const float scale = 1.0f / sqrtf(sum / (float)p.vdim_real + p.eps);
        const float *gate = row + (size_t)p.heads * (2 * p.dim + p.vdim) + h * p.vdim;
        typedef T t4 __attribute__((ext_vector_type(4)));
        T *y = static_cast<T *>(p.y) + (size_t)r * p.ldy + h * p.vdim;
        for (int d = d0; d < p.vdim; d += 512)
        {
            f32x4 o = (d == d0 ? kept : total(d) * inv) * scale * *reinterpret_cast<const f32x4 *>(p.norm + h * p.vdim + d);
            const f32x4 z = *reinterpret_cast<const f32x4 *>(gate + d);
#pragma unroll
            for (int k = 0; k < 4; ++k)
                o[k] *= sigmoidf(z[k]);
            *reinterpret_cast<t4 *>(y + d) = __builtin_convertvector(o, t4);
        }
    }

    namespace
    {
        constexpr int LC16 = 64, LC32 = 32; // chunk lengths of the two number formats
        constexpr int STEP_SPLIT_ENTRIES = 32; // sequences up to which a decoding step splits the rows of S (in at most 8)

        struct MemoryScratch
        {
            size_t ga, a, mt, m0, prod, num, qk, total;
        };
        MemoryScratch memory_scratch(int rows, int heads, int dim, int vdim)
        {
            MemoryScratch s{};
            size_t at = 0;
            auto take = [&at](size_t bytes) {
                const size_t here = at;
                at += (bytes + 255) & ~(size_t)255;
                return here;
            };
            s.ga = take((size_t)rows * heads * 8);
            s.a = take((size_t)rows * heads * 8);
            s.mt = take((size_t)rows * heads * 4);
            s.m0 = take((size_t)heads * 4);
            s.prod = take((size_t)round_up(rows, LC16) * heads * LC16 * 4);
            const size_t outs = (size_t)(rows > STEP_SPLIT_ENTRIES * 8 ? rows : STEP_SPLIT_ENTRIES * 8);
            s.num = take(outs * heads * (vdim + 16) * 4);
            s.qk = take((size_t)2 * heads * round_up(rows, LC16) * dim * 4);
            s.total = at;
            return s;
        }

        bool memory_args(const char *fn, const llam_seq_memory_args *a, const llam_seq_entries *e, void *d_scratch,
                         int dtype, MemoryArgs &p)
        {
            if (!a || !e || !a->d_proj || !a->d_gate_bias || !a->d_norm || !a->d_state || !a->d_m || !a->d_y || !d_scratch ||
                !e->d_row0 || !e->d_ntok || !e->d_slot || !e->d_pos)
                return fail(fn, "null pointer");
            if (dtype != LLAM_SEQ_BF16 && dtype != LLAM_SEQ_F32)
                return fail(fn, "dtype %d", dtype);
            if (a->heads < 1 || a->heads > 65535 || a->dim < 1 || a->dim > 512 || (a->dim % PAD) != 0 || a->vdim < 1 || (a->vdim % PAD) != 0 ||
                a->vdim_real < 1 || a->vdim_real > a->vdim)
                return fail(fn, "heads=%d dim=%d vdim=%d: dim up to 512, both multiples of %d", a->heads, a->dim, a->vdim, PAD);
            if (a->ldp < a->heads * (2 * a->dim + 2 * a->vdim + 2) || (a->ldp % 4) != 0 || !aligned16(a->d_proj))
                return fail(fn, "ldp=%d too small or rows misaligned", a->ldp);
            if (a->ldy < a->heads * a->vdim || (a->ldy % 8) != 0)
                return fail(fn, "ldy=%d too small or rows misaligned", a->ldy);
            if (!(a->gate_cap > 0.0f))
                return fail(fn, "gate_cap must be positive");
            p = MemoryArgs{};
            p.proj = a->d_proj, p.ldp = a->ldp, p.gate_bias = a->d_gate_bias, p.norm = a->d_norm, p.state = a->d_state;
            p.m = a->d_m, p.y = a->d_y, p.ldy = a->ldy, p.heads = a->heads, p.dim = a->dim, p.vdim = a->vdim, p.vdim_real = a->vdim_real;
            p.q_scale = a->q_scale, p.gate_cap = a->gate_cap, p.eps = a->eps;
            p.row0 = e->d_row0, p.ntok = e->d_ntok, p.slot = e->d_slot, p.pos = e->d_pos;
            return true;
        }
        void place_scratch(MemoryArgs &p, void *d_scratch, size_t scratch_bytes)
        {
            // rows of the step are absolute, so the offsets are those of the whole buffer: the largest
            // row count whose scratch fits
            int rows = 64;
            while (memory_scratch(rows + 64, p.heads, p.dim, p.vdim).total <= scratch_bytes)
                rows += 64;
            const MemoryScratch at = memory_scratch(rows, p.heads, p.dim, p.vdim);
            char *s = static_cast<char *>(d_scratch);
            p.ga = reinterpret_cast<double *>(s + at.ga), p.a = reinterpret_cast<double *>(s + at.a);
            p.mt = reinterpret_cast<float *>(s + at.mt), p.m0 = reinterpret_cast<float *>(s + at.m0);
            p.prod = reinterpret_cast<float *>(s + at.prod), p.num = reinterpret_cast<float *>(s + at.num);
            p.qk = s + at.qk, p.qk_rows = rows;
        }

        template <typename T, int LC, int DT, bool FULL>
        bool chunk_launch_as(const char *fn, const MemoryArgs &p, hipStream_t st)
        {
            static LdsGrant grant;
            const size_t lds = (size_t)2 * LC * (p.dim + 16 / sizeof(T)) * sizeof(T);
            if (lds > 48 * 1024 && allow_lds(grant, reinterpret_cast<const void *>(&memory_chunk_kernel<T, LC, DT, FULL>), 140 * 1024) != hipSuccess)
                return fail(fn, "cannot reserve %zu bytes of LDS", lds);
            hipLaunchKernelGGL((memory_chunk_kernel<T, LC, DT, FULL>), dim3(ceil_div(p.vdim + 16, 64), p.heads), dim3(256), lds, st, p);
            return launched(fn);
        }
        template <typename T, int LC, int DT>
        bool chunk_launch(const char *fn, const MemoryArgs &p, hipStream_t st)
        {
            if constexpr (sizeof(T) == 2)
            {
                if (p.dim == 16 * DT)
                    return chunk_launch_as<T, LC, DT, true>(fn, p, st);
            }
            return chunk_launch_as<T, LC, DT, false>(fn, p, st);
        }
        template <typename T, int LC>
        bool prefill_run(const char *fn, const MemoryArgs &p, int ntok, hipStream_t st)
        {
            hipLaunchKernelGGL(memory_gates_kernel<LC>, dim3(p.heads), dim3(GATE_WAVES * 64), 0, st, p);
            if (!launched(fn))
                return false;
            hipLaunchKernelGGL((memory_product_kernel<T, LC>), dim3(ceil_div(ntok, LC), p.heads), dim3(LC * 4), 0, st, p);
            if (!launched(fn))
                return false;
            const bool ok = p.dim <= 64 ? chunk_launch<T, LC, 4>(fn, p, st) : p.dim <= 128 ? chunk_launch<T, LC, 8>(fn, p, st)
                            : p.dim <= 256 ? chunk_launch<T, LC, 16>(fn, p, st) : chunk_launch<T, LC, 32>(fn, p, st);
            if (!ok)
                return false;
            hipLaunchKernelGGL((memory_output_kernel<T, false>), dim3(p.heads, ntok), dim3(128), 0, st, p);
            return launched(fn);
        }
        template <typename T>
        bool decode_run(const char *fn, MemoryArgs p, int n, hipStream_t st)
        {
            p.splits = n <= STEP_SPLIT_ENTRIES ? p.dim / STEP_ROWS : 1;
            hipLaunchKernelGGL(memory_step_kernel<T>, dim3(ceil_div(p.vdim + 16, 64) * p.splits, p.heads, n), dim3(256), 0, st, p);
            if (!launched(fn))
                return false;
            hipLaunchKernelGGL((memory_output_kernel<T, true>), dim3(p.heads, n), dim3(128), 0, st, p);
            return launched(fn);
        }
    } // namespace
} // namespace llamql

using namespace llamql;

extern "C" size_t llam_seq_memory_scratch_bytes(int max_rows, int heads, int dim, int vdim)
{
    if (max_rows < 1 || heads < 1 || dim < 1 || vdim < 1)
        return 0;
    return memory_scratch(round_up(max_rows, LC16), heads, dim, vdim).total;
}

extern "C" bool llam_seq_memory_decode(const llam_seq_memory_args *a, const llam_seq_entries *e, int first, int n,
                                       void *d_scratch, size_t scratch_bytes, int dtype, int device_id, void *stream)
{
    static const char *fn = "llam_seq_memory_decode";
    MemoryArgs p;
    if (n < 0 || first < 0 || n > 65535)
        return fail(fn, "bad size (first=%d n=%d)", first, n);
    if (n == 0)
        return true;
    if (!memory_args(fn, a, e, d_scratch, dtype, p))
        return false;
    if (llam_seq_memory_scratch_bytes(first + n, p.heads, p.dim, p.vdim) > scratch_bytes)
        return fail(fn, "scratch too small");
    p.entry = first;
    place_scratch(p, d_scratch, scratch_bytes);
    if (!set_device(fn, device_id))
        return false;
    return dtype == LLAM_SEQ_F32 ? decode_run<float>(fn, p, n, as_stream(stream)) : decode_run<bf16>(fn, p, n, as_stream(stream));
}

extern "C" bool llam_seq_memory_prefill(const llam_seq_memory_args *a, const llam_seq_entries *e, int entry, int ntok,
                                        void *d_scratch, size_t scratch_bytes, int dtype, int device_id, void *stream)
{
    static const char *fn = "llam_seq_memory_prefill";
    MemoryArgs p;
    if (ntok < 0 || entry < 0 || ntok > 65535)
        return fail(fn, "bad size (entry=%d ntok=%d)", entry, ntok);
    if (ntok == 0)
        return true;
    if (!memory_args(fn, a, e, d_scratch, dtype, p))
        return false;
    if (llam_seq_memory_scratch_bytes(ntok, p.heads, p.dim, p.vdim) > scratch_bytes)
        return fail(fn, "scratch too small");
    p.entry = entry;
    place_scratch(p, d_scratch, scratch_bytes);
    if (!set_device(fn, device_id))
        return false;
    return dtype == LLAM_SEQ_F32 ? prefill_run<float, LC32>(fn, p, ntok, as_stream(stream))
                                 : prefill_run<bf16, LC16>(fn, p, ntok, as_stream(stream));
}
