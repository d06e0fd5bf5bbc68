// Linear layers over tiled bf16 weights, as the launchers inside the library see them.
#pragma once

#include "seq_common.h"
#include "llaminar_amd/seq_api.h"

namespace llamql
{
    struct LinearArgs
    {
        const void *a; // T [M][lda], or fp32 [M][lda] when norm is set
        const void *w;
        void *y;
        const float *bias;
        const float *norm;
        void *h_out;
        float eps;
        int k_real;
        int M, N, K;
        int lda, ldy;
        int out; // LLAM_SEQ_OUT_*
        float limit;
        long a_stride, w_stride, y_stride;
        // rows in groups (routed experts): group z has the rows group_offset[z] .. group_offset[z + 1] - 1
        // of y; row r reads a[row_source ? row_source[r] / source_div : r]
        const int *group_offset;
        const int *row_source;
        int source_div;
    };

    constexpr int SMALL_M = 16;         // most rows of the row-at-a-time kernel: one operand of the matrix unit
    constexpr int NORM_FUSE_MAX = 8192; // most values (rows x columns) every workgroup norms for itself

    __host__ __device__ inline bool is_gated(int out) { return out == LLAM_SEQ_OUT_GATED || out == LLAM_SEQ_OUT_GATED_CLAMP; }
    bool linear_small(const char *fn, const LinearArgs &a, int batch, int dtype, hipStream_t st);
    bool linear_tiled(const char *fn, const LinearArgs &a, int batch, int dtype, hipStream_t st);

    // LLAM_SEQ_OUT_*: four neighbouring output columns of one row
    template <typename T>
    __device__ __forceinline__ void store4(const LinearArgs &p, char *ybase, int row, int col, f32x4 v)
    {
        typedef T t4 __attribute__((ext_vector_type(4)));
        const size_t at = (size_t)row * p.ldy + col;
        switch (p.out)
        {
        case LLAM_SEQ_OUT_F32:
            if (p.bias)
            {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    v[r] += p.bias[col + r];
            }
            *reinterpret_cast<f32x4 *>(reinterpret_cast<float *>(ybase) + at) = v;
            break;
        case LLAM_SEQ_OUT_ADD:
        {
            f32x4 *dst = reinterpret_cast<f32x4 *>(reinterpret_cast<float *>(ybase) + at);
            *dst = *dst + v;
            break;
        }
        case LLAM_SEQ_OUT_RELU2:
#pragma unroll
            for (int r = 0; r < 4; ++r)
            {
                const float z = fmaxf(v[r], 0.0f);
                v[r] = z * z;
            }
            *reinterpret_cast<t4 *>(reinterpret_cast<T *>(ybase) + at) = __builtin_convertvector(v, t4);
            break;
        default:
            *reinterpret_cast<t4 *>(reinterpret_cast<T *>(ybase) + at) = __builtin_convertvector(v, t4);
        }
    }

    __device__ __forceinline__ f32x4 gated4(const LinearArgs &p, f32x4 gate, f32x4 up)
    {
        f32x4 v;
        if (p.out == LLAM_SEQ_OUT_GATED_CLAMP)
        {
#pragma unroll
            for (int r = 0; r < 4; ++r)
            {
                const float a = fminf(gate[r], p.limit), u = fminf(fmaxf(up[r], -p.limit), p.limit);
                v[r] = a * sigmoidf(1.702f * a) * (u + 1.0f);
            }
            return v;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r)
            v[r] = gelu_tanh(gate[r]) * up[r];
        return v;
    }
} // namespace llamql
