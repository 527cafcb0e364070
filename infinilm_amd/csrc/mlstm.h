// What the kernels of the mLSTM recurrence share: the rows a launch reads, the gates, the numbering of pieces.
#pragma once
#include "common.h"

#define MC 64              // tokens a chunk of a long segment
#define MW 8               // waves a block of the chunked kernels; a wave owns 16 columns of v
#define MCOLS (16 * MW)    // columns a block

__device__ __forceinline__ float ml_ld(const float* p) { return *p; }
__device__ __forceinline__ float ml_ld(const bf16* p) { return to_f32(*p); }
__device__ __forceinline__ void ml_ld4(const float* p, float* v) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
}
__device__ __forceinline__ void ml_ld4(const bf16* p, float* v) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(t.x << 16); v[1] = __uint_as_float(t.x & 0xffff0000u);
    v[2] = __uint_as_float(t.y << 16); v[3] = __uint_as_float(t.y & 0xffff0000u);
}
__device__ __forceinline__ float ml_any(const void* p, int dt, size_t i) {
    return dt == ILM_DTYPE_F32 ? ((const float*)p)[i] : to_f32(((const bf16*)p)[i]);
}
__device__ __forceinline__ float ml_capped(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float ml_log_sigmoid(float z) { return -(log1pf(expf(-fabsf(z))) + fmaxf(-z, 0.f)); }
__device__ __forceinline__ float ml_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// what a launch knows of its rows
struct MlRows {
    const void* rows;       // [T, stride]
    const void *bias_i, *bias_f;
    const void *norm_w;     // [H dv]
    long stride;
    int i_off, f_off, g_off;    // columns of the raw gates and of the output gate
    int b_dt, w_dt;
    float cap, scale, eps;
};

template <typename T>
__device__ __forceinline__ void ml_raw_gates(const MlRows& a, size_t t, int h, float& zi, float& zf) {
    const T* row = (const T*)a.rows + t * a.stride;
    zi = ml_ld(row + a.i_off + h) + ml_any(a.bias_i, a.b_dt, h);
    zf = ml_ld(row + a.f_off + h) + ml_any(a.bias_f, a.b_dt, h);
}
template <typename T>
__device__ __forceinline__ void ml_gates(const MlRows& a, size_t t, int h, float& li, float& lf) {
    float zi, zf;
    ml_raw_gates<T>(a, t, h, zi, zf);
    li = ml_capped(zi, a.cap);
    lf = ml_log_sigmoid(ml_capped(zf, a.cap));
}

#define ML_CHECK_ROWS(what)                                                                                                            \
    ILM_REQUIRE(R > 0 && R <= 65535 && H > 0 && H <= 65535 && dk > 0 && dv > 0, what ": bad sizes");                                    \
    ILM_REQUIRE(rows_dt == ILM_DTYPE_F32 || rows_dt == ILM_DTYPE_BF16, what ": unknown dtype %d of the rows", rows_dt);                 \
    ILM_REQUIRE(row_stride % 8 == 0 && (((uintptr_t)rows | (uintptr_t)pool) & 15) == 0, what ": rows must be 16-byte aligned");         \
    ILM_REQUIRE(bias_i != nullptr && bias_f != nullptr && norm_w != nullptr, what ": gate biases and the norm's weight are needed");    \
    ILM_REQUIRE(i_off >= 0 && f_off >= 0 && g_off >= 0 && i_off + H <= row_stride && f_off + H <= row_stride                             \
                && (long)g_off + (long)H * dv <= row_stride && (long)H * (2L * dk + dv) <= row_stride, what ": rows of %d are too short", row_stride); \
    ILM_REQUIRE(cap > 0.f, what ": the gates' cap must be positive");                                                                   \
    const MlRows a = {rows, bias_i, bias_f, norm_w, (long)row_stride, i_off, f_off, g_off, b_dt, w_dt, cap, scale, eps}


// the segment whose slots hold slot s (-1: none), its piece p
__device__ __forceinline__ int ml_find(const int* __restrict__ seg_offsets, int R, int piece, int s, int& p) {
    int lo = 0, hi = R - 1;     // the last segment whose first slot is <= s
    while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (seg_offsets[mid] / piece + mid <= s) lo = mid; else hi = mid - 1;
    }
    p = s - (seg_offsets[lo] / piece + lo);
    return (p >= 0 && p * piece < seg_offsets[lo + 1] - seg_offsets[lo]) ? lo : -1;
}

// From the segments' starts and what every piece leaves behind: the state before each piece in the place of the latter, and the
// segments' last states into the pools' rows (mlstm_chunks.hip).  KT: key entries / 16, as the state's tiles lie in the workspace.
int ml_combine(int KT, float4* ws_s, float* ws_n, double* ws_m, float* pool, const float* pool_m, const int* state_in, const int* state_out,
               const int* seg_offsets, int R, int H, int dk, int dv, int CT, int piece, int min_len, hipStream_t stream);

struct MlLaunch {
    void *o, *y;
    MlRows rows;
    float *pool, *pool_m;
    const int *state_in, *state_out, *seg_offsets;
    int R, H, dk, dv, T, min_len, piece, y_stride, y_dt;
    void* ws;
};
// bfloat16 rows, dk <= 128 (mlstm_mfma.hip)
int ml_chunks_bf16(const MlLaunch& l, hipStream_t stream);
long ml_chunks_bf16_ws(int dk, int dv);      // floats a (slot, head) takes; and four floats a (token, head) more
