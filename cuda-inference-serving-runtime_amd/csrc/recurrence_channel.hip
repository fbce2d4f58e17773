// The gated delta rule with a decay a key channel, per head, over the rows of a step as they come (portions and single
// tokens of several requests), S [R, C] float in the state slot of the row's request:
//
//   S <- diag(g_t) S;  u = beta_t (v_t - S^T k_t);  S <- S + k_t u^T;  o_t = S^T q_t
//
// g_t a decay a head and key channel, beta_t = sigmoid(b_t) one write strength a head, q and k shared by `share` heads.
// The operands (short convolution with silu of q, k, v, unit vectors of q and k,
// decays and gates from their low-rank projections) are one kernel; the recurrence comes in three forms: a scan row by
// row, a step of single rows with the result's norm and gate in it, and for prompt portions a walk chunk by chunk on
// the matrix cores (recurrence_chunk.hip).  All float.
#include "common.h"

#define MAX_TAPS 16

// ------------------------------------------------------------------------------------------------ operands
struct ChannelInputs {
    const float* in; int ld;                   // [q: G R | k: G R | v: H C | ...]; the convolution's inputs of row t
    const float* taps_w; int taps;             // [taps, channels] (taps - 1: the newest input)
    float* conv_state; long long slot_stride;  // [slot][taps - 1][channels], oldest first
    float* qkv;                                // [T, channels]
    const int* seg_of_row; const int* seg_start; const int* state_slots;
    int rows, G, R, H, C;
    float unit_eps;
    // decays: exp(-exp(a_log[h]) softplus(sum_r up_a[h R + c, r] in[t, off_a + r] + dt_bias[h R + c]))
    int off_a, rank_a; const void* up_a; const float* dt_bias; const float* a_log; float* decay;      // [T, H R]
    // gates: sum_r up_g[h C + c, r] in[t, off_g + r]
    int off_g, rank_g; const void* up_g; float* gate;                                                 // [T, H C]
    int ldu_a, ldu_g;                          // row strides of up_a, up_g: the ranks rounded up to 32, the rest zero
    int conv_blocks, row_tiles;                // how the grid divides: conv_blocks, then row_tiles x column blocks
};

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;

// exp(-rate softplus(z)), softplus(z) = max(z, 0) + log(1 + e), e = exp(-|z|); log(1 + e) = log(u) e / (u - 1) with the rounded
// u = 1 + e: the rounding of u cancels, so small e keep their precision.
__device__ __forceinline__ float channel_decay(float z, float rate) {
    const float e = __expf(-fabsf(z)), u = 1.0f + e;
    const float l = u == 1.0f ? e : __logf(u) * e * __builtin_amdgcn_rcpf(u - 1.0f);
    return __expf(-rate * (fmaxf(z, 0.f) + l));
}

// An item of the convolution for the rows t .. t + n - 1 (n <= RB): a q head, a k head (both made unit vectors) or up to 256
// channels of v; four channels a lane.  TAPS > 0: that many taps, the rows' inputs and those before them asked for at
// once (of a single row from the state); rows whose inputs reach back before their segment, and TAPS 0 (any number of taps),
// take them one by one, from the state where they lie before the segment.  SINGLE: every segment has one row, and the lane of a (row, channel)
// moves that channel's state on itself.
template <bool SINGLE, int TAPS>
__device__ __forceinline__ void conv_item(const ChannelInputs& p, int t0, int n_rows, int item, int lane) {
    constexpr int RB = TAPS && !SINGLE ? 8 : 1, BACK = TAPS ? TAPS - 1 : 0, TN = TAPS ? TAPS : 1;
    const int qk = p.G * p.R, inner = p.H * p.C, channels = 2 * qk + inner;
    const bool head = item < 2 * p.G;
    const int first = head ? item * p.R : 2 * qk + (item - 2 * p.G) * 256;
    const int n = head ? p.R : min(256, channels - first);
    int seg[RB], rel[RB];
#pragma unroll
    for (int r = 0; r < RB; ++r) seg[r] = p.seg_of_row[min(t0 + r, p.rows - 1)];
    float x[RB + BACK][4], w[TN][4];
    float* single = nullptr;
    if (TAPS) {
        if (SINGLE) {
            if (seg[0] < 0) return;
            single = p.conv_state + (long long)p.state_slots[seg[0]] * p.slot_stride;
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int ch = first + min(lane + WAVE * i, n - 1);
#pragma unroll
            for (int r = 0; r < RB + BACK; ++r)
                x[r][i] = SINGLE && r < BACK ? single[(size_t)r * channels + ch] : p.in[(size_t)min(max(t0 - BACK + r, 0), p.rows - 1) * p.ld + ch];
#pragma unroll
            for (int j = 0; j < TAPS; ++j) w[j][i] = p.taps_w[(size_t)j * channels + ch];
        }
    }
#pragma unroll
    for (int r = 0; r < RB; ++r) rel[r] = SINGLE || seg[r] < 0 ? 0 : t0 + r - p.seg_start[seg[r]];
#pragma unroll
    for (int r = 0; r < RB; ++r) {
        if (r >= n_rows) break;
        const int t = t0 + r;
        if (seg[r] < 0) continue;
        float y[4] = {0.f, 0.f, 0.f, 0.f}, ss = 0.f;
        if (TAPS && (SINGLE || rel[r] >= BACK)) {
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < TN; ++j) {
                    y[i] += w[j][i] * x[TAPS ? r + j : 0][i];
                    if (SINGLE && j > 0 && lane + WAVE * i < n) single[(size_t)(j - 1) * channels + first + lane + WAVE * i] = x[TAPS ? j : 0][i];
                }
        } else {
            float* st = p.conv_state + (long long)p.state_slots[seg[r]] * p.slot_stride;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int ch = first + lane + WAVE * i;
                if (lane + WAVE * i >= n) continue;
                for (int j = 0; j < p.taps; ++j) {
                    const int src = rel[r] - (p.taps - 1) + j;
                    const float a = src >= 0 ? p.in[(size_t)(t - rel[r] + src) * p.ld + ch] : st[(size_t)(p.taps - 1 + src) * channels + ch];
                    y[i] += p.taps_w[(size_t)j * channels + ch] * a;
                    if (SINGLE && j > 0) st[(size_t)(j - 1) * channels + ch] = a;     // (input j of this row is input j - 1 of the next)
                }
            }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            y[i] = lane + WAVE * i < n ? y[i] / (1.0f + expf(-y[i])) : 0.f;
            ss += y[i] * y[i];
        }
        const float f = head ? 1.0f / sqrtf(wave_sum(ss) + p.unit_eps) : 1.0f;
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (lane + WAVE * i < n) p.qkv[(size_t)t * channels + first + lane + WAVE * i] = y[i] * f;
    }
}

// A block is four waves.  The first conv_blocks blocks: a wave an (item, run of rows) of the convolution.  The others make a
// tile of rows by 256 columns of the decays or of the gates.
//   bf16 matrices: 16 RT rows, on the matrix cores, a wave four tiles of 16 columns; the low-rank coordinates, float,
//   as the sum of two bf16 numbers each (16 bits of mantissa), so two products.
//   float matrices: RT rows, a thread a column, float sums in the order of the coordinates.
#define RANK_CHUNK 64

// A step of single rows runs both parts in one launch (PART 0), others each in a launch of its own (1, 2: two kernels with
// the registers that each needs).
template <int PART, bool SINGLE, int TAPS, int RT, typename TW>
__global__ void __launch_bounds__(256) channel_inputs_kernel(ChannelInputs p) {
    const int inner = p.H * p.C;
    const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
    if (PART == 1 || (PART == 0 && (int)blockIdx.x < p.conv_blocks)) {
        constexpr int RB = TAPS && !SINGLE ? 8 : 1;
        const int per_run = 2 * p.G + (inner + 255) / 256;
        const int work = blockIdx.x * 4 + wave, t0 = work / per_run * RB;
        if (t0 < p.rows) conv_item<SINGLE, TAPS>(p, t0, min(RB, p.rows - t0), work % per_run, lane);
        return;
    }
    if (PART == 1) return;
    const int b = PART == 0 ? blockIdx.x - p.conv_blocks : blockIdx.x, tid = threadIdx.x;
    const int col_block = b / p.row_tiles;
    const int a_cols = p.H * p.R, a_blocks = (a_cols + 255) / 256;
    const bool is_decay = col_block < a_blocks;
    const int cols = is_decay ? a_cols : inner, rank = is_decay ? p.rank_a : p.rank_g, off = is_decay ? p.off_a : p.off_g;
    const int ldu = is_decay ? p.ldu_a : p.ldu_g;
    const TW* up = (const TW*)(is_decay ? p.up_a : p.up_g);
    const int c_first = (is_decay ? col_block : col_block - a_blocks) * 256;
    float* out = is_decay ? p.decay : p.gate;
    if constexpr (sizeof(TW) == 2) {
        const int t0 = (b % p.row_tiles) * 16 * RT, m = lane % 16, kg = lane / 16;
        const int n_tiles = min(4, (cols - c_first - wave * 64 + 15) / 16);           // this wave's tiles of 16 columns
        if (n_tiles <= 0) return;
        f32x4_t acc[4][RT];
#pragma unroll
        for (int c = 0; c < 4; ++c)
#pragma unroll
            for (int j = 0; j < RT; ++j) acc[c][j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (int k0 = 0; k0 < rank; k0 += 32) {
            bf16x8_t hi[RT], lo[RT], wt[4];
            const int k = k0 + kg * 8;
#pragma unroll
            for (int c = 0; c < 4; ++c)
                wt[c] = *(const bf16x8_t*)(up + (size_t)min(c_first + wave * 64 + c * 16 + m, cols - 1) * ldu + k);
#pragma unroll
            for (int j = 0; j < RT; ++j) {
                const float* row = p.in + (size_t)min(t0 + j * 16 + m, p.rows - 1) * p.ld + off + k;
                f32x4_t v[2];                      // (16-byte words; the last one may reach into the row's next columns)
                v[0] = k < rank ? *(const f32x4_t*)row : (f32x4_t){0.f, 0.f, 0.f, 0.f};
                v[1] = k + 4 < rank ? *(const f32x4_t*)(row + 4) : (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const float a = k + e < rank ? v[e / 4][e % 4] : 0.f;
                    const __bf16 h = (__bf16)a;
                    hi[j][e] = h;
                    lo[j][e] = (__bf16)(a - (float)h);
                }
            }
#pragma unroll
            for (int c = 0; c < 4; ++c)
#pragma unroll
                for (int j = 0; j < RT; ++j) {
                    acc[c][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo[j], wt[c], acc[c][j], 0, 0, 0);
                    acc[c][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi[j], wt[c], acc[c][j], 0, 0, 0);
                }
        }
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const int col = c_first + wave * 64 + c * 16 + m;
            if (col >= cols) continue;
            const float bias = is_decay ? p.dt_bias[col] : 0.f, rate = is_decay ? expf(p.a_log[col / p.R]) : 0.f;
#pragma unroll
            for (int j = 0; j < RT; ++j)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int t = t0 + j * 16 + kg * 4 + i;
                    if (t < p.rows) out[(size_t)t * cols + col] = is_decay ? channel_decay(acc[c][j][i] + bias, rate) : acc[c][j][i];
                }
        }
    } else {
        __shared__ __attribute__((aligned(16))) float low[RT][RANK_CHUNK];
        const int t0 = (b % p.row_tiles) * RT, c = c_first + tid, cc = min(c, cols - 1);
        float acc[RT];
#pragma unroll
        for (int j = 0; j < RT; ++j) acc[j] = 0.f;
        for (int r0 = 0; r0 < rank; r0 += RANK_CHUNK) {
            __syncthreads();                                       // (the chunk before is used up)
            for (int i = tid; i < RT * RANK_CHUNK; i += 256) {
                const int j = i / RANK_CHUNK, r = r0 + i % RANK_CHUNK;
                low[j][i % RANK_CHUNK] = r < rank ? p.in[(size_t)min(t0 + j, p.rows - 1) * p.ld + off + r] : 0.f;
            }
            __syncthreads();
            const int m = min(RANK_CHUNK, rank - r0);
            for (int r = 0; r < m; ++r) {
                const float w = load_f32(up + (size_t)cc * ldu + r0 + r);
#pragma unroll
                for (int j = 0; j < RT; ++j) acc[j] += w * low[j][r];
            }
        }
        if (c >= cols) return;
        const float bias = is_decay ? p.dt_bias[c] : 0.f, rate = is_decay ? expf(p.a_log[c / p.R]) : 0.f;
#pragma unroll
        for (int j = 0; j < RT; ++j) {
            if (t0 + j >= p.rows) break;
            out[(size_t)(t0 + j) * cols + c] = is_decay ? channel_decay(acc[j] + bias, rate) : acc[j];
        }
    }
}

// After the convolution has read it: the state becomes the last taps - 1 inputs of (state, portion).
__global__ void __launch_bounds__(256)
channel_conv_state_kernel(const float* __restrict__ in, int ld, float* __restrict__ conv_state, long long slot_stride,
                          const int* __restrict__ seg_start, const int* __restrict__ state_slots, int channels, int taps) {
    const int seg = blockIdx.x, ch = blockIdx.y * 256 + threadIdx.x;
    const int t0 = seg_start[seg], count = seg_start[seg + 1] - t0;
    if (count <= 0 || ch >= channels) return;
    float* st = conv_state + (long long)state_slots[seg] * slot_stride;
    float keep[MAX_TAPS];
#pragma unroll
    for (int i = 0; i < MAX_TAPS; ++i) {
        if (i >= taps - 1) break;
        const int src = count - (taps - 1) + i;
        keep[i] = src >= 0 ? in[(size_t)(t0 + src) * ld + ch] : st[(size_t)(taps - 1 + src) * channels + ch];
    }
#pragma unroll
    for (int i = 0; i < MAX_TAPS; ++i) {
        if (i >= taps - 1) break;
        st[(size_t)i * channels + ch] = keep[i];
    }
}

template <bool SINGLE, int TAPS, typename TW>
static int launch_channel_inputs_of(ChannelInputs& p, hipStream_t stream) {
    const int inner = p.H * p.C, a_cols = p.H * p.R, run = TAPS && !SINGLE ? 8 : 1;
    const long long items = (long long)((p.rows + run - 1) / run) * (2 * p.G + (inner + 255) / 256);
    const int col_blocks = (a_cols + 255) / 256 + (inner + 255) / 256;
    constexpr int unit = sizeof(TW) == 2 ? 16 : 1;                // rows of a step of RT
    const int rt = sizeof(TW) == 2 ? (p.rows > 128 ? 2 : 1) : (p.rows > 16 ? 16 : 1);      // many rows share a column's weights
    p.conv_blocks = (int)((items + 3) / 4);
    p.row_tiles = (p.rows + rt * unit - 1) / (rt * unit);
    const long long tiles = (long long)p.row_tiles * col_blocks;
    if (p.conv_blocks + tiles > 0x7fffffff) return (int)hipErrorInvalidValue;
    constexpr int MANY = sizeof(TW) == 2 ? 2 : 16;
    if (SINGLE) {
        const unsigned blocks = (unsigned)(p.conv_blocks + tiles);
        if (rt == 1) channel_inputs_kernel<0, SINGLE, TAPS, 1, TW><<<blocks, 256, 0, stream>>>(p);
        else channel_inputs_kernel<0, SINGLE, TAPS, MANY, TW><<<blocks, 256, 0, stream>>>(p);
        return CISR_LAUNCH_CHECK();
    }
    channel_inputs_kernel<1, SINGLE, TAPS, 1, TW><<<(unsigned)p.conv_blocks, 256, 0, stream>>>(p);
    const int err = CISR_LAUNCH_CHECK();
    if (err) return err;
    if (rt == 1) channel_inputs_kernel<2, SINGLE, 0, 1, TW><<<(unsigned)tiles, 256, 0, stream>>>(p);
    else channel_inputs_kernel<2, SINGLE, 0, MANY, TW><<<(unsigned)tiles, 256, 0, stream>>>(p);
    return CISR_LAUNCH_CHECK();
}

template <typename TW>
static int launch_channel_inputs(ChannelInputs& p, bool single, hipStream_t stream) {
#define CHANNEL_INPUTS(TAPS) single ? launch_channel_inputs_of<true, TAPS, TW>(p, stream) : launch_channel_inputs_of<false, TAPS, TW>(p, stream)
    if (p.taps == 2) return CHANNEL_INPUTS(2);
    if (p.taps == 3) return CHANNEL_INPUTS(3);
    if (p.taps == 4) return CHANNEL_INPUTS(4);
    return CHANNEL_INPUTS(0);
#undef CHANNEL_INPUTS
}

// up_a [heads * R, ldu_a], up_g [heads * C, ldu_g]: rows of rank_a / rank_g coordinates, then zeros up to ldu; bf16 matrices
// are read in 16-byte words, 32 coordinates a step, so their ldu is a multiple of 32 and they are 16-byte aligned, and so are
// the rows' low-rank coordinates.
extern "C" int cisr_channel_inputs(const float* in, int ld, const float* taps_w, int taps, float* conv_state, long long slot_stride,
                                   float* qkv, const int* seg_of_row, const int* seg_start, const int* state_slots, int rows,
                                   int segments, int kv_heads, int R, int heads, int C, float unit_eps, int off_a, int rank_a,
                                   const void* up_a, int ldu_a, const float* dt_bias, const float* a_log, float* decay, int off_g,
                                   int rank_g, const void* up_g, int ldu_g, float* gate, int single_rows, int weight_dtype, hipStream_t stream) {
    if (rows <= 0 || segments <= 0) return 0;
    const int channels = 2 * kv_heads * R + heads * C;
    if (kv_heads <= 0 || heads <= 0 || R <= 0 || R > 256 || C <= 0 || taps < 1 || taps > MAX_TAPS || rank_a <= 0 || rank_g <= 0 ||
        channels > ld || off_a < 0 || off_a + rank_a > ld || off_g < 0 || off_g + rank_g > ld || segments > 65535 || ldu_a < rank_a ||
        ldu_g < rank_g)
        return (int)hipErrorInvalidValue;
    if (weight_dtype == DT_BF16 && (off_a % 4 || off_g % 4 || ld % 4 || (uintptr_t)in % 16)) return (int)hipErrorInvalidValue;
    if (weight_dtype == DT_BF16 && (ldu_a % 32 || ldu_g % 32 || (uintptr_t)up_a % 16 || (uintptr_t)up_g % 16)) return (int)hipErrorInvalidValue;
    ChannelInputs p{in, ld, taps_w, taps, conv_state, slot_stride, qkv, seg_of_row, seg_start, state_slots, rows, kv_heads, R, heads, C,
                    unit_eps, off_a, rank_a, up_a, dt_bias, a_log, decay, off_g, rank_g, up_g, gate, ldu_a, ldu_g, 0, 0};
    const int err = weight_dtype == DT_F32 ? launch_channel_inputs<float>(p, single_rows, stream) : launch_channel_inputs<bf16_t>(p, single_rows, stream);
    if (err || taps == 1 || single_rows) return err;
    channel_conv_state_kernel<<<dim3(segments, (channels + 255) / 256), 256, 0, stream>>>(in, ld, conv_state, slot_stride, seg_start,
                                                                                       state_slots, channels, taps);
    return CISR_LAUNCH_CHECK();
}

// ------------------------------------------------------------------------------------------------ the scan
struct ChannelScan {
    const float* q; int ldq;          // q[t * ldq + (head / share) * R + r]
    const float* k; int ldk;
    const float* v; int ldv;          // v[t * ldv + head * C + c]
    const float* g; int ldg;          // g[t * ldg + head * R + r]
    const float* b; int ldb;          // b[t * ldb + head], beta = sigmoid(b)
    float* out; int ldo;
    float* state; long long slot_stride;
    const int* seg_start; const int* state_slots;
    int R, C, share, heads;
    float q_scale;
};

template <int CTRL>
__device__ __forceinline__ float lanes_moved(float x) {
    return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), CTRL, 0xF, 0xF, false));
}

// The sum of x over the NG (4, 8 or 16) neighbouring lanes of an aligned group, in every lane of the group, by moves
// inside a row of 16 lanes: neighbours, pairs, the mirror images of a half row and of a row.
template <int NG>
__device__ __forceinline__ float group_sum(float x) {
    x += lanes_moved<0xB1>(x);                   // quad_perm [1, 0, 3, 2]
    x += lanes_moved<0x4E>(x);                   // quad_perm [2, 3, 0, 1]
    if (NG >= 8) x += lanes_moved<0x141>(x);     // row_half_mirror
    if (NG >= 16) x += lanes_moved<0x140>(x);    // row_mirror
    return x;
}

#define CHANNEL_GROUP_OF(RPT) ((RPT) >= 32 ? 4 : 8)

// A wave a (segment, head, tile of COLS = NC 64 / NG columns): columns of S go their own ways.  NG neighbouring lanes
// share NC neighbouring columns, and lane l of them owns the rows l RPT + i, i < RPT, of the state in registers.  Rows
// of a segment are walked in order, GROUP at a time through LDS, the next group's loads in flight while this one is
// walked.  In LDS a lane's RPT coordinates of q, k and g lie side by side (wide reads), the lanes' runs PAD floats apart
// so that the reads of the sixteen lanes of a row fall into different banks.  The results of a group's rows wait in
// registers (lane l of a column's lanes keeps row l's) and are stored together.
template <int NG, int RPT, int NC>
__global__ void __launch_bounds__(64) channel_scan_kernel(ChannelScan p) {
    constexpr int LPG = WAVE / NG, COLS = NC * LPG, GROUP = CHANNEL_GROUP_OF(RPT), RP = NG * RPT;
    constexpr int PAD = RPT >= 4 ? 4 : 2, RUN = RPT + PAD, RPS = NG * RUN;     // floats of a lane's run, of a row in LDS
    constexpr int KEEP = (GROUP + NG - 1) / NG;                                // results a lane keeps a group
    __shared__ __attribute__((aligned(16))) float sq[GROUP * RPS], sk[GROUP * RPS], sg[GROUP * RPS];
    __shared__ float sb[GROUP], sv[GROUP * COLS];
    const int seg = blockIdx.x, head = blockIdx.y, lane = threadIdx.x;
    const int t0 = p.seg_start[seg], t1 = p.seg_start[seg + 1];
    if (t1 <= t0) return;
    const int pair = lane / NG, rg = lane % NG;
    const int c0 = blockIdx.z * COLS + NC * pair;
    const int R = p.R, C = p.C;
    float* state = p.state + (long long)p.state_slots[seg] * p.slot_stride + (size_t)head * R * C;
    float S[NC][RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i)
#pragma unroll
        for (int n = 0; n < NC; ++n)
            S[n][i] = rg * RPT + i < R ? state[(size_t)(rg * RPT + i) * C + min(c0 + n, C - 1)] : 0.f;
    const float* qh = p.q + (size_t)(head / p.share) * R;
    const float* kh = p.k + (size_t)(head / p.share) * R;
    const float* gh = p.g + (size_t)head * R;
    const float* vh = p.v + (size_t)head * C;
    constexpr int PF = GROUP * RP / WAVE, PV = (GROUP * COLS + WAVE - 1) / WAVE;
    static_assert(GROUP * RP % WAVE == 0, "a group's rows divide among the lanes");
    float fq[PF], fk[PF], fg[PF], fv[PV], fb = 0.f;
    auto fetch = [&](int tb) {
        const int last = t1 - 1;
#pragma unroll
        for (int j = 0; j < PF; ++j) {
            const int idx = lane + WAVE * j, tt = idx / RP, r = idx % RP;
            const size_t t = (size_t)min(tb + tt, last);
            const bool in = r < R;
            const int rr = in ? r : 0;
            fk[j] = in ? kh[t * p.ldk + rr] : 0.f;
            fq[j] = in ? qh[t * p.ldq + rr] : 0.f;
            fg[j] = in ? gh[t * p.ldg + rr] : 0.f;
        }
#pragma unroll
        for (int j = 0; j < PV; ++j) {
            const int idx = lane + WAVE * j, tt = min(idx / COLS, GROUP - 1), cc = blockIdx.z * COLS + idx % COLS;
            fv[j] = vh[(size_t)min(tb + tt, last) * p.ldv + min(cc, C - 1)];
        }
        if (lane < GROUP) fb = p.b[(size_t)min(tb + lane, last) * p.ldb + head];
    };
    fetch(t0);
    for (int tb = t0; tb < t1; tb += GROUP) {
        const int n_rows = min(GROUP, t1 - tb);
        __syncthreads();                                   // (the walk before is over: LDS may be written)
#pragma unroll
        for (int j = 0; j < PF; ++j) {
            const int idx = lane + WAVE * j, tt = idx / RP, r = idx % RP, at = tt * RPS + (r / RPT) * RUN + r % RPT;
            sk[at] = fk[j];
            sq[at] = fq[j];
            sg[at] = fg[j];
        }
#pragma unroll
        for (int j = 0; j < PV; ++j)
            if (lane + WAVE * j < GROUP * COLS) sv[lane + WAVE * j] = fv[j];
        if (lane < GROUP) sb[lane] = 1.0f / (1.0f + expf(-fb));
        __syncthreads();
        if (tb + GROUP < t1) fetch(tb + GROUP);
        float keep[KEEP][NC];
#pragma unroll
        for (int tt = 0; tt < GROUP; ++tt) {
            if (tt >= n_rows) break;                       // (uniform over the wave)
            float kc[RPT], qc[RPT];
            const float beta = sb[tt];
            float dot[NC];
#pragma unroll
            for (int n = 0; n < NC; ++n) dot[n] = 0.f;
#pragma unroll
            for (int i = 0; i < RPT; ++i) {
                const float g = sg[tt * RPS + rg * RUN + i];
                kc[i] = sk[tt * RPS + rg * RUN + i];
                qc[i] = sq[tt * RPS + rg * RUN + i];
#pragma unroll
                for (int n = 0; n < NC; ++n) {
                    S[n][i] *= g;
                    dot[n] += S[n][i] * kc[i];
                }
            }
#pragma unroll
            for (int n = 0; n < NC; ++n) {
                const float u = beta * (sv[tt * COLS + NC * pair + n] - group_sum<NG>(dot[n]));
                float o = 0.f;
#pragma unroll
                for (int i = 0; i < RPT; ++i) {
                    S[n][i] += kc[i] * u;
                    o += S[n][i] * qc[i];
                }
                o = group_sum<NG>(o) * p.q_scale;
                keep[tt / NG][n] = rg == tt % NG ? o : (tt % NG ? keep[tt / NG][n] : 0.f);
            }
        }
#pragma unroll
        for (int m = 0; m < KEEP; ++m) {
            const int tt = m * NG + rg;
            if (tt >= n_rows) continue;
            float* o = p.out + (size_t)(tb + tt) * p.ldo + (size_t)head * C;
#pragma unroll
            for (int n = 0; n < NC; ++n)
                if (c0 + n < C) o[c0 + n] = keep[m][n];
        }
    }
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        if (rg * RPT + i >= R) continue;
#pragma unroll
        for (int n = 0; n < NC; ++n)
            if (c0 + n < C) state[(size_t)(rg * RPT + i) * C + c0 + n] = S[n][i];
    }
}

template <int NG, int NC>
static int launch_channel_scan(const ChannelScan& p, int segments, hipStream_t stream) {
    constexpr int COLS = NC * WAVE / NG;
    const int per = (p.R + NG - 1) / NG;                          // rows a lane
    const dim3 grid(segments, p.heads, (p.C + COLS - 1) / COLS);
    if (per <= 2) channel_scan_kernel<NG, 2, NC><<<grid, 64, 0, stream>>>(p);
    else if (per <= 4) channel_scan_kernel<NG, 4, NC><<<grid, 64, 0, stream>>>(p);
    else if (per <= 8) channel_scan_kernel<NG, 8, NC><<<grid, 64, 0, stream>>>(p);
    else if (per <= 16) channel_scan_kernel<NG, 16, NC><<<grid, 64, 0, stream>>>(p);
    else if (per <= 32) {
        // (32 rows of two columns a lane are what the registers hold; 16 lanes a column reach 256 rows with 16 each)
        if constexpr (NG <= 8) channel_scan_kernel<NG, 32, NC><<<grid, 64, 0, stream>>>(p);
        else return (int)hipErrorInvalidValue;
    } else return (int)hipErrorInvalidValue;
    return CISR_LAUNCH_CHECK();
}

// cols: 4, 8, 16 or 32 columns a wave (fewer columns are more waves for the same head, and shorter runs of the state);
// a lane holds at most 32 rows of its columns, so states of more than 128 rows need 16 columns or fewer.
extern "C" int cisr_channel_scan(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* g, int ldg,
                                 const float* b, int ldb, float* out, int ldo, float* state, long long slot_stride,
                                 const int* seg_start, const int* state_slots, int segments, int heads, int R, int C, int share,
                                 float q_scale, int cols, hipStream_t stream) {
    if (segments <= 0 || heads <= 0) return 0;
    if (R <= 0 || C <= 0 || share <= 0 || heads % share || heads > 65535 || (cols != 4 && cols != 8 && cols != 16 && cols != 32) ||
        (C + cols - 1) / cols > 65535 || R > 256)
        return (int)hipErrorInvalidValue;
    ChannelScan p{q, ldq, k, ldk, v, ldv, g, ldg, b, ldb, out, ldo, state, slot_stride, seg_start, state_slots, R, C, share, heads, q_scale};
    if (cols == 4) return launch_channel_scan<16, 1>(p, segments, stream);
    if (cols == 8) return launch_channel_scan<16, 2>(p, segments, stream);
    if (cols == 16) return launch_channel_scan<8, 2>(p, segments, stream);
    return launch_channel_scan<4, 2>(p, segments, stream);
}

// ------------------------------------------------------------------------------------------------ a step of single rows
// One row a segment: a block of 256 threads takes a head's whole state.  A thread owns four neighbouring columns of RPT
// rows (16-byte accesses, runs of a whole row of the state), the 256 / (C / 4) groups of rows meet through LDS for S^T k
// and for S^T q, and the block ends with the head's result, so it norms and gates it too:
// act = o / rms(o) * weight * sigmoid(gate).
struct ChannelStep {
    ChannelScan s;
    const float* gate; int ldgate;    // gate[t * ldgate + head * C + c]
    const float* weight; float eps;   // [C]
    void* act; int ldact;
};

template <int RPT, typename T>
__global__ void __launch_bounds__(256) channel_step_kernel(ChannelStep a) {
    const ChannelScan& p = a.s;
    __shared__ float sk[256], sq[256], sg[256], red[4];
    __shared__ __attribute__((aligned(16))) float4 part[256];
    const int seg = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
    const int t = p.seg_start[seg];
    if (p.seg_start[seg + 1] <= t) return;
    const int R = p.R, C = p.C, quads = C / 4, groups = 256 / quads;
    const int quad = tid % quads, group = tid / quads;
    const bool on = group < groups;                    // (256 need not be a multiple of the quads)
    float4* state = (float4*)(p.state + (long long)p.state_slots[seg] * p.slot_stride + (size_t)head * R * C);
    float4 S[RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = group * RPT + i;
        S[i] = on && r < R ? state[(size_t)r * quads + quad] : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    if (tid < R) {
        sk[tid] = p.k[(size_t)t * p.ldk + (size_t)(head / p.share) * R + tid];
        sq[tid] = p.q[(size_t)t * p.ldq + (size_t)(head / p.share) * R + tid] * p.q_scale;
        sg[tid] = p.g[(size_t)t * p.ldg + (size_t)head * R + tid];
    } else {
        sk[tid] = sq[tid] = sg[tid] = 0.f;
    }
    const float beta = 1.0f / (1.0f + expf(-p.b[(size_t)t * p.ldb + head]));
    const float4 v = tid < quads ? make_float4(p.v[(size_t)t * p.ldv + (size_t)head * C + 4 * tid], p.v[(size_t)t * p.ldv + (size_t)head * C + 4 * tid + 1],
                                               p.v[(size_t)t * p.ldv + (size_t)head * C + 4 * tid + 2], p.v[(size_t)t * p.ldv + (size_t)head * C + 4 * tid + 3])
                                 : make_float4(0.f, 0.f, 0.f, 0.f);
    __syncthreads();
    // the sum of x over the groups, for the quad of this thread if it is one of the first `quads`
    auto meet = [&](float4 x) {
        part[tid] = x;
        __syncthreads();
        float4 sum = make_float4(0.f, 0.f, 0.f, 0.f);
        if (tid < quads)
            for (int g = 0; g < groups; ++g) {
                const float4 y = part[g * quads + tid];
                sum.x += y.x; sum.y += y.y; sum.z += y.z; sum.w += y.w;
            }
        return sum;
    };
    float4 d = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = min(group * RPT + i, 255);
        const float g = sg[r], k = sk[r];
        S[i].x *= g; S[i].y *= g; S[i].z *= g; S[i].w *= g;
        d.x += S[i].x * k; d.y += S[i].y * k; d.z += S[i].z * k; d.w += S[i].w * k;
    }
    d = meet(d);
    __syncthreads();
    if (tid < quads) part[tid] = make_float4(beta * (v.x - d.x), beta * (v.y - d.y), beta * (v.z - d.z), beta * (v.w - d.w));
    __syncthreads();
    const float4 u = part[quad];
    __syncthreads();
    float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = group * RPT + i, rc = min(r, 255);
        const float k = sk[rc], q = sq[rc];
        S[i].x += k * u.x; S[i].y += k * u.y; S[i].z += k * u.z; S[i].w += k * u.w;
        o.x += S[i].x * q; o.y += S[i].y * q; o.z += S[i].z * q; o.w += S[i].w * q;
        if (on && r < R) state[(size_t)r * quads + quad] = S[i];
    }
    o = meet(o);
    const float scale = 1.0f / sqrtf(block_sum<256>(o.x * o.x + o.y * o.y + o.z * o.z + o.w * o.w, red) / (float)C + a.eps);
    if (tid >= quads) return;
    const float* z = a.gate + (size_t)t * a.ldgate + (size_t)head * C + 4 * tid;
    const float* w = a.weight + 4 * tid;
    T* out = (T*)a.act + (size_t)t * a.ldact + (size_t)head * C + 4 * tid;
    store_f32(out, o.x * scale * w[0] / (1.0f + expf(-z[0])));
    store_f32(out + 1, o.y * scale * w[1] / (1.0f + expf(-z[1])));
    store_f32(out + 2, o.z * scale * w[2] / (1.0f + expf(-z[2])));
    store_f32(out + 3, o.w * scale * w[3] / (1.0f + expf(-z[3])));
}

// Rows of the state a thread owns, or 0 if the step kernel does not take these sizes.
static int channel_step_rows(int R, int C, long long slot_stride) {
    if (C % 4 || C < 4 || C > 1024 || R > 256 || slot_stride % 4) return 0;
    const int groups = 256 / (C / 4), per = (R + groups - 1) / groups;
    return per <= 4 ? 4 : per <= 8 ? 8 : per <= 16 ? 16 : per <= 32 ? 32 : 0;
}

extern "C" int cisr_channel_step_ok(int R, int C, long long slot_stride) { return channel_step_rows(R, C, slot_stride) > 0; }

extern "C" int cisr_channel_step(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* g, int ldg,
                                 const float* b, int ldb, float* state, long long slot_stride, const int* seg_start,
                                 const int* state_slots, int segments, int heads, int R, int C, int share, float q_scale,
                                 const float* gate, int ldgate, const float* weight, float eps, void* act, int ldact, int dtype,
                                 hipStream_t stream) {
    if (segments <= 0 || heads <= 0) return 0;
    const int per = channel_step_rows(R, C, slot_stride);
    if (!per || R <= 0 || share <= 0 || heads % share || heads > 65535 || (uintptr_t)state % 16) return (int)hipErrorInvalidValue;
    ChannelStep a{{q, ldq, k, ldk, v, ldv, g, ldg, b, ldb, nullptr, 0, state, slot_stride, seg_start, state_slots, R, C, share, heads, q_scale},
                  gate, ldgate, weight, eps, act, ldact};
    const dim3 grid(segments, heads);
#define CHANNEL_STEP(RPT) \
    if (dtype == DT_F32) channel_step_kernel<RPT, float><<<grid, 256, 0, stream>>>(a); \
    else channel_step_kernel<RPT, bf16_t><<<grid, 256, 0, stream>>>(a)
    if (per == 4) { CHANNEL_STEP(4); }
    else if (per == 8) { CHANNEL_STEP(8); }
    else if (per == 16) { CHANNEL_STEP(16); }
    else { CHANNEL_STEP(32); }
#undef CHANNEL_STEP
    return CISR_LAUNCH_CHECK();
}
