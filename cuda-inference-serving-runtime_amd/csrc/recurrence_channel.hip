// The gated delta rule with a decay a key channel, per head, over the rows of a step as they come (portions and single
// tokens of several requests), S [R, C] float in the state slot of the row's request:
//
//   S <- diag(g_t) S;  u = beta_t (v_t - S^T k_t);  S <- S + k_t u^T;  o_t = S^T q_t
//
// g_t a decay a head and key channel, beta_t = sigmoid(b_t) one write strength a head, q and k shared by `share` heads.
// Two kernels: the operands (short convolution with silu of q, k, v, unit vectors of q and k, decays and gates from
// their low-rank projections) and the scan.  All float.
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
    // decays: exp(-exp(a_log[h]) softplus(sum_r up_a[r, h R + c] in[t, off_a + r] + dt_bias[h R + c]))
    int off_a, rank_a; const void* up_a; const float* dt_bias; const float* a_log; float* decay;      // [T, H R]
    // gates: sum_r up_g[r, h C + c] in[t, off_g + r]
    int off_g, rank_g; const void* up_g; float* gate;                                                 // [T, H C]
    int conv_blocks, row_tiles;                // how the grid divides: conv_blocks, then row_tiles x column blocks
};

#define RANK_CHUNK 64

// A block is four waves.  The first conv_blocks blocks: a wave a (row, item), an item being a q head, a k head (both made
// unit vectors) or up to 256 channels of v.  The others: a tile of RT rows by 256 columns of the decays or of the gates,
// a thread a column, the rows' low-rank coordinates in LDS.  SINGLE: every segment has one row, and the wave of a
// (row, channel) moves that channel's state on itself.
template <bool SINGLE, int RT, typename TW>
__global__ void __launch_bounds__(256) channel_inputs_kernel(ChannelInputs p) {
    const int qk = p.G * p.R, inner = p.H * p.C, channels = 2 * qk + inner;
    if ((int)blockIdx.x < p.conv_blocks) {
        const int v_items = (inner + 255) / 256, per_row = 2 * p.G + v_items;
        const int work = blockIdx.x * 4 + threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
        const int t = work / per_row, item = work % per_row;
        if (t >= p.rows) return;
        const int seg = p.seg_of_row[t];
        if (seg < 0) return;
        const bool head = item < 2 * p.G;
        const int first = head ? item * p.R : 2 * qk + (item - 2 * p.G) * 256;
        const int n = head ? p.R : min(256, channels - first);
        const int rel = t - p.seg_start[seg];
        float* st = p.conv_state + (long long)p.state_slots[seg] * p.slot_stride;
        float y[4], ss = 0.f;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int at = lane + WAVE * i, ch = first + at;
            y[i] = 0.f;
            if (at >= n) continue;
            for (int j = 0; j < p.taps; ++j) {
                const int src = rel - (p.taps - 1) + j;
                const float x = src >= 0 ? p.in[(size_t)(t - rel + src) * p.ld + ch] : st[(size_t)(p.taps - 1 + src) * channels + ch];
                y[i] += p.taps_w[(size_t)j * channels + ch] * x;
                if (SINGLE && j > 0) st[(size_t)(j - 1) * channels + ch] = x;     // (input j of this row is input j - 1 of the next)
            }
            y[i] = y[i] / (1.0f + expf(-y[i]));
            ss += y[i] * y[i];
        }
        const float f = head ? 1.0f / sqrtf(wave_sum(ss) + p.unit_eps) : 1.0f;
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (lane + WAVE * i < n) p.qkv[(size_t)t * channels + first + lane + WAVE * i] = y[i] * f;
        return;
    }
    __shared__ __attribute__((aligned(16))) float low[RT][RANK_CHUNK];
    const int b = blockIdx.x - p.conv_blocks, tid = threadIdx.x;
    const int t0 = (b % p.row_tiles) * RT, col_block = b / p.row_tiles;
    const int a_cols = p.H * p.R, a_blocks = (a_cols + 255) / 256;
    const bool is_decay = col_block < a_blocks;
    const int cols = is_decay ? a_cols : inner, rank = is_decay ? p.rank_a : p.rank_g, off = is_decay ? p.off_a : p.off_g;
    const int c = (is_decay ? col_block : col_block - a_blocks) * 256 + tid, cc = min(c, cols - 1);
    const TW* up = (const TW*)(is_decay ? p.up_a : p.up_g) + cc;
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
        int r = 0;
        for (; r + 8 <= m; r += 8) {
            float w[8];
#pragma unroll
            for (int k = 0; k < 8; ++k) w[k] = load_f32(up + (size_t)(r0 + r + k) * cols);
#pragma unroll
            for (int j = 0; j < RT; ++j)
#pragma unroll
                for (int k = 0; k < 8; ++k) acc[j] += w[k] * low[j][r + k];
        }
        for (; r < m; ++r) {
            const float w = load_f32(up + (size_t)(r0 + r) * cols);
#pragma unroll
            for (int j = 0; j < RT; ++j) acc[j] += w * low[j][r];
        }
    }
    if (c >= cols) return;
    const float bias = is_decay ? p.dt_bias[c] : 0.f, rate = is_decay ? expf(p.a_log[c / p.R]) : 0.f;
#pragma unroll
    for (int j = 0; j < RT; ++j) {
        if (t0 + j >= p.rows) break;
        if (is_decay) {
            const float z = acc[j] + bias;
            const float soft = fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
            p.decay[(size_t)(t0 + j) * cols + c] = expf(-rate * soft);
        } else {
            p.gate[(size_t)(t0 + j) * cols + c] = acc[j];
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

template <bool SINGLE, typename TW>
static int launch_channel_inputs(ChannelInputs& p, hipStream_t stream) {
    const int inner = p.H * p.C, a_cols = p.H * p.R;
    const long long items = (long long)p.rows * (2 * p.G + (inner + 255) / 256);
    const int col_blocks = (a_cols + 255) / 256 + (inner + 255) / 256;
    const int rt = p.rows >= 256 ? 16 : p.rows > 2 ? 4 : 1;       // rows a tile: many rows share a column's weights
    p.conv_blocks = (int)((items + 3) / 4);
    p.row_tiles = (p.rows + rt - 1) / rt;
    const long long blocks = p.conv_blocks + (long long)p.row_tiles * col_blocks;
    if (blocks > 0x7fffffff) return (int)hipErrorInvalidValue;
    if (rt == 16) channel_inputs_kernel<SINGLE, 16, TW><<<(unsigned)blocks, 256, 0, stream>>>(p);
    else if (rt == 4) channel_inputs_kernel<SINGLE, 4, TW><<<(unsigned)blocks, 256, 0, stream>>>(p);
    else channel_inputs_kernel<SINGLE, 1, TW><<<(unsigned)blocks, 256, 0, stream>>>(p);
    return CISR_LAUNCH_CHECK();
}

extern "C" int cisr_channel_inputs(const float* in, int ld, const float* taps_w, int taps, float* conv_state, long long slot_stride,
                                   float* qkv, const int* seg_of_row, const int* seg_start, const int* state_slots, int rows,
                                   int segments, int kv_heads, int R, int heads, int C, float unit_eps, int off_a, int rank_a,
                                   const void* up_a, const float* dt_bias, const float* a_log, float* decay, int off_g, int rank_g,
                                   const void* up_g, float* gate, int single_rows, int weight_dtype, hipStream_t stream) {
    if (rows <= 0 || segments <= 0) return 0;
    const int channels = 2 * kv_heads * R + heads * C;
    if (kv_heads <= 0 || heads <= 0 || R <= 0 || R > 256 || C <= 0 || taps < 1 || taps > MAX_TAPS || rank_a <= 0 || rank_g <= 0 ||
        channels > ld || off_a < 0 || off_a + rank_a > ld || off_g < 0 || off_g + rank_g > ld || segments > 65535)
        return (int)hipErrorInvalidValue;
    ChannelInputs p{in, ld, taps_w, taps, conv_state, slot_stride, qkv, seg_of_row, seg_start, state_slots, rows, kv_heads, R, heads, C,
                    unit_eps, off_a, rank_a, up_a, dt_bias, a_log, decay, off_g, rank_g, up_g, gate, 0, 0};
    if (single_rows)
        return weight_dtype == DT_F32 ? launch_channel_inputs<true, float>(p, stream) : launch_channel_inputs<true, bf16_t>(p, stream);
    const int err = weight_dtype == DT_F32 ? launch_channel_inputs<false, float>(p, stream) : launch_channel_inputs<false, bf16_t>(p, stream);
    if (err || taps == 1) return err;
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
